// PyTorch bindings for latent attention (bf16 or f32 activations).  Shapes,
// strides and dtypes are checked here, before launch.
#include "bind_util.h"
#include "latent_args.h"

extern "C" {
void launch_latent_store(const LatentStoreArgs*, int, int, hipStream_t);
void launch_rotate(const RotateArgs*, int, int, hipStream_t);
int latent_decode_fits(int, int);
void launch_attn_rows(const AttnRowsArgs*, int, hipStream_t);
int window_attn_rows();
void launch_window_attn(const WindowAttnArgs*, hipStream_t);
void launch_latent_decode(const LatentDecodeArgs*, hipStream_t);
void launch_head_linear(const HeadLinearArgs*, int, int, hipStream_t);
}

namespace {

// table [positions, dims] = [cos | sin]
RotaryArgs rotary_args(const OptTensor& table, const OptTensor& positions,
                       bool interleaved, int64_t rows) {
  RotaryArgs r{};
  if (!table) return r;
  TORCH_CHECK(positions, "rotation needs positions");
  TORCH_CHECK(table->dim() == 2 && table->size(0) > 0 &&
              table->size(1) % 2 == 0, "table [positions, rotated dims]");
  check_f32(*table, "table", table->numel());
  r.cos_sin = table->data_ptr<float>();
  r.positions = i32(*positions, "positions", rows);
  r.dims = (int)table->size(1);
  r.interleaved = interleaved;
  r.table_rows = (int)table->size(0);
  return r;
}

void check_sink(const OptTensor& sink, int64_t heads) {
  if (sink) check_f32(*sink, "sink", heads);
}

// x [T, rank + rotated dims]; returns what the cache got, and the norm of x2
// under w2
std::vector<Tensor> latent_store(Tensor x, Tensor w, Tensor cache,
                                 Tensor slots, double eps, OptTensor table,
                                 OptTensor positions, bool interleaved,
                                 OptTensor x2, OptTensor w2) {
  check_rows(x, "x");
  const int64_t T = x.size(0), N = x.size(1);
  LatentStoreArgs p{};
  p.rot = rotary_args(table, positions, interleaved, T);
  const int64_t R = N - p.rot.dims;
  TORCH_CHECK(R > 0, "no latent columns");
  same_dtype(x, cache, "latent cache");
  TORCH_CHECK(cache.is_cuda() && cache.is_contiguous() && cache.dim() == 3 &&
              cache.size(2) == N, "cache must be [pages, page_size, columns]");
  check_f32(w, "w", R);
  auto c = torch::empty({T, N}, x.options());
  std::vector<Tensor> out{c};
  bool vec = mult8({R, N, x.stride(0)}) && aligned(x, 16) &&
             aligned(cache, 16) && aligned(w, 16);
  p.x = x.data_ptr(); p.w = w.data_ptr<float>(); p.c = c.data_ptr();
  p.cache = cache.data_ptr(); p.slots = i32(slots, "slots", T);
  p.x_row = x.stride(0);
  if (x2) {
    check_rows(*x2, "x2");
    same_dtype(x, *x2, "second latent");
    TORCH_CHECK(x2->size(0) == T && w2, "rows or weight of x2");
    const int64_t R2 = x2->size(1);
    check_f32(*w2, "w2", R2);
    out.push_back(torch::empty({T, R2}, x.options()));
    p.x2 = x2->data_ptr(); p.w2 = w2->data_ptr<float>();
    p.c2 = out[1].data_ptr();
    p.x2_row = x2->stride(0);
    p.rank2 = (int)R2;
    vec = vec && mult8({R2, x2->stride(0)}) && aligned(*x2, 16) &&
          aligned(*w2, 16);
  }
  p.rows = (int)T; p.rank = (int)R; p.eps = (float)eps;
  if (T) launch_latent_store(&p, is_f32(x), vec, current_stream());
  return out;
}

// x [T, H, dims], rotated in place
void rotate_rows(Tensor x, Tensor table, Tensor positions, bool interleaved) {
  check_heads(x, "x");
  TORCH_CHECK(x.scalar_type() == torch::kBFloat16 || is_f32(x),
              "x must be bf16 or f32");
  RotateArgs p{};
  p.rot = rotary_args(table, positions, interleaved, x.size(0));
  TORCH_CHECK(x.size(2) == p.rot.dims, "x has ", x.size(2), " dims, not ",
              p.rot.dims);
  p.x = x.data_ptr();
  p.x_row = x.stride(0); p.x_head = x.stride(1);
  p.rows = (int)x.size(0); p.heads = (int)x.size(1);
  const bool vec = !is_f32(x) && aligned(x, 16) && aligned(table, 16) &&
                   mult8({p.x_row, p.x_head}) &&
                   p.rot.dims % (interleaved ? 8 : 16) == 0;
  if (x.numel()) launch_rotate(&p, is_f32(x), vec, current_stream());
}

// q [rows, H, D], k [keys, H, D], v [keys, H, Dv] (any row/head strides);
// out [rows, H*Dv] (row stride free), times sigmoid(gate) when given.
// row_info locates each query, seq_info/blocks each 128-row block of them.  k2
// [keys, D2]: the last D2 of q's dims meet it instead of k; sink [H].
void window_attention(Tensor q, Tensor k, Tensor v, OptTensor gate, Tensor out,
                      Tensor row_info, Tensor seq_info, Tensor blocks,
                      double scale, int64_t window, OptTensor k2,
                      OptTensor sink) {
  check_heads(q, "q"); check_heads(k, "k"); check_heads(v, "v");
  check_rows(out, "out");
  same_dtype(q, k, "attn k"); same_dtype(q, v, "attn v");
  same_dtype(q, out, "attn out");
  const int64_t R = q.size(0), H = q.size(1), D = q.size(2), DV = v.size(2);
  const int64_t D1 = k.size(2);
  if (k2) {
    check_rows(*k2, "k2");
    same_dtype(q, *k2, "attn k2");
    TORCH_CHECK(k2->size(0) == k.size(0), "k2 rows");
  }
  TORCH_CHECK(k.size(1) == H && v.size(1) == H && v.size(0) == k.size(0) &&
              D1 + (k2 ? k2->size(1) : 0) == D, "k/v shapes");
  check_sink(sink, H);
  const int64_t k2_row = k2 ? k2->stride(0) : 0;
  TORCH_CHECK(out.size(0) == R && out.size(1) == H * DV, "out shape");
  TORCH_CHECK(D <= 1024 && DV <= 1024, "head size above 1024");
  if (gate) {
    check_rows(*gate, "gate");
    same_dtype(q, *gate, "attn gate");
    TORCH_CHECK(gate->size(0) == R && gate->size(1) == H * DV, "gate shape");
  }
  if (!R) return;
  const int64_t g_row = gate ? gate->stride(0) : 0;
  const bool tiled =
      !is_f32(q) && D <= 256 && DV <= 256 &&
      mult8({D, D1, DV, q.stride(0), q.stride(1), k.stride(0), k.stride(1),
             k2_row, v.stride(0), v.stride(1), g_row}) && out.stride(0) % 4 == 0 &&
      aligned(q, 16) && aligned(k, 16) && aligned(v, 16) && aligned(out, 8) &&
      (!gate || aligned(*gate, 8)) && (!k2 || aligned(*k2, 16));
  if (tiled) {
    TORCH_CHECK(window_attn_rows() == 128, "block size");
    TORCH_CHECK(blocks.dim() == 2 && blocks.size(1) == 2, "blocks [n, 2]");
    WindowAttnArgs p{};
    p.q = q.data_ptr(); p.k = k.data_ptr(); p.v = v.data_ptr();
    p.gate = gate ? gate->data_ptr() : nullptr;
    p.out = out.data_ptr();
    p.blocks = i32(blocks, "blocks", 2);
    p.seq_info = i32(seq_info, "seq_info", 4);
    p.q_row = q.stride(0); p.q_head = q.stride(1);
    p.k_row = k.stride(0); p.k_head = k.stride(1);
    p.v_row = v.stride(0); p.v_head = v.stride(1);
    p.k2 = k2 ? k2->data_ptr() : nullptr;
    p.sink = sink ? sink->data_ptr<float>() : nullptr;
    p.k2_row = k2_row; p.d1 = (int)D1;
    p.g_row = g_row; p.o_row = out.stride(0);
    p.n_blocks = (int)blocks.size(0); p.heads = (int)H;
    p.d = (int)D; p.dv = (int)DV;
    p.window = (int)window; p.scale = (float)scale;
    launch_window_attn(&p, current_stream());
    return;
  }
  AttnRowsArgs p{};
  p.gate = gate ? gate->data_ptr() : nullptr;
  p.g_row = g_row;
  p.q = q.data_ptr(); p.k = k.data_ptr(); p.v = v.data_ptr();
  p.out = out.data_ptr();
  p.row_info = i32(row_info, "row_info", 2 * R);
  p.k2 = k2 ? k2->data_ptr() : nullptr;
  p.sink = sink ? sink->data_ptr<float>() : nullptr;
  p.k2_row = k2_row; p.d1 = (int)D1;
  p.q_row = q.stride(0); p.q_head = q.stride(1);
  p.k_row = k.stride(0); p.k_head = k.stride(1);
  p.v_row = v.stride(0); p.v_head = v.stride(1);
  p.o_row = out.stride(0); p.o_head = DV;
  p.rows = (int)R; p.heads = (int)H; p.d = (int)D; p.dv = (int)DV;
  p.window = (int)window; p.scale = (float)scale;
  launch_attn_rows(&p, is_f32(q), current_stream());
}

// q [rows, H, D] absorbed queries over the paged latents [.., D], whose first
// `rank` columns are the value; out [rows, H, rank]; sink [H]
Tensor latent_decode(Tensor q, Tensor cache, Tensor tables, Tensor ctx,
                     double scale, int64_t window, int64_t splits,
                     int64_t rank, OptTensor sink) {
  check_heads(q, "q");
  same_dtype(q, cache, "latent cache");
  const int64_t R = q.size(0), H = q.size(1), D = q.size(2), K = rank;
  TORCH_CHECK(cache.is_cuda() && cache.dim() == 3 && cache.is_contiguous() &&
              cache.size(2) == D, "cache must be [pages, page_size, columns]");
  TORCH_CHECK(K > 0 && K <= D && D <= 2048 && K <= 1024, "latent sizes");
  TORCH_CHECK(tables.dim() == 2 && tables.size(0) == R, "tables [rows, pages]");
  check_sink(sink, H);
  auto out = torch::empty({R, H, K}, q.options());
  if (!R) return out;
  if (!is_f32(q) && latent_decode_fits((int)D, (int)K) &&
      cache.size(1) % 16 == 0 && mult8({D, K, q.stride(0), q.stride(1)}) &&
      aligned(q, 16) && aligned(cache, 16)) {
    LatentDecodeArgs p{};
    p.q = q.data_ptr(); p.cache = cache.data_ptr(); p.out = out.data_ptr();
    p.sink = sink ? sink->data_ptr<float>() : nullptr;
    p.tables = i32(tables, "tables", 1);
    p.ctx = i32(ctx, "ctx", R);
    p.q_row = q.stride(0); p.q_head = q.stride(1);
    p.seqs = (int)R; p.heads = (int)H; p.d = (int)D; p.rank = (int)K;
    p.window = (int)window; p.page_size = (int)cache.size(1);
    p.max_pages = (int)tables.size(1); p.scale = (float)scale;
    p.splits = (int)(splits < 1 ? 1 : splits > 64 ? 64 : splits);
    Tensor po, pml;
    if (p.splits > 1) {
      auto f32 = q.options().dtype(torch::kFloat32);
      po = torch::empty({p.splits, R, H, K}, f32);
      pml = torch::empty({p.splits, R, H, 2}, f32);
      p.part_o = po.data_ptr<float>();
      p.part_ml = pml.data_ptr<float>();
    }
    launch_latent_decode(&p, current_stream());
    return out;
  }
  AttnRowsArgs p{};
  p.q = q.data_ptr(); p.k = cache.data_ptr(); p.v = cache.data_ptr();
  p.out = out.data_ptr();
  p.sink = sink ? sink->data_ptr<float>() : nullptr;
  p.tables = i32(tables, "tables", 1);
  p.ctx = i32(ctx, "ctx", R);
  p.q_row = q.stride(0); p.q_head = q.stride(1);
  p.k_row = D; p.v_row = D;
  p.o_row = H * K; p.o_head = K;
  p.rows = (int)R; p.heads = (int)H; p.d = p.d1 = (int)D; p.dv = (int)K;
  p.window = (int)window; p.page_size = (int)cache.size(1);
  p.max_pages = (int)tables.size(1); p.scale = (float)scale;
  launch_attn_rows(&p, is_f32(q), current_stream());
  return out;
}

// out[s, h, j] = sum_k x[s, h, k] w[h, j, k] (times sigmoid(gate)); out
// [rows, H, n] may be a slice.  With a tail [rows, H, dims] out is dims longer
// per head and ends in its rotation.
void head_linear(Tensor x, Tensor w, OptTensor gate, Tensor out,
                 OptTensor tail, OptTensor table, OptTensor positions,
                 bool interleaved) {
  check_heads(x, "x");
  check_heads(out, "out");
  same_dtype(x, w, "head_linear w");
  same_dtype(x, out, "head_linear out");
  TORCH_CHECK(w.is_cuda() && w.dim() == 3 && w.is_contiguous(), "w [H, n, k]");
  const int64_t R = x.size(0), H = x.size(1), K = x.size(2), N = w.size(1);
  HeadLinearArgs p{};
  p.rot = rotary_args(table, positions, interleaved, R);
  TORCH_CHECK(w.size(0) == H && w.size(2) == K && out.size(0) == R &&
              out.size(1) == H && out.size(2) == N + p.rot.dims,
              "head_linear shapes");
  TORCH_CHECK(tail.has_value() == (p.rot.dims > 0), "a tail and its rotation");
  if (tail) {
    check_heads(*tail, "tail");
    same_dtype(x, *tail, "tail");
    TORCH_CHECK(tail->size(0) == R && tail->size(1) == H &&
                tail->size(2) == p.rot.dims, "tail shape");
    p.tail = tail->data_ptr();
    p.t_row = tail->stride(0); p.t_head = tail->stride(1);
  }
  if (gate) {
    check_rows(*gate, "gate");
    same_dtype(x, *gate, "head_linear gate");
    TORCH_CHECK(gate->size(0) == R && gate->size(1) == H * N, "gate shape");
    p.gate = gate->data_ptr();
    p.g_row = gate->stride(0);
  }
  p.x = x.data_ptr(); p.w = w.data_ptr(); p.out = out.data_ptr();
  p.x_row = x.stride(0); p.x_head = x.stride(1);
  p.o_row = out.stride(0); p.o_head = out.stride(1);
  p.rows = (int)R; p.heads = (int)H; p.n = (int)N; p.k = (int)K;
  p.pack = N % 4 == 0 && p.o_row % 4 == 0 && p.o_head % 4 == 0 &&
           aligned(out, 8) &&
           (!gate || (p.g_row % 4 == 0 && aligned(*gate, 8)));
  p.tail_vec = tail && !is_f32(x) && aligned(*tail, 16) && aligned(out, 16) &&
               aligned(*table, 16) &&
               mult8({N, p.t_row, p.t_head, p.o_row, p.o_head}) &&
               p.rot.dims % (interleaved ? 8 : 16) == 0;
  const bool vec = mult8({K, p.x_row, p.x_head}) && aligned(x, 16) &&
                   aligned(w, 16);
  if (R) launch_head_linear(&p, is_f32(x), vec, current_stream());
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("latent_store", &latent_store,
        "normed latent and rotated key part into the paged pool");
  m.def("rotate_rows", &rotate_rows, "rotary positions, in place");
  m.def("window_attention", &window_attention, "varlen window attention");
  m.def("head_linear", &head_linear, "per-head linear maps, decode shapes");
  m.def("latent_decode", &latent_decode,
        "absorbed decode attention over paged latents");
}
