// PyTorch bindings for latent attention (bf16 or f32 activations).  Shapes,
// strides and dtypes are checked here, before launch.
#include "bind_util.h"
#include "latent_args.h"

extern "C" {
void launch_latent_store(void*, void*, const void*, long, const float*,
                         const int*, int, int, float, int, hipStream_t);
void launch_attn_rows(const AttnRowsArgs*, int, hipStream_t);
int window_attn_rows();
void launch_window_attn(const WindowAttnArgs*, hipStream_t);
void launch_latent_decode(const LatentDecodeArgs*, hipStream_t);
void launch_head_linear(const HeadLinearArgs*, int, int, hipStream_t);
}

namespace {

Tensor latent_store(Tensor x, Tensor w, Tensor cache, Tensor slots,
                    double eps) {
  check_rows(x, "x");
  const int64_t T = x.size(0), R = x.size(1);
  same_dtype(x, cache, "latent cache");
  TORCH_CHECK(cache.is_cuda() && cache.is_contiguous() && cache.dim() == 3 &&
              cache.size(2) == R, "cache must be [pages, page_size, rank]");
  check_f32(w, "w", R);
  auto c = torch::empty({T, R}, x.options());
  if (T)
    launch_latent_store(c.data_ptr(), cache.data_ptr(), x.data_ptr(),
                        x.stride(0), w.data_ptr<float>(),
                        i32(slots, "slots", T), (int)T, (int)R, (float)eps,
                        is_f32(x), current_stream());
  return c;
}

// q [rows, H, D], k [keys, H, D], v [keys, H, Dv] (any row/head strides);
// out [rows, H*Dv] (row stride free), times sigmoid(gate) when given.
// row_info locates each query, seq_info/blocks each 128-row block of them.
void window_attention(Tensor q, Tensor k, Tensor v, OptTensor gate, Tensor out,
                      Tensor row_info, Tensor seq_info, Tensor blocks,
                      double scale, int64_t window) {
  check_heads(q, "q"); check_heads(k, "k"); check_heads(v, "v");
  check_rows(out, "out");
  same_dtype(q, k, "attn k"); same_dtype(q, v, "attn v");
  same_dtype(q, out, "attn out");
  const int64_t R = q.size(0), H = q.size(1), D = q.size(2), DV = v.size(2);
  TORCH_CHECK(k.size(1) == H && k.size(2) == D && v.size(1) == H &&
              v.size(0) == k.size(0), "k/v shapes");
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
      mult8({D, DV, q.stride(0), q.stride(1), k.stride(0), k.stride(1),
             v.stride(0), v.stride(1), g_row}) && out.stride(0) % 4 == 0 &&
      aligned(q, 16) && aligned(k, 16) && aligned(v, 16) && aligned(out, 8) &&
      (!gate || aligned(*gate, 8));
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
  p.q_row = q.stride(0); p.q_head = q.stride(1);
  p.k_row = k.stride(0); p.k_head = k.stride(1);
  p.v_row = v.stride(0); p.v_head = v.stride(1);
  p.o_row = out.stride(0); p.o_head = DV;
  p.rows = (int)R; p.heads = (int)H; p.d = (int)D; p.dv = (int)DV;
  p.window = (int)window; p.scale = (float)scale;
  launch_attn_rows(&p, is_f32(q), current_stream());
}

// q [rows, H, rank] absorbed queries over the paged latents; out the same
Tensor latent_decode(Tensor q, Tensor cache, Tensor tables, Tensor ctx,
                     double scale, int64_t window, int64_t splits) {
  check_heads(q, "q");
  same_dtype(q, cache, "latent cache");
  const int64_t R = q.size(0), H = q.size(1), K = q.size(2);
  TORCH_CHECK(cache.is_cuda() && cache.dim() == 3 && cache.is_contiguous() &&
              cache.size(2) == K, "cache must be [pages, page_size, rank]");
  TORCH_CHECK(K <= 1024, "rank above 1024");
  TORCH_CHECK(tables.dim() == 2 && tables.size(0) == R, "tables [rows, pages]");
  auto out = torch::empty({R, H, K}, q.options());
  if (!R) return out;
  if (!is_f32(q) && K <= 512 && cache.size(1) % 16 == 0 &&
      mult8({K, q.stride(0), q.stride(1)}) && aligned(q, 16) &&
      aligned(cache, 16)) {
    LatentDecodeArgs p{};
    p.q = q.data_ptr(); p.cache = cache.data_ptr(); p.out = out.data_ptr();
    p.tables = i32(tables, "tables", 1);
    p.ctx = i32(ctx, "ctx", R);
    p.q_row = q.stride(0); p.q_head = q.stride(1);
    p.seqs = (int)R; p.heads = (int)H; p.rank = (int)K;
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
  p.tables = i32(tables, "tables", 1);
  p.ctx = i32(ctx, "ctx", R);
  p.q_row = q.stride(0); p.q_head = q.stride(1);
  p.k_row = K; p.v_row = K;
  p.o_row = H * K; p.o_head = K;
  p.rows = (int)R; p.heads = (int)H; p.d = (int)K; p.dv = (int)K;
  p.window = (int)window; p.page_size = (int)cache.size(1);
  p.max_pages = (int)tables.size(1); p.scale = (float)scale;
  launch_attn_rows(&p, is_f32(q), current_stream());
  return out;
}

// out[s, h*n + j] = sum_k x[s, h, k] w[h, j, k] (times sigmoid(gate)); out is
// given as rows, and may be a column slice
void head_linear(Tensor x, Tensor w, OptTensor gate, Tensor out) {
  check_heads(x, "x");
  check_rows(out, "out");
  same_dtype(x, w, "head_linear w");
  same_dtype(x, out, "head_linear out");
  TORCH_CHECK(w.is_cuda() && w.dim() == 3 && w.is_contiguous(), "w [H, n, k]");
  const int64_t R = x.size(0), H = x.size(1), K = x.size(2), N = w.size(1);
  TORCH_CHECK(w.size(0) == H && w.size(2) == K && out.size(0) == R &&
              out.size(1) == H * N, "head_linear shapes");
  HeadLinearArgs p{};
  if (gate) {
    check_rows(*gate, "gate");
    same_dtype(x, *gate, "head_linear gate");
    TORCH_CHECK(gate->size(0) == R && gate->size(1) == H * N, "gate shape");
    p.gate = gate->data_ptr();
    p.g_row = gate->stride(0);
  }
  p.x = x.data_ptr(); p.w = w.data_ptr(); p.out = out.data_ptr();
  p.x_row = x.stride(0); p.x_head = x.stride(1); p.o_row = out.stride(0);
  p.rows = (int)R; p.heads = (int)H; p.n = (int)N; p.k = (int)K;
  p.pack = N % 4 == 0 && p.o_row % 4 == 0 && aligned(out, 8) &&
           (!gate || (p.g_row % 4 == 0 && aligned(*gate, 8)));
  const bool vec = mult8({K, p.x_row, p.x_head}) && aligned(x, 16) &&
                   aligned(w, 16);
  if (R) launch_head_linear(&p, is_f32(x), vec, current_stream());
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("latent_store", &latent_store, "normed latent into the paged pool");
  m.def("window_attention", &window_attention, "varlen window attention");
  m.def("head_linear", &head_linear, "per-head linear maps, decode shapes");
  m.def("latent_decode", &latent_decode,
        "absorbed decode attention over paged latents");
}
