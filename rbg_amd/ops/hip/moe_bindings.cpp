// PyTorch bindings for sandwich norms, paged attention and sparse experts (bf16
// or f32 activations).  Shapes, strides and dtypes are checked here, before
// launch.
#include "bind_util.h"
#include "gemm_bindings.h"
#include "moe_args.h"

extern "C" {
void launch_embed_pairs(float*, const void*, const void*, const long*,
                        const long*, long, long, long, int, int, int,
                        hipStream_t);
int sandwich_max_width(int);
void launch_sandwich_norm(float*, const void*, const int*, const float*, int,
                          const float*, const float*, void*, int, int, float,
                          int, hipStream_t);
void launch_rope_paged(const RopePagedArgs*, int, int, hipStream_t);
int paged_block_rows();
void launch_paged_prefill(const PagedAttnArgs*, hipStream_t);
void launch_paged_decode(const PagedAttnArgs*, hipStream_t);
void launch_paged_rows(const PagedAttnArgs*, int, hipStream_t);
}

namespace {

const long* i64(const Tensor& t, const char* name, int64_t numel) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kInt64 &&
              t.is_contiguous() && t.numel() == numel, name,
              " must be contiguous int64 on GPU, one per token");
  return (const long*)t.data_ptr<int64_t>();
}

Tensor embed_pairs(Tensor tokens, Tensor prev, Tensor table, Tensor pairs,
                   int64_t mul_prev, int64_t mul_cur) {
  check_rows(table, "table");
  check_rows(pairs, "pairs");
  same_dtype(table, pairs, "pairs");
  TORCH_CHECK(table.is_contiguous() && pairs.is_contiguous() &&
              pairs.size(1) == table.size(1) && pairs.size(0) >= 2,
              "tables must be contiguous and equally wide");
  TORCH_CHECK(mul_prev >= 0 && mul_cur >= 0, "multipliers must not be negative");
  const int64_t T = tokens.numel(), W = table.size(1);
  auto x = torch::empty({T, W}, table.options().dtype(torch::kFloat32));
  if (T)
    launch_embed_pairs(x.data_ptr<float>(), table.data_ptr(), pairs.data_ptr(),
                       i64(tokens, "tokens", T), i64(prev, "prev", T),
                       mul_prev, mul_cur, pairs.size(0) - 1, (int)T, (int)W,
                       is_f32(table), current_stream());
  return x;
}

OptTensor sandwich_norm(Tensor x, OptTensor y, OptTensor inv,
                        OptTensor weights, OptTensor wb, OptTensor w,
                        double eps, bool f32) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && is_f32(x) && x.is_contiguous(),
              "x must be a contiguous f32 [T, W] stream");
  const int64_t T = x.size(0), W = x.size(1);
  TORCH_CHECK(W <= sandwich_max_width((int)W), "width too large");
  const int* ip = nullptr;
  const float* wp = nullptr;
  int top = 1;
  if (y) {
    check_rows(*y, "y");
    TORCH_CHECK(y->is_contiguous() && y->size(1) == W && is_f32(*y) == f32,
                "y must be contiguous rows of the stream's width");
    TORCH_CHECK(wb, "y needs its norm's weight");
    check_f32(*wb, "wb", W);
    if (inv) {
      TORCH_CHECK(weights, "inv needs weights");
      check_experts(*y, *inv, *weights, T);
      ip = i32(*inv, "inv", weights->numel());
      wp = weights->data_ptr<float>();
      top = (int)weights->size(1);
    } else {
      TORCH_CHECK(y->size(0) == T, "one row of y per token");
    }
  }
  if (w) check_f32(*w, "w", W);
  OptTensor out;
  if (w)
    out = torch::empty({T, W}, x.options().dtype(
        f32 ? torch::kFloat32 : torch::kBFloat16));
  if (T && (y || w))
    launch_sandwich_norm(x.data_ptr<float>(), y ? y->data_ptr() : nullptr, ip,
                         wp, top, y ? wb->data_ptr<float>() : nullptr,
                         w ? w->data_ptr<float>() : nullptr,
                         w ? out->data_ptr() : nullptr, (int)T, (int)W,
                         (float)eps, f32, current_stream());
  return out;
}

// k, v: [pages, kv_heads, page_size, size]
void check_pages(const Tensor& k, const Tensor& v, const Tensor& like) {
  for (const auto& t : {k, v})
    TORCH_CHECK(t.is_cuda() && t.dim() == 4 && t.is_contiguous(),
                "pages must be contiguous [pages, heads, rows, size]");
  same_dtype(k, like, "key pages");
  same_dtype(v, like, "value pages");
  TORCH_CHECK(k.size(0) == v.size(0) && k.size(1) == v.size(1) &&
              k.size(2) == v.size(2), "key and value pages differ");
}

// offs: columns of q, k, v, or of q alone (nothing is stored then)
void rope_store_paged(Tensor proj, OptTensor bias, OptTensor cos_sin,
                      Tensor positions, Tensor slots, int64_t heads,
                      int64_t dim, Tensor k, Tensor v,
                      std::vector<int64_t> offs) {
  check_rows(proj, "proj");
  check_pages(k, v, proj);
  const int64_t T = proj.size(0), N = proj.size(1);
  if (bias) check_f32(*bias, "bias", N);
  if (cos_sin) {
    TORCH_CHECK(cos_sin->dim() == 2 && cos_sin->size(1) % 2 == 0 &&
                cos_sin->size(1) <= dim, "cos_sin [positions, rotated dims]");
    check_f32(*cos_sin, "cos_sin", cos_sin->numel());
  }
  TORCH_CHECK(k.size(3) == dim, "key size");
  TORCH_CHECK(offs.size() == 1 || offs.size() == 3, "columns of q or q, k, v");
  const int64_t G = k.size(1), DV = v.size(3);
  TORCH_CHECK(offs[0] >= 0 && offs[0] + heads * dim <= N, "q columns");
  RopePagedArgs p{};
  if (offs.size() == 3) {
    TORCH_CHECK(offs[1] >= 0 && offs[1] + G * dim <= N && offs[2] >= 0 &&
                offs[2] + G * DV <= N, "k or v columns");
    p.k = k.data_ptr();
    p.v = v.data_ptr();
    p.off_k = (int)offs[1];
    p.off_v = (int)offs[2];
  }
  p.proj = proj.data_ptr();
  p.bias = bias ? bias->data_ptr<float>() : nullptr;
  p.cos_sin = cos_sin ? cos_sin->data_ptr<float>() : nullptr;
  p.positions = i32(positions, "positions", T);
  p.slots = i32(slots, "slots", T);
  p.stride = proj.stride(0);
  p.off_q = (int)offs[0];
  // queries that neither shift nor turn stay as they are
  p.rows = (int)T; p.heads = bias || cos_sin ? (int)heads : 0;
  p.kv_heads = (int)G;
  p.d = (int)dim; p.dv = (int)DV;
  p.rot = cos_sin ? (int)cos_sin->size(1) : 0;
  p.page_size = (int)k.size(2);
  p.table_rows = cos_sin ? (int)cos_sin->size(0) : 0;
  const bool vec = mult8({dim, DV, p.rot / 2, p.stride, p.off_q, p.off_k,
                          p.off_v}) && aligned(proj, 16) && aligned(k, 16) &&
                   aligned(v, 16);
  if (T && (p.heads || p.k)) launch_rope_paged(&p, is_f32(proj), vec, current_stream());
}

// fields that prompts and decode share; returns whether the matrix-core forms
// take the sizes
bool paged_args(PagedAttnArgs& p, const Tensor& q, const Tensor& k,
                const Tensor& v, const Tensor& tables, const Tensor& out,
                double scale, double softcap, bool sink, int64_t window,
                const OptTensor& lam, double out_scale, double out_eps) {
  check_heads(q, "q");
  check_pages(k, v, q);
  check_rows(out, "out");
  same_dtype(q, out, "attn out");
  const int64_t M = lam ? 2 : 1;
  const int64_t R = q.size(0), H = q.size(1), D = q.size(2) / M,
                DV = v.size(3);
  const int64_t G = k.size(1), PS = k.size(2);
  TORCH_CHECK(k.size(3) == q.size(2) && q.size(2) % M == 0 && G > 0 &&
              H % G == 0, "key heads or size");
  TORCH_CHECK(window >= 0 && window < (1ll << 31), "window");
  if (lam) check_f32(*lam, "lam", 1);
  TORCH_CHECK(out.size(0) == R && out.size(1) == H * DV, "out shape");
  TORCH_CHECK(D <= 1024 && DV <= 1024, "head size above 1024");
  TORCH_CHECK(tables.dim() == 2, "tables [seqs, pages]");
  p.q = q.data_ptr(); p.k = k.data_ptr(); p.v = v.data_ptr();
  p.out = out.data_ptr();
  p.tables = i32(tables, "tables", 1);
  p.q_row = q.stride(0); p.q_head = q.stride(1); p.o_row = out.stride(0);
  p.rows = (int)R; p.heads = (int)H; p.kv_heads = (int)G;
  p.d = (int)D; p.dv = (int)DV;
  p.page_size = (int)PS; p.max_pages = (int)tables.size(1);
  while ((1 << (p.page_shift + 1)) <= PS) ++p.page_shift;
  p.splits = 1;
  p.scale = (float)scale; p.softcap = (float)softcap; p.sink = sink;
  p.window = (int)window; p.maps = (int)M;
  p.lam = lam ? lam->data_ptr<float>() : nullptr;
  p.out_scale = (float)out_scale; p.out_eps = (float)out_eps;
  return !is_f32(q) && D * M <= 256 && DV <= 256 && PS % 16 == 0 &&
         (1 << p.page_shift) == PS && mult8({D, DV, p.q_row, p.q_head}) &&
         p.o_row % 4 == 0 && aligned(q, 16) && aligned(k, 16) &&
         aligned(v, 16) && aligned(out, 8);
}

void paged_prefill(Tensor q, Tensor k, Tensor v, Tensor tables,
                   Tensor seq_info, Tensor row_info, Tensor blocks, Tensor out,
                   double scale, double softcap, bool sink, int64_t window,
                   OptTensor lam, double out_scale, double out_eps) {
  PagedAttnArgs p{};
  const bool tiled = paged_args(p, q, k, v, tables, out, scale, softcap, sink,
                                window, lam, out_scale, out_eps);
  if (!p.rows) return;
  if (tiled) {
    TORCH_CHECK(paged_block_rows() == 128, "block size");
    TORCH_CHECK(blocks.dim() == 2 && blocks.size(1) == 2 &&
                seq_info.dim() == 2 && seq_info.size(1) == 3 &&
                seq_info.size(0) == tables.size(0), "blocks, seq_info shapes");
    p.blocks = i32(blocks, "blocks", 2);
    p.seq_info = i32(seq_info, "seq_info", 3);
    p.n_blocks = (int)blocks.size(0);
    launch_paged_prefill(&p, current_stream());
  } else {
    p.row_info = i32(row_info, "row_info", 2 * q.size(0));
    launch_paged_rows(&p, is_f32(q), current_stream());
  }
}

void paged_decode(Tensor q, Tensor k, Tensor v, Tensor tables, Tensor ctx,
                  Tensor out, double scale, double softcap, bool sink,
                  int64_t window, OptTensor lam, double out_scale,
                  double out_eps, int64_t splits) {
  PagedAttnArgs p{};
  const bool tiled = paged_args(p, q, k, v, tables, out, scale, softcap, sink,
                                window, lam, out_scale, out_eps);
  TORCH_CHECK(tables.size(0) == q.size(0), "one table per row");
  if (!p.rows) return;
  p.ctx = i32(ctx, "ctx", p.rows);
  if (!tiled) {
    launch_paged_rows(&p, is_f32(q), current_stream());
    return;
  }
  p.splits = (int)(splits < 1 ? 1 : splits > 64 ? 64 : splits);
  Tensor po, pml;
  if (p.splits > 1 || p.maps > 1) {
    auto f32 = q.options().dtype(torch::kFloat32);
    po = torch::empty({p.splits, p.rows, p.heads * p.maps, p.dv}, f32);
    pml = torch::empty({p.splits, p.rows, p.heads * p.maps, 2}, f32);
    p.part_o = po.data_ptr<float>();
    p.part_ml = pml.data_ptr<float>();
  }
  launch_paged_decode(&p, current_stream());
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("embed_pairs", &embed_pairs, "token row + hashed pair row, f32");
  m.def("sandwich_norm", &sandwich_norm,
        "stream += norm(branch or weighed experts); norm of the stream");
  m.def("rope_store_paged", &rope_store_paged,
        "biases, rotary positions, paged store of keys and values");
  m.def("paged_prefill", &paged_prefill, "varlen attention over pages");
  m.def("paged_decode", &paged_decode, "one query per sequence over pages");
  m.def("skinny_gemm", &skinny_gemm, "decode-shape GEMM (M<=128)",
        py::arg("a"), py::arg("w"), py::arg("force_splits") = 0);
}
