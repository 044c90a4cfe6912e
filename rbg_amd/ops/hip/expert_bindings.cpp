// PyTorch bindings for mixtures of experts (bf16 or f32 activations).  Shapes,
// strides and dtypes are checked here, before launch.
#include "bind_util.h"
#include "expert_args.h"

extern "C" {
void launch_moe_combine(void*, const void*, const int*, const float*, int, int,
                        int, int, hipStream_t);
void launch_router_logits(float*, const void*, const void*, int, int, int, int,
                          int, hipStream_t);
int moe_max_experts();
int moe_route_blocks(int);
void launch_moe_route(const MoeRouteArgs*, hipStream_t);
void launch_moe_gemm(const MoeGemmArgs*, int, int, hipStream_t);
}

namespace {

Tensor moe_combine(Tensor y, Tensor inv, Tensor weights) {
  check_rows(y, "y");
  TORCH_CHECK(y.is_contiguous(), "y must be contiguous");
  const int64_t T = weights.size(0);
  check_experts(y, inv, weights, T);
  auto out = torch::empty({T, y.size(1)}, y.options());
  if (T)
    launch_moe_combine(out.data_ptr(), y.data_ptr(),
                       i32(inv, "inv", weights.numel()),
                       weights.data_ptr<float>(), (int)weights.size(1), (int)T,
                       (int)y.size(1), is_f32(y), current_stream());
  return out;
}

Tensor router_logits(Tensor x, Tensor w) {
  check_rows(x, "x");
  check_rows(w, "router");
  same_dtype(x, w, "router");
  TORCH_CHECK(x.is_contiguous() && w.is_contiguous() && x.size(1) == w.size(1),
              "x [T, K], router [E, K]");
  const int64_t T = x.size(0), E = w.size(0), K = x.size(1);
  auto out = torch::empty({T, E}, x.options().dtype(torch::kFloat32));
  const bool vec = !is_f32(x) && K % 8 == 0 && aligned(x, 16) && aligned(w, 16);
  if (T)
    launch_router_logits(out.data_ptr<float>(), x.data_ptr(), w.data_ptr(),
                         (int)T, (int)E, (int)K, is_f32(x), vec,
                         current_stream());
  return out;
}

int64_t most_tiles(int64_t pairs, int64_t experts, int64_t tile) {
  return std::min(pairs, experts) + pairs / tile;
}

// weights [T, top], inv, rows [T * top], tiles [most, 3], count [1]; the last
// `identity` of the experts return their input and get no rows
std::vector<Tensor> moe_route(Tensor logits, Tensor correction, int64_t groups,
                              int64_t keep, int64_t top, int64_t tile,
                              int64_t mode, int64_t identity, double scale) {
  TORCH_CHECK(logits.dim() == 2, "logits [T, E]");
  const int64_t T = logits.size(0), E = logits.size(1), P = T * top;
  check_f32(logits, "logits", T * E);
  check_f32(correction, "correction", E);
  TORCH_CHECK(E <= moe_max_experts(), "too many experts");
  TORCH_CHECK(groups > 0 && E % groups == 0 && keep > 0 && keep <= groups &&
              top > 0 && top <= keep * (E / groups) && tile > 0,
              "groups, keep or top out of range");
  TORCH_CHECK(mode >= ROUTE_SIGMOID && mode <= ROUTE_SHARE, "route mode");
  TORCH_CHECK(identity >= 0 && identity < E, "identity experts");
  const int64_t real = E - identity;
  auto i = logits.options().dtype(torch::kInt32);
  auto weights = torch::empty({T, top}, logits.options());
  auto ids = torch::empty({T, top}, i), inv = torch::empty({P}, i),
       rows = torch::empty({P}, i),
       tiles = torch::empty({most_tiles(P, real, tile), 3}, i),
       count = torch::empty({1}, i);
  MoeRouteArgs p{};
  p.logits = logits.data_ptr<float>();
  p.correction = correction.data_ptr<float>();
  p.weights = weights.data_ptr<float>();
  p.ids = ids.data_ptr<int>(); p.inv = inv.data_ptr<int>();
  p.rows = rows.data_ptr<int>(); p.tiles = tiles.data_ptr<int>();
  p.count = count.data_ptr<int>();
  const int blocks = moe_route_blocks((int)T);
  Tensor part;
  if (blocks) {
    part = torch::empty({blocks, E}, i);
    p.part = part.data_ptr<int>();
  }
  p.tokens = (int)T; p.experts = (int)E; p.groups = (int)groups;
  p.keep = (int)keep; p.top = (int)top; p.tile = (int)tile;
  p.real = (int)real; p.mode = (int)mode; p.scale = (float)scale;
  if (T) launch_moe_route(&p, current_stream());
  return {weights, inv, rows, tiles, count};
}

Tensor expert_linear(Tensor x, Tensor w, OptTensor rows, Tensor tiles,
                     Tensor count, int64_t pairs, int64_t tile, int64_t act,
                     double limit) {
  check_rows(x, "x");
  TORCH_CHECK(w.is_cuda() && w.dim() == 3 && w.is_contiguous() &&
              x.is_contiguous(), "w [E, N, K] and x must be contiguous");
  same_dtype(x, w, "expert weights");
  const int64_t E = w.size(0), N = w.size(1), K = w.size(2);
  TORCH_CHECK(x.size(1) == K, "K mismatch");
  TORCH_CHECK(rows || x.size(0) == pairs, "one row of x per pair");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 3 &&
              tiles.size(0) == most_tiles(pairs, E, tile), "tiles shape");
  TORCH_CHECK(act >= EXPERT_NONE && act <= EXPERT_CLAMPED_GLU, "activation");
  const bool glu = act >= EXPERT_SILU_GLU;
  TORCH_CHECK(!glu || N % 4 == 0, "gate and up rows");
  auto out = torch::empty({pairs, glu ? N / 2 : N}, x.options());
  MoeGemmArgs p{};
  p.x = x.data_ptr(); p.w = w.data_ptr(); p.out = out.data_ptr();
  p.rows = rows ? i32(*rows, "rows", pairs) : nullptr;
  p.tiles = i32(tiles, "tiles", 0);
  p.count = i32(count, "count", 1);
  p.max_tiles = (int)tiles.size(0); p.tile = (int)tile;
  p.n = (int)N; p.k = (int)K;
  p.act = (int)act; p.limit = (float)limit;
  const bool vec = !is_f32(x) && mult8({N, K}) && aligned(x, 16) &&
                   aligned(w, 16);
  TORCH_CHECK(tile <= (vec ? 128 : 16), "tile too large for these sizes");
  TORCH_CHECK(p.max_tiles <= 65535, "too many tiles");
  // the tiled form counts bytes of x and of one expert's weights in 32 bits
  TORCH_CHECK(x.numel() < (1ll << 31) && N * K < (1ll << 31), "x or w too large");
  if (pairs) launch_moe_gemm(&p, is_f32(x), vec, current_stream());
  return out;
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("moe_combine", &moe_combine, "weighed sums of expert rows");
  m.def("router_logits", &router_logits, "x W^T with f32 sums and result");
  m.def("moe_route", &moe_route, "choice of experts and pairs by expert");
  m.def("expert_linear", &expert_linear, "grouped products by expert");
  m.attr("ROUTE_SIGMOID") = (int)ROUTE_SIGMOID;
  m.attr("ROUTE_CHOSEN") = (int)ROUTE_CHOSEN;
  m.attr("ROUTE_SHARE") = (int)ROUTE_SHARE;
  m.attr("EXPERT_NONE") = (int)EXPERT_NONE;
  m.attr("EXPERT_RELU2") = (int)EXPERT_RELU2;
  m.attr("EXPERT_SILU_GLU") = (int)EXPERT_SILU_GLU;
  m.attr("EXPERT_CLAMPED_GLU") = (int)EXPERT_CLAMPED_GLU;
}
