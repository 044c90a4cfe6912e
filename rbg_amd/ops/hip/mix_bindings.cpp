// PyTorch bindings for the f32-stream and token-mixer kernels (bf16 or f32
// activations).  Shapes, strides and dtypes are checked here, before launch.
#include "bind_util.h"
#include "embed_bindings.h"
#include "gemm_bindings.h"
#include "glu_bindings.h"
#include "mix_args.h"

extern "C" {
void launch_stream_norm(float*, const void*, const float*, const float*, void*,
                        void*, int, int, int, float, const float*, void*,
                        const int*, const int*, int, int, hipStream_t);
void launch_causal_conv(void*, const void*, const float*, void*, const int*,
                        const int*, const int*, const int*, int, int, int, int,
                        int, hipStream_t);
void launch_tanh_rows(void*, const void*, long, long, int, int, hipStream_t);
void launch_delta_step(const DeltaArgs*, int, int, hipStream_t);
int delta_chunk_tokens();
long delta_chunk_record(int);
void launch_delta_chunk(const DeltaArgs*, const int*, const int*, float*,
                        float*, int, int, long, int, hipStream_t);
}

namespace {

// x += delta; n1, n2 = grouped norms of x under w1, w2 (w2 optional).  With
// conv arguments n1 becomes the convolved mixer input of a decode step.
std::vector<Tensor> stream_norm(Tensor x, OptTensor delta, Tensor w1,
                                OptTensor w2, int64_t groups, double eps,
                                bool f32, OptTensor conv_w,
                                OptTensor conv_state, OptTensor slots,
                                OptTensor positions) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && is_f32(x) && x.is_contiguous(),
              "x must be a contiguous f32 [T, W] stream");
  const int64_t T = x.size(0), W = x.size(1);
  TORCH_CHECK(groups > 0 && W % groups == 0, "groups must divide the width");
  TORCH_CHECK((W + 3 * groups + 16) * 4 <= 65536, "width too large");
  check_f32(w1, "w1", W);
  if (w2) check_f32(*w2, "w2", W);
  auto opts = x.options().dtype(f32 ? torch::kFloat32 : torch::kBFloat16);
  if (delta) {
    check_rows(*delta, "delta");
    TORCH_CHECK(delta->is_contiguous() && delta->size(0) == T &&
                delta->size(1) == W && is_f32(*delta) == f32, "bad delta");
  }
  const float* cw = nullptr;
  void* cs = nullptr;
  const int *sl = nullptr, *po = nullptr;
  int taps = 0;
  if (conv_w) {
    TORCH_CHECK(conv_state && slots && positions, "conv needs its state");
    taps = (int)conv_w->size(0);
    check_f32(*conv_w, "conv_w", taps * W);
    TORCH_CHECK(conv_state->is_contiguous() && conv_state->dim() == 3 &&
                conv_state->size(1) == taps - 1 && conv_state->size(2) == W &&
                is_f32(*conv_state) == f32, "bad conv_state");
    cw = conv_w->data_ptr<float>();
    cs = conv_state->data_ptr();
    sl = i32(*slots, "slots", T);
    po = i32(*positions, "positions", T);
  }
  auto n1 = torch::empty({T, W}, opts);
  Tensor n2;
  if (w2) n2 = torch::empty({T, W}, opts);
  if (T)
    launch_stream_norm(x.data_ptr<float>(),
                       delta ? delta->data_ptr() : nullptr,
                       w1.data_ptr<float>(),
                       w2 ? w2->data_ptr<float>() : nullptr, n1.data_ptr(),
                       w2 ? n2.data_ptr() : nullptr, (int)T, (int)W,
                       (int)groups, (float)eps, cw, cs, sl, po, taps, f32,
                       current_stream());
  return w2 ? std::vector<Tensor>{n1, n2} : std::vector<Tensor>{n1};
}

Tensor causal_conv(Tensor x, Tensor conv_w, Tensor state, Tensor tiles,
                   Tensor cu, Tensor starts, Tensor slots, int64_t tile) {
  check_rows(x, "x");
  const int64_t W = x.size(1), taps = conv_w.size(0);
  TORCH_CHECK(x.is_contiguous() && state.is_contiguous(), "contiguous only");
  same_dtype(x, state, "conv state");
  check_f32(conv_w, "conv_w", taps * W);
  TORCH_CHECK(state.dim() == 3 && state.size(1) == taps - 1 &&
              state.size(2) == W, "bad conv state");
  TORCH_CHECK(tile >= taps - 1, "tile must cover the history");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2, "tiles [n, 2]");
  const int64_t B = slots.numel();
  auto out = torch::empty_like(x);
  if (x.size(0))
    launch_causal_conv(out.data_ptr(), x.data_ptr(), conv_w.data_ptr<float>(),
                       state.data_ptr(), i32(tiles, "tiles", 2),
                       i32(cu, "cu", B + 1), i32(starts, "starts", B),
                       i32(slots, "slots", B), (int)tiles.size(0), (int)tile,
                       (int)W, (int)taps, is_f32(x), current_stream());
  return out;
}

Tensor tanh_rows(Tensor x) {
  check_rows(x, "x");
  auto out = torch::empty({x.size(0), x.size(1)}, x.options());
  if (x.numel())
    launch_tanh_rows(out.data_ptr(), x.data_ptr(), x.stride(0), x.size(0),
                     (int)x.size(1), is_f32(x), current_stream());
  return out;
}

// offs: columns of r, k, v, a, g, low in proj
DeltaArgs delta_args(const Tensor& proj, const OptTensor& z, const Tensor& w2,
                     const Tensor& w0, const Tensor& a_bias,
                     const Tensor& norm_w, const Tensor& state,
                     const Tensor& slots, const OptTensor& cu,
                     const Tensor& starts, const Tensor& out,
                     const std::vector<int64_t>& offs, double decay_scale,
                     double unit_eps, double norm_eps) {
  check_rows(proj, "proj");
  check_rows(out, "out");
  same_dtype(proj, out, "delta");
  TORCH_CHECK(state.dim() == 4 && state.is_cuda() && is_f32(state) &&
              state.is_contiguous() && state.size(2) == state.size(3),
              "state must be f32 [slots, heads, dim, dim]");
  const int64_t H = state.size(1), D = state.size(2), HD = H * D;
  TORCH_CHECK(D <= 256, "head dim above 256");
  TORCH_CHECK(w2.dim() == 2 && w2.is_contiguous() && w2.size(0) == HD,
              "w2 must be [heads*dim, rank]");
  same_dtype(proj, w2, "delta w2");
  const int64_t rank = w2.size(1), rows = proj.size(0), B = slots.numel();
  TORCH_CHECK(rank <= 4096, "decay rank above 4096");
  check_f32(w0, "w0", HD);
  check_f32(a_bias, "a_bias", HD);
  check_f32(norm_w, "norm_w", HD);
  TORCH_CHECK(out.size(0) == rows && out.size(1) == HD, "out shape");
  TORCH_CHECK(offs.size() == 6, "six column offsets");
  for (int i = 0; i < 6; ++i)
    TORCH_CHECK(offs[i] >= 0 &&
                offs[i] + (i < 5 ? HD : rank) <= proj.size(1),
                "column offset outside proj");
  if (z) {
    check_rows(*z, "z");
    same_dtype(proj, *z, "delta z");
    TORCH_CHECK(z->is_contiguous() && z->size(0) == rows && z->size(1) == HD,
                "z shape");
  }
  if (!cu) TORCH_CHECK(B == rows, "one row per sequence without cu");
  DeltaArgs p{};
  p.proj = proj.data_ptr();
  p.z = z ? z->data_ptr() : nullptr;
  p.w2 = w2.data_ptr();
  p.w0 = w0.data_ptr<float>();
  p.a_bias = a_bias.data_ptr<float>();
  p.norm_w = norm_w.data_ptr<float>();
  p.state = state.data_ptr<float>();
  p.slots = i32(slots, "slots", B);
  p.cu = cu ? i32(*cu, "cu", B + 1) : nullptr;
  p.starts = i32(starts, "starts", B);
  p.out = out.data_ptr();
  p.proj_stride = proj.stride(0);
  p.out_stride = out.stride(0);
  p.off_r = (int)offs[0]; p.off_k = (int)offs[1]; p.off_v = (int)offs[2];
  p.off_a = (int)offs[3]; p.off_g = (int)offs[4]; p.off_low = (int)offs[5];
  p.heads = (int)H; p.dim = (int)D; p.rank = (int)rank;
  p.decay_scale = (float)decay_scale;
  p.unit_eps = (float)unit_eps;
  p.norm_eps = (float)norm_eps;
  return p;
}

void delta_step(Tensor proj, OptTensor z, Tensor w2, Tensor w0, Tensor a_bias,
                Tensor norm_w, Tensor state, Tensor slots, OptTensor cu,
                Tensor starts, Tensor out, std::vector<int64_t> offs,
                double decay_scale, double unit_eps, double norm_eps) {
  const DeltaArgs p = delta_args(proj, z, w2, w0, a_bias, norm_w, state, slots,
                                 cu, starts, out, offs, decay_scale, unit_eps,
                                 norm_eps);
  if (slots.numel() && proj.size(0))
    launch_delta_step(&p, (int)slots.numel(), is_f32(proj), current_stream());
}

// The same over rows of several tokens per sequence, 16 at a time; tiles
// [n, 2] = (sequence, first token) and chunk_cu [B+1] number the chunks.
void delta_chunk(Tensor proj, Tensor z, Tensor w2, Tensor w0, Tensor a_bias,
                 Tensor norm_w, Tensor state, Tensor slots, Tensor cu,
                 Tensor starts, Tensor out, std::vector<int64_t> offs,
                 double decay_scale, double unit_eps, double norm_eps,
                 Tensor tiles, Tensor chunk_cu) {
  const DeltaArgs p = delta_args(proj, z, w2, w0, a_bias, norm_w, state, slots,
                                 cu, starts, out, offs, decay_scale, unit_eps,
                                 norm_eps);
  TORCH_CHECK(p.dim <= 128 && decay_scale * delta_chunk_tokens() <= 60.0,
              "delta_chunk: head dim or decay out of range");
  const int64_t B = slots.numel(), rows = proj.size(0);
  if (!B || !rows) return;
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2, "tiles [n, 2]");
  const int64_t n = tiles.size(0);
  auto f32 = proj.options().dtype(torch::kFloat32);
  auto ws = torch::empty({n * p.heads * delta_chunk_record(p.dim)}, f32);
  auto o = torch::empty({rows, (int64_t)p.heads * p.dim}, f32);
  launch_delta_chunk(&p, i32(tiles, "tiles", 2 * n),
                     i32(chunk_cu, "chunk_cu", B + 1), ws.data_ptr<float>(),
                     o.data_ptr<float>(), (int)n, (int)B, rows, is_f32(proj),
                     current_stream());
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("embed_stream", &embed_stream, "f32 stream = embed[token] * scale");
  m.def("stream_norm", &stream_norm,
        "stream += delta; grouped RMS norms (+ decode input convolution)");
  m.def("causal_conv", &causal_conv, "x + causal depthwise conv, varlen");
  m.def("gelu_mul", &gelu_mul, "gelu_tanh(gate) * up");
  m.def("tanh_rows", &tanh_rows, "tanh of a column slice");
  m.def("delta_step", &delta_step, "generalized delta rule, token by token");
  m.def("delta_chunk", &delta_chunk, "generalized delta rule, by chunks");
  m.attr("DELTA_CHUNK") = delta_chunk_tokens();
  m.def("skinny_gemm", &skinny_gemm, "decode-shape GEMM (M<=128)",
        py::arg("a"), py::arg("w"), py::arg("force_splits") = 0);
}
