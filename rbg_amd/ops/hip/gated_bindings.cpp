// PyTorch bindings for the gated delta rule, its short convolution, gated norms
// and gated linear units (bf16 or f32 activations).  Shapes, strides and dtypes
// are checked here, before launch.
#include "bind_util.h"
#include "embed_bindings.h"
#include "gated_args.h"
#include "gemm_bindings.h"
#include "glu_bindings.h"

extern "C" {
int gate_norm_max_width(int);
void launch_gate_norm(const GateNormArgs*, int, int, hipStream_t);
void launch_short_conv(const ShortConvArgs*, int, int, hipStream_t);
void launch_gated_step(const GatedDeltaArgs*, int, int, hipStream_t);
int gated_chunk_tokens();
int gated_chunk_max_dim();
long gated_chunk_record(int);
void launch_gated_chunk(const GatedDeltaArgs*, const int*, const int*, float*,
                        float*, int, int, long, int, hipStream_t);
}

namespace {

// one branch: (rows, inv, weights, logits, gate_bias, scale, bias)
using Branch = std::tuple<Tensor, OptTensor, OptTensor, Tensor, Tensor, Tensor,
                          OptTensor>;

// x += the branches; their norm under w (one number, or one per coordinate)
OptTensor gate_norm(Tensor x, std::vector<Branch> branches, OptTensor w,
                    double eps, bool f32) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && is_f32(x) && x.is_contiguous(),
              "x must be a contiguous f32 [T, W] stream");
  TORCH_CHECK(branches.size() <= 2, "at most two branches");
  const int64_t T = x.size(0), W = x.size(1);
  GateNormArgs p{};
  bool vec = W % 8 == 0;
  for (size_t i = 0; i < branches.size(); ++i) {
    const auto& [rows, inv, weights, logits, gate_bias, scale, bias] =
        branches[i];
    GateBranch& b = p.branch[i];
    check_rows(rows, "rows");
    check_rows(logits, "logits");
    TORCH_CHECK(rows.is_contiguous() && rows.size(1) == W &&
                is_f32(rows) == f32, "rows must be contiguous, W wide");
    same_dtype(rows, logits, "gate logits");
    TORCH_CHECK(logits.size(0) == T && logits.size(1) == W, "logits [T, W]");
    check_f32(gate_bias, "gate_bias", W);
    check_f32(scale, "scale", W);
    if (bias) check_f32(*bias, "bias", W);
    if (inv) {
      TORCH_CHECK(weights && weights->dim() == 2 && weights->size(0) == T,
                  "weights [T, top]");
      check_f32(*weights, "weights", weights->numel());
      TORCH_CHECK(rows.size(0) == weights->numel() &&
                  inv->numel() == weights->numel(),
                  "one row per (token, choice)");
      b.inv = i32(*inv, "inv", weights->numel());
      b.weights = weights->data_ptr<float>();
      b.top = (int)weights->size(1);
    } else {
      TORCH_CHECK(rows.size(0) == T, "one row per token");
    }
    b.rows = rows.data_ptr();
    b.logits = logits.data_ptr();
    b.logit_row = logits.stride(0);
    b.gate_bias = gate_bias.data_ptr<float>();
    b.scale = scale.data_ptr<float>();
    b.bias = bias ? bias->data_ptr<float>() : nullptr;
    vec = vec && b.logit_row % 8 == 0 && aligned(logits, 16) &&
          aligned(rows, 16);
  }
  TORCH_CHECK(W <= gate_norm_max_width(vec), "width too large");
  OptTensor out;
  if (w) {
    TORCH_CHECK(w->numel() == 1 || w->numel() == W, "norm weight");
    check_f32(*w, "w", w->numel());
    out = torch::empty({T, W}, x.options().dtype(
        f32 ? torch::kFloat32 : torch::kBFloat16));
    p.w = w->data_ptr<float>();
    p.w_step = w->numel() > 1;
    p.out = out->data_ptr();
  }
  p.x = x.data_ptr<float>();
  p.tokens = (int)T; p.width = (int)W;
  p.eps = (float)eps;
  if (T && (w || !branches.empty()))
    launch_gate_norm(&p, f32, vec, current_stream());
  return out;
}

// out = silu(gate + gate_bias) * (up + up_bias)
void silu_glu(Tensor gate, Tensor up, OptTensor gate_bias, OptTensor up_bias,
              Tensor out) {
  glu_slices(gate, up, gate_bias, up_bias, out, GLU_SILU, 0.0);
}

void check_ring(const Tensor& ring, const Tensor& conv_w, const Tensor& like,
                int64_t channels) {
  TORCH_CHECK(conv_w.dim() == 2 && conv_w.size(0) >= 1 &&
              conv_w.size(1) == channels, "conv_w [taps, channels]");
  check_f32(conv_w, "conv_w", conv_w.numel());
  TORCH_CHECK(ring.is_cuda() && ring.is_contiguous() && ring.dim() == 3 &&
              ring.size(1) == conv_w.size(0) && ring.size(2) == channels,
              "ring [slots, taps, channels]");
  same_dtype(ring, like, "ring");
}

Tensor short_conv(Tensor x, Tensor conv_w, Tensor ring, Tensor tiles,
                  Tensor cu, Tensor starts, Tensor slots, int64_t tile) {
  check_rows(x, "x");
  const int64_t W = x.size(1), taps = conv_w.size(0), B = slots.numel();
  check_ring(ring, conv_w, x, W);
  TORCH_CHECK(tile >= taps - 1, "tile must cover the past");
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2, "tiles [n, 2]");
  auto out = torch::empty({x.size(0), W}, x.options());
  ShortConvArgs p{};
  p.x = x.data_ptr(); p.w = conv_w.data_ptr<float>();
  p.ring = ring.data_ptr(); p.out = out.data_ptr();
  p.tiles = i32(tiles, "tiles", 2);
  p.cu = i32(cu, "cu", B + 1);
  p.starts = i32(starts, "starts", B);
  p.slots = i32(slots, "slots", B);
  p.x_row = x.stride(0);
  p.n_tiles = (int)tiles.size(0); p.tile = (int)tile;
  p.width = (int)W; p.taps = (int)taps;
  const bool vec = mult8({W, p.x_row}) && aligned(x, 16) && aligned(ring, 16);
  if (x.size(0) && p.n_tiles)
    launch_short_conv(&p, is_f32(x), vec, current_stream());
  return out;
}

// qkv: rows with q, k, v at columns offs; beta, decay, gate: slices of logits
GatedDeltaArgs delta_args(const Tensor& qkv, const Tensor& beta,
                          const Tensor& decay, const Tensor& gate,
                          const Tensor& a_log, const Tensor& dt_bias,
                          const Tensor& norm_w, const Tensor& state,
                          const Tensor& slots, const OptTensor& cu,
                          const Tensor& starts, const Tensor& out,
                          const std::vector<int64_t>& offs, int64_t kv_heads,
                          bool silu, double q_scale, double unit_eps,
                          double norm_eps) {
  TORCH_CHECK(state.is_cuda() && state.dim() == 4 && is_f32(state) &&
              state.is_contiguous(), "state must be f32 [slots, heads, dim, vdim]");
  const int64_t H = state.size(1), D = state.size(2), E = state.size(3);
  const int64_t R = qkv.size(0), B = slots.numel();
  TORCH_CHECK(D <= 256 && E <= 256, "delta head size above 256");
  TORCH_CHECK(kv_heads > 0 && H % kv_heads == 0, "heads over key heads");
  TORCH_CHECK(offs.size() == 3, "columns of q, k, v");
  TORCH_CHECK(offs[0] >= 0 && offs[1] >= 0 && offs[2] >= 0 &&
              offs[0] + kv_heads * D <= qkv.size(1) &&
              offs[1] + kv_heads * D <= qkv.size(1) &&
              offs[2] + H * E <= qkv.size(1), "q, k or v outside the rows");
  for (const auto& [t, n, name] :
       {std::make_tuple(qkv, qkv.size(1), "qkv"),
        std::make_tuple(beta, H, "beta"),
        std::make_tuple(decay, decay.size(1), "decay"),
        std::make_tuple(gate, H * E, "gate"),
        std::make_tuple(out, H * E, "out")}) {
    check_rows(t, name);
    same_dtype(t, qkv, name);
    TORCH_CHECK(t.size(0) == R && t.size(1) == n, name, " shape");
  }
  TORCH_CHECK(decay.size(1) == H || decay.size(1) == H * D,
              "decay logits per head or per head and key channel");
  const bool per_channel = dt_bias.numel() == H * D && decay.size(1) == H * D;
  check_f32(a_log, "a_log", H);
  check_f32(dt_bias, "dt_bias", decay.size(1));
  check_f32(norm_w, "norm_w", E);
  if (!cu) TORCH_CHECK(B == R, "one row per sequence without cu");
  GatedDeltaArgs p{};
  p.qkv = qkv.data_ptr(); p.beta = beta.data_ptr();
  p.decay = decay.data_ptr(); p.gate = gate.data_ptr();
  p.a_log = a_log.data_ptr<float>();
  p.dt_bias = dt_bias.data_ptr<float>();
  p.norm_w = norm_w.data_ptr<float>();
  p.state = state.data_ptr<float>();
  p.slots = i32(slots, "slots", B);
  p.cu = cu ? i32(*cu, "cu", B + 1) : nullptr;
  p.starts = i32(starts, "starts", B);
  p.out = out.data_ptr();
  p.qkv_row = qkv.stride(0); p.beta_row = beta.stride(0);
  p.decay_row = decay.stride(0); p.gate_row = gate.stride(0);
  p.out_row = out.stride(0);
  p.off_q = (int)offs[0]; p.off_k = (int)offs[1]; p.off_v = (int)offs[2];
  p.heads = (int)H; p.kv_heads = (int)kv_heads;
  p.dim = (int)D; p.vdim = (int)E;
  p.per_channel = per_channel; p.silu = silu;
  p.q_scale = (float)q_scale;
  p.unit_eps = (float)unit_eps; p.norm_eps = (float)norm_eps;
  return p;
}

// With conv_w and ring: a decode step, whose q, k, v are the inputs of a short
// convolution over the columns from q's on.
void gated_step(Tensor qkv, Tensor beta, Tensor decay, Tensor gate,
                Tensor a_log, Tensor dt_bias, Tensor norm_w, Tensor state,
                Tensor slots, OptTensor cu, Tensor starts, Tensor out,
                std::vector<int64_t> offs, int64_t kv_heads, bool silu,
                double q_scale, double unit_eps, double norm_eps,
                OptTensor conv_w, OptTensor ring) {
  GatedDeltaArgs p = delta_args(qkv, beta, decay, gate, a_log, dt_bias, norm_w,
                                state, slots, cu, starts, out, offs, kv_heads,
                                silu, q_scale, unit_eps, norm_eps);
  if (conv_w) {
    TORCH_CHECK(ring && !cu, "the convolution is part of decode steps");
    const int64_t C = conv_w->size(1);
    check_ring(*ring, *conv_w, qkv, C);
    TORCH_CHECK(offs[1] >= offs[0] && offs[2] >= offs[0] &&
                offs[0] + C <= qkv.size(1) &&
                offs[1] + kv_heads * p.dim <= offs[0] + C &&
                offs[2] + (int64_t)p.heads * p.vdim <= offs[0] + C,
                "convolved columns");
    p.conv_w = conv_w->data_ptr<float>();
    p.ring = ring->data_ptr();
    p.taps = (int)conv_w->size(0);
    p.channels = (int)C;
  }
  if (slots.numel() && qkv.size(0))
    launch_gated_step(&p, (int)slots.numel(), is_f32(qkv), current_stream());
}

// Rows of several tokens per sequence, convolved, 16 at a time; tiles [n, 2] =
// (sequence, first token) and chunk_cu [B+1] number the chunks.
void gated_chunk(Tensor qkv, Tensor beta, Tensor decay, Tensor gate,
                 Tensor a_log, Tensor dt_bias, Tensor norm_w, Tensor state,
                 Tensor slots, Tensor cu, Tensor starts, Tensor out,
                 std::vector<int64_t> offs, int64_t kv_heads, bool silu,
                 double q_scale, double unit_eps, double norm_eps,
                 Tensor tiles, Tensor chunk_cu) {
  const GatedDeltaArgs p = delta_args(
      qkv, beta, decay, gate, a_log, dt_bias, norm_w, state, slots, cu, starts,
      out, offs, kv_heads, silu, q_scale, unit_eps, norm_eps);
  TORCH_CHECK(p.dim <= gated_chunk_max_dim(), "gated_chunk: head size");
  const int64_t B = slots.numel(), rows = qkv.size(0);
  if (!B || !rows) return;
  TORCH_CHECK(tiles.dim() == 2 && tiles.size(1) == 2, "tiles [n, 2]");
  const int64_t n = tiles.size(0);
  auto f32 = qkv.options().dtype(torch::kFloat32);
  auto ws = torch::empty({n * p.heads * gated_chunk_record(p.dim)}, f32);
  auto o = torch::empty({rows, (int64_t)p.heads * p.vdim}, f32);
  launch_gated_chunk(&p, i32(tiles, "tiles", 2 * n),
                     i32(chunk_cu, "chunk_cu", B + 1), ws.data_ptr<float>(),
                     o.data_ptr<float>(), (int)n, (int)B, rows, is_f32(qkv),
                     current_stream());
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("embed_stream", &embed_stream, "f32 stream = embed[token] * scale");
  m.def("gate_norm", &gate_norm,
        "stream += scaled, gated branches; norm of the stream");
  m.def("silu_glu", &silu_glu, "silu(gate + b) * (up + b)");
  m.def("short_conv", &short_conv, "causal depthwise conv + silu, varlen");
  m.def("gated_step", &gated_step, "gated delta rule, token by token");
  m.def("gated_chunk", &gated_chunk, "gated delta rule, by chunks");
  m.attr("CHUNK") = gated_chunk_tokens();
  m.attr("CHUNK_MAX_DIM") = gated_chunk_max_dim();
  m.def("skinny_gemm", &skinny_gemm, "decode-shape GEMM (M<=128)",
        py::arg("a"), py::arg("w"), py::arg("force_splits") = 0);
}
