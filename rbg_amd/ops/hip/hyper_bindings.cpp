// PyTorch bindings for hyper-connections with dynamic tanh norms and gated linear
// units (bf16 or f32 activations).  Shapes, strides and dtypes are checked here,
// before launch.
#include "bind_util.h"
#include "embed_bindings.h"
#include "gemm_bindings.h"
#include "glu_bindings.h"
#include "hyper_args.h"

extern "C" {
int hyper_max_streams();
void launch_hyper_norm(const HyperArgs*, int, int, hipStream_t);
}

namespace {

// x [T, S * W]: the streams.  conn (with what is pending: rows, experts, or
// both) moves them on; with w the next sublayer's normed input is returned.
OptTensor hyper_norm(Tensor x, int64_t streams, OptTensor conn, OptTensor rows,
                     OptTensor experts, OptTensor inv, OptTensor weights,
                     OptTensor self, double mult, OptTensor read, OptTensor w,
                     OptTensor b, OptTensor alpha, bool f32) {
  TORCH_CHECK(x.is_cuda() && x.dim() == 2 && is_f32(x) && x.is_contiguous(),
              "x must be contiguous f32 [T, S * W] streams");
  TORCH_CHECK(streams > 0 && streams <= hyper_max_streams() &&
              x.size(1) % streams == 0, "number of streams");
  const int64_t T = x.size(0), W = x.size(1) / streams;
  TORCH_CHECK(T * W < (1ll << 31), "too many rows");
  HyperArgs p{};
  bool vec = W % 8 == 0;
  auto take = [&](const OptTensor& t, const char* name,
                  int64_t n) -> const void* {
    if (!t) return nullptr;
    check_rows(*t, name);
    TORCH_CHECK(t->is_contiguous() && t->size(1) == W && t->size(0) == n &&
                is_f32(*t) == f32, name, " must be contiguous, W wide");
    vec = vec && aligned(*t, 16);
    return t->data_ptr();
  };
  if (conn) {
    check_f32(*conn, "conn", streams * (streams + 1));
    p.conn = conn->data_ptr<float>();
    p.rows = take(rows, "rows", T);
    if (inv) {
      TORCH_CHECK(weights && weights->dim() == 2 && weights->size(0) == T,
                  "weights [T, top]");
      check_f32(*weights, "weights", weights->numel());
      p.inv = i32(*inv, "inv", weights->numel());
      p.weights = weights->data_ptr<float>();
      p.top = (int)weights->size(1);
      p.experts = take(experts, "experts", weights->numel());
      p.self = take(self, "self", T);
    }
  }
  OptTensor out;
  if (w) {
    TORCH_CHECK(read && b && alpha, "a norm needs read, b and alpha");
    check_f32(*w, "w", W);
    check_f32(*b, "b", W);
    check_f32(*alpha, "alpha", 1);
    check_f32(*read, "read", streams);
    vec = vec && aligned(*w, 16) && aligned(*b, 16);
    out = torch::empty({T, W}, x.options().dtype(
        f32 ? torch::kFloat32 : torch::kBFloat16));
    p.w = w->data_ptr<float>();
    p.b = b->data_ptr<float>();
    p.alpha = alpha->data_ptr<float>();
    p.read = read->data_ptr<float>();
    p.out = out->data_ptr();
  }
  p.x = x.data_ptr<float>();
  p.tokens = (int)T; p.streams = (int)streams; p.width = (int)W;
  p.mult = (float)mult;
  if (T && (p.conn || p.w)) launch_hyper_norm(&p, f32, vec, current_stream());
  return out;
}

// out = clamped_glu_f(gate, up); gate, up: slices of one buffer
void clamped_glu(Tensor gate, Tensor up, double limit, Tensor out) {
  glu_slices(gate, up, c10::nullopt, c10::nullopt, out, GLU_CLAMPED, limit);
}

}  // namespace

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("embed_stream", &embed_stream, "f32 streams = embed[token] * scale");
  m.def("hyper_norm", &hyper_norm,
        "streams take a sublayer's output; tanh norm of what is read next");
  m.def("gelu_mul", &gelu_mul, "gelu_tanh(gate) * up");
  m.def("clamped_glu", &clamped_glu, "clamped gated unit");
  m.def("skinny_gemm", &skinny_gemm, "decode-shape GEMM (M<=128)",
        py::arg("a"), py::arg("w"), py::arg("force_splits") = 0);
}
