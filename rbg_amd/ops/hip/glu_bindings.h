// Bindings of the gated linear units, for every extension that links
// gated_act.hip.
#pragma once
#include "act_kinds.h"
#include "bind_util.h"

extern "C" void launch_glu(void*, long, const void*, const void*, long,
                           const float*, const float*, long, int, int, float,
                           int, hipStream_t);

// out = gelu_tanh(x[:, :F]) * x[:, F:]
[[maybe_unused]] static void gelu_mul(torch::Tensor x, torch::Tensor out) {
  check_rows(x, "x");
  check_rows(out, "out");
  same_dtype(x, out, "gelu_mul");
  TORCH_CHECK(x.is_contiguous() && x.size(1) == 2 * out.size(1) &&
              x.size(0) == out.size(0), "x must be [T, 2*ff] of out's rows");
  const int64_t F = out.size(1);
  if (x.size(0) && F)
    launch_glu(out.data_ptr(), out.stride(0), x.data_ptr(),
               (const char*)x.data_ptr() + F * x.element_size(), 2 * F, nullptr,
               nullptr, x.size(0), (int)F, GLU_GELU, 0.f, is_f32(x),
               current_stream());
}

// gate, up: slices of one buffer; the biases may be missing, both
[[maybe_unused]] static void glu_slices(
    const torch::Tensor& gate, const torch::Tensor& up,
    const OptTensor& gate_bias, const OptTensor& up_bias,
    const torch::Tensor& out, GluAct act, double limit) {
  check_rows(gate, "gate");
  check_rows(up, "up");
  check_rows(out, "out");
  same_dtype(gate, up, "up");
  same_dtype(gate, out, "glu out");
  const int64_t T = gate.size(0), F = gate.size(1);
  TORCH_CHECK(up.size(0) == T && up.size(1) == F && out.size(0) == T &&
              out.size(1) == F && up.stride(0) == gate.stride(0),
              "gate, up and out must have one shape, gate and up one stride");
  TORCH_CHECK(gate_bias.has_value() == up_bias.has_value(), "both biases");
  if (gate_bias) {
    check_f32(*gate_bias, "gate_bias", F);
    check_f32(*up_bias, "up_bias", F);
  }
  if (T && F)
    launch_glu(out.data_ptr(), out.stride(0), gate.data_ptr(), up.data_ptr(),
               gate.stride(0),
               gate_bias ? gate_bias->data_ptr<float>() : nullptr,
               up_bias ? up_bias->data_ptr<float>() : nullptr, T, (int)F, act,
               (float)limit, is_f32(gate), current_stream());
}
