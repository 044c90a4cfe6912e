// Argument checks shared by the extensions' bindings.
#pragma once
#include <torch/extension.h>
#include <ATen/hip/HIPContext.h>

#include <hip/hip_runtime.h>

namespace {

using torch::Tensor;
using OptTensor = c10::optional<torch::Tensor>;

[[maybe_unused]] hipStream_t current_stream() {
  return at::hip::getCurrentHIPStream().stream();
}

[[maybe_unused]] bool is_f32(const Tensor& t) {
  return t.scalar_type() == torch::kFloat32;
}

// activation: bf16 or f32 on the GPU, 2-D rows with a contiguous inner dim
[[maybe_unused]] void check_rows(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda(), name, " must be on GPU");
  TORCH_CHECK(t.scalar_type() == torch::kBFloat16 || is_f32(t), name,
              " must be bf16 or f32");
  TORCH_CHECK(t.dim() == 2 && (t.stride(1) == 1 || t.size(1) == 1), name,
              " must be 2-D with contiguous rows");
}

[[maybe_unused]] void check_f32(const Tensor& t, const char* name,
                                int64_t numel) {
  TORCH_CHECK(t.is_cuda() && is_f32(t) && t.is_contiguous(), name,
              " must be contiguous f32 on GPU");
  TORCH_CHECK(t.numel() == numel, name, " has ", t.numel(), " elements, not ",
              numel);
}

[[maybe_unused]] const int* i32(const Tensor& t, const char* name,
                                int64_t at_least) {
  TORCH_CHECK(t.is_cuda() && t.scalar_type() == torch::kInt32 &&
              t.is_contiguous(), name, " must be contiguous int32 on GPU");
  TORCH_CHECK(t.numel() >= at_least, name, " is too short");
  return t.data_ptr<int>();
}

[[maybe_unused]] void same_dtype(const Tensor& a, const Tensor& b,
                                 const char* name) {
  TORCH_CHECK(a.scalar_type() == b.scalar_type(), name, ": dtype mismatch");
}

[[maybe_unused]] void check_heads(const Tensor& t, const char* name) {
  TORCH_CHECK(t.is_cuda() && t.dim() == 3 &&
              (t.stride(2) == 1 || t.size(2) == 1), name,
              " must be 3-D with a contiguous inner dim");
}

[[maybe_unused]] bool mult8(std::initializer_list<int64_t> xs) {
  for (auto x : xs)
    if (x % 8) return false;
  return true;
}

[[maybe_unused]] bool aligned(const Tensor& t, int bytes) {
  return ((uintptr_t)t.data_ptr() % bytes) == 0;
}

// y [tokens * top, width] in expert order, as inv and weights [tokens, top] say
[[maybe_unused]] void check_experts(const Tensor& y, const Tensor& inv, const Tensor& weights,
                   int64_t tokens) {
  TORCH_CHECK(weights.dim() == 2 && weights.size(0) == tokens,
              "weights [tokens, top]");
  check_f32(weights, "weights", weights.numel());
  TORCH_CHECK(y.size(0) == weights.numel() && inv.numel() == weights.numel(),
              "one row per (token, choice)");
}

}  // namespace
