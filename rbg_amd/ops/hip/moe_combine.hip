// Weighed sums of each token's expert rows.
#include "expert_rows.h"

namespace {

constexpr int NT = 256;

template <typename T, int V>
__global__ __launch_bounds__(NT) void moe_combine_kernel(
    T* __restrict__ out, const T* __restrict__ y, const int* __restrict__ inv,
    const float* __restrict__ wts, const int top, const int width) {
  for (int i = threadIdx.x * V; i < width; i += NT * V) {
    float o[V];
    branch_row<T, V>(y, inv, wts, top, blockIdx.x, width, i, o);
    store_vec<V>(out + (size_t)blockIdx.x * width + i, o);
  }
}

}  // namespace

extern "C" void launch_moe_combine(void* out, const void* y, const int* inv,
                        const float* wts, int top, int tokens, int width,
                        int f32, hipStream_t s) {
#define MC_GO(T, V) moe_combine_kernel<T, V><<<tokens, NT, 0, s>>>(           \
      (T*)out, (const T*)y, inv, wts, top, width)
  const bool vec = width % 8 == 0;
  if (f32) { if (vec) MC_GO(float, 8); else MC_GO(float, 1); }
  else { if (vec) MC_GO(__hip_bfloat16, 8); else MC_GO(__hip_bfloat16, 1); }
#undef MC_GO
}
