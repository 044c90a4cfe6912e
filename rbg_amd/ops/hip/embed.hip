// Token rows into the f32 residual stream, times a constant; into each of the
// streams of designs that have several.
#include "vec_io.h"

namespace {

constexpr int NT = 256;

template <typename T, int V>
__global__ __launch_bounds__(NT) void embed_stream_kernel(
    float* __restrict__ x, const T* __restrict__ table,
    const long* __restrict__ tokens, const float scale, const int width,
    const int copies) {
  const T* src = table + (size_t)tokens[blockIdx.x] * width;
  float* dst = x + (size_t)blockIdx.x * copies * width;
  for (int i = threadIdx.x * V; i < width; i += NT * V) {
    float v[V];
    load_vec<V>(src + i, v);
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] *= scale;
    for (int c = 0; c < copies; ++c)
      store_vec<V>(dst + (size_t)c * width + i, v);
  }
}

}  // namespace

extern "C" void launch_embed_stream(float* x, const void* table,
                                    const long* tokens, float scale, int n,
                                    int width, int copies, int f32,
                                    hipStream_t s) {
#define EM_GO(T, V) embed_stream_kernel<T, V><<<n, NT, 0, s>>>(               \
      x, (const T*)table, tokens, scale, width, copies)
  const bool vec = width % 8 == 0;
  if (f32) { if (vec) EM_GO(float, 8); else EM_GO(float, 1); }
  else { if (vec) EM_GO(__hip_bfloat16, 8); else EM_GO(__hip_bfloat16, 1); }
#undef EM_GO
}
