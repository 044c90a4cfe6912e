// Elementwise gates in bf16 or f32: gelu_tanh(gate) * up, and tanh of a low-rank
// projection.  Inputs and outputs are column slices of the
// fused projection buffers (row strides), so no copy stands between a GEMM and
// its gate, and the products land in the operand of the layer's output GEMM.
#include "vec_io.h"

namespace {

DEV_INLINE float gelu_tanh_f(float z) {
  const float c = 0.7978845608028654f;   // sqrt(2/pi)
  return 0.5f * z * (1.f + tanhf(c * (z + 0.044715f * z * z * z)));
}

template <typename T, int V>
__global__ void gelu_mul_kernel(T* __restrict__ out, const long out_stride,
                                const T* __restrict__ x, const int inter,
                                const long total) {
  const long step = (long)gridDim.x * blockDim.x;
  const int nv = inter / V;
  for (long i = blockIdx.x * (long)blockDim.x + threadIdx.x; i < total;
       i += step) {
    const long row = i / nv;
    const int c = (int)(i % nv) * V;
    float g[V], u[V];
    load_vec<V>(x + row * 2 * inter + c, g);
    load_vec<V>(x + row * 2 * inter + inter + c, u);
#pragma unroll
    for (int j = 0; j < V; ++j) u[j] *= gelu_tanh_f(g[j]);
    store_vec<V>(out + row * out_stride + c, u);
  }
}

template <typename T>
__global__ void tanh_rows_kernel(T* __restrict__ out, const T* __restrict__ x,
                                 const long stride, const int width,
                                 const long total) {
  const long i = blockIdx.x * (long)blockDim.x + threadIdx.x;
  if (i >= total) return;
  out[i] = from_f<T>(tanhf(to_f(x[(i / width) * stride + i % width])));
}

int blocks_for(long total) {
  long b = (total + 255) / 256;
  return (int)(b < 1 ? 1 : b);
}

bool aligned16(const void* p) { return ((uintptr_t)p & 15) == 0; }

template <typename T>
void gelu_mul_t(void* out, long os, const void* x, long rows, int inter,
                hipStream_t s) {
  const bool vec = inter % 8 == 0 && os % 8 == 0 && aligned16(out);
  const long total = rows * (inter / (vec ? 8 : 1));
  int b = blocks_for(total);
  if (b > 16384) b = 16384;
  if (vec)
    gelu_mul_kernel<T, 8><<<b, 256, 0, s>>>((T*)out, os, (const T*)x, inter,
                                            total);
  else
    gelu_mul_kernel<T, 1><<<b, 256, 0, s>>>((T*)out, os, (const T*)x, inter,
                                            total);
}

}  // namespace

extern "C" {

void launch_gelu_mul(void* out, long out_stride, const void* x, long rows,
                     int inter, int f32, hipStream_t s) {
  if (f32) gelu_mul_t<float>(out, out_stride, x, rows, inter, s);
  else gelu_mul_t<__hip_bfloat16>(out, out_stride, x, rows, inter, s);
}

void launch_tanh_rows(void* out, const void* x, long stride, long rows,
                      int width, int f32, hipStream_t s) {
  const long total = rows * width;
  if (f32)
    tanh_rows_kernel<float><<<blocks_for(total), 256, 0, s>>>(
        (float*)out, (const float*)x, stride, width, total);
  else
    tanh_rows_kernel<__hip_bfloat16><<<blocks_for(total), 256, 0, s>>>(
        (__hip_bfloat16*)out, (const __hip_bfloat16*)x, stride, width, total);
}

}  // extern "C"
