// Elementwise gates in bf16 or f32: gelu_tanh(gate) * up, silu(gate) * up with
// or without biases, clamped units, and tanh of a low-rank projection.  Inputs and
// outputs are column slices of the fused projection buffers (row strides), so no
// copy stands between a GEMM and its gate, and the products land in the operand of the layer's output GEMM.
#include "act.h"
#include "vec_io.h"

namespace {

DEV_INLINE float gelu_tanh_f(float z) {
  const float c = 0.7978845608028654f;   // sqrt(2/pi)
  return 0.5f * z * (1.f + tanhf(c * (z + 0.044715f * z * z * z)));
}

struct GluArgs {
  void* out;              // [rows, out_row]
  const void* gate;       // + row*x_row
  const void* up;         // + row*x_row
  const float* gate_bias; // [inter], or null (both)
  const float* up_bias;
  long out_row, x_row;
  int inter;
  float limit;            // clamped units
};

template <typename T, int V, int ACT>
__global__ void glu_kernel(const GluArgs p, const long total) {
  const long step = (long)gridDim.x * blockDim.x;
  const int nv = p.inter / V;
  for (long i = blockIdx.x * (long)blockDim.x + threadIdx.x; i < total;
       i += step) {
    const long row = i / nv;
    const int c = (int)(i % nv) * V;
    float g[V], u[V];
    load_vec<V>((const T*)p.gate + row * p.x_row + c, g);
    load_vec<V>((const T*)p.up + row * p.x_row + c, u);
    if (p.gate_bias != nullptr) {
      float b[V];
      load_vec<V>(p.gate_bias + c, b);
#pragma unroll
      for (int j = 0; j < V; ++j) g[j] += b[j];
      load_vec<V>(p.up_bias + c, b);
#pragma unroll
      for (int j = 0; j < V; ++j) u[j] += b[j];
    }
#pragma unroll
    for (int j = 0; j < V; ++j)
      u[j] = ACT == GLU_GELU   ? gelu_tanh_f(g[j]) * u[j]
             : ACT == GLU_SILU ? g[j] * sigmoid_f(g[j]) * u[j]
                               : clamped_glu_f(g[j], u[j], p.limit);
    store_vec<V>((T*)p.out + row * p.out_row + c, u);
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

template <typename T, int ACT>
void glu_t(const GluArgs& p, long rows, hipStream_t s) {
  const bool vec = p.inter % 8 == 0 && p.out_row % 8 == 0 &&
                   p.x_row % 8 == 0 && aligned16(p.out) &&
                   aligned16(p.gate) && aligned16(p.up) &&
                   aligned16(p.gate_bias) && aligned16(p.up_bias);
  const long total = rows * (p.inter / (vec ? 8 : 1));
  int b = blocks_for(total);
  if (b > 16384) b = 16384;
  if (vec) {
    glu_kernel<T, 8, ACT><<<b, 256, 0, s>>>(p, total);
  } else {
    glu_kernel<T, 1, ACT><<<b, 256, 0, s>>>(p, total);
  }
}

}  // namespace

extern "C" {

// out = act(gate + gate_bias) * (up + up_bias); act: GLU_GELU or GLU_SILU.
// GLU_CLAMPED: clamped_glu_f of the two, with `limit`.
void launch_glu(void* out, long out_row, const void* gate, const void* up,
                long x_row, const float* gate_bias, const float* up_bias,
                long rows, int inter, int act, float limit, int f32,
                hipStream_t s) {
  const GluArgs p{out,     gate,  up,    gate_bias, up_bias,
                  out_row, x_row, inter, limit};
#define GLU_T(ACT)                                                            \
  do {                                                                        \
    if (f32) glu_t<float, ACT>(p, rows, s);                                   \
    else glu_t<__hip_bfloat16, ACT>(p, rows, s);                              \
  } while (0)
  if (act == GLU_GELU) GLU_T(GLU_GELU);
  else if (act == GLU_SILU) GLU_T(GLU_SILU);
  else GLU_T(GLU_CLAMPED);
#undef GLU_T
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
