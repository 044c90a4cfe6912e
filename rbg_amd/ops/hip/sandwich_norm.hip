// f32 residual stream of designs that norm a branch before adding it: token
// pair embedding, and
//     x += rms(y) * wb;   out = rms(x) * w
// in one pass, where y is a row of the branch's output or the weighed sum of a
// token's expert rows (so the experts' combination costs no pass of its own).
// One workgroup per token; the row stays in registers between the two norms.
#include "expert_rows.h"

namespace {

constexpr int NT = 256, NW = NT / 64;

template <typename T, int V>
__global__ __launch_bounds__(NT) void embed_pairs_kernel(
    float* __restrict__ x, const T* __restrict__ table,
    const T* __restrict__ pairs, const long* __restrict__ tokens,
    const long* __restrict__ prev, const long mul_prev, const long mul_cur,
    const long buckets, const int width) {
  const long tok = tokens[blockIdx.x], before = prev[blockIdx.x];
  const long row =
      before < 0 ? buckets : (before * mul_prev + tok * mul_cur) % buckets;
  const T* a = table + (size_t)tok * width;
  const T* b = pairs + (size_t)row * width;
  float* dst = x + (size_t)blockIdx.x * width;
  for (int i = threadIdx.x * V; i < width; i += NT * V) {
    float u[V], v[V];
    load_vec<V>(a + i, u);
    load_vec<V>(b + i, v);
#pragma unroll
    for (int j = 0; j < V; ++j) u[j] += v[j];
    store_vec<V>(dst + i, u);
  }
}

// IT * NT * V >= width
template <typename T, int V, int IT>
__global__ __launch_bounds__(NT) void sandwich_norm_kernel(
    float* __restrict__ x, const T* __restrict__ y,
    const int* __restrict__ inv, const float* __restrict__ wts, const int top,
    const float* __restrict__ wb, const float* __restrict__ w,
    T* __restrict__ out, const int width, const float eps) {
  __shared__ float red[2][NW];
  const size_t token = blockIdx.x, base = token * width;
  float xr[IT][V];
#pragma unroll
  for (int k = 0; k < IT; ++k) {
    const int i = (k * NT + threadIdx.x) * V;
    if (i < width) load_vec<V>(x + base + i, xr[k]);
  }
  if (y != nullptr) {
    float yr[IT][V], ss = 0.f;
#pragma unroll
    for (int k = 0; k < IT; ++k) {
      const int i = (k * NT + threadIdx.x) * V;
      if (i >= width) continue;
      branch_row<T, V>(y, inv, wts, top, token, width, i, yr[k]);
#pragma unroll
      for (int j = 0; j < V; ++j) ss += yr[k][j] * yr[k][j];
    }
    const float sc = 1.f / sqrtf(block_sum<NW>(ss, red[0]) / width + eps);
#pragma unroll
    for (int k = 0; k < IT; ++k) {
      const int i = (k * NT + threadIdx.x) * V;
      if (i >= width) continue;
      float g[V];
      load_vec<V>(wb + i, g);
#pragma unroll
      for (int j = 0; j < V; ++j) xr[k][j] += yr[k][j] * sc * g[j];
      store_vec<V>(x + base + i, xr[k]);
    }
  }
  if (w == nullptr) return;
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < IT; ++k) {
    const int i = (k * NT + threadIdx.x) * V;
    if (i >= width) continue;
#pragma unroll
    for (int j = 0; j < V; ++j) ss += xr[k][j] * xr[k][j];
  }
  const float sc = 1.f / sqrtf(block_sum<NW>(ss, red[1]) / width + eps);
#pragma unroll
  for (int k = 0; k < IT; ++k) {
    const int i = (k * NT + threadIdx.x) * V;
    if (i >= width) continue;
    float g[V];
    load_vec<V>(w + i, g);
#pragma unroll
    for (int j = 0; j < V; ++j) g[j] *= xr[k][j] * sc;
    store_vec<V>(out + base + i, g);
  }
}

template <typename T, int V>
void sandwich_v(float* x, const void* y, const int* inv, const float* wts,
                int top, const float* wb, const float* w, void* out,
                int tokens, int width, float eps, hipStream_t s) {
#define SN_GO(IT)                                                             \
  sandwich_norm_kernel<T, V, IT><<<tokens, NT, 0, s>>>(                       \
      x, (const T*)y, inv, wts, top, wb, w, (T*)out, width, eps)
  const int it = (width + NT * V - 1) / (NT * V);
  if (it <= 1) SN_GO(1);
  else if (it <= 2) SN_GO(2);
  else if (it <= 4) SN_GO(4);
  else SN_GO(8);
#undef SN_GO
}

}  // namespace

extern "C" {

void launch_embed_pairs(float* x, const void* table, const void* pairs,
                        const long* tokens, const long* prev, long mul_prev,
                        long mul_cur, long buckets, int n, int width, int f32,
                        hipStream_t s) {
#define EP_GO(T, V) embed_pairs_kernel<T, V><<<n, NT, 0, s>>>(                \
      x, (const T*)table, (const T*)pairs, tokens, prev, mul_prev, mul_cur,   \
      buckets, width)
  const bool vec = width % 8 == 0;
  if (f32) { if (vec) EP_GO(float, 8); else EP_GO(float, 1); }
  else { if (vec) EP_GO(__hip_bfloat16, 8); else EP_GO(__hip_bfloat16, 1); }
#undef EP_GO
}

// widest row: 8 steps of a workgroup
int sandwich_max_width(int width) { return width % 8 ? NT * 8 : NT * 64; }

void launch_sandwich_norm(float* x, const void* y, const int* inv,
                          const float* wts, int top, const float* wb,
                          const float* w, void* out, int tokens, int width,
                          float eps, int f32, hipStream_t s) {
#define SN_T(T)                                                               \
  do {                                                                        \
    if (width % 8 == 0)                                                       \
      sandwich_v<T, 8>(x, y, inv, wts, top, wb, w, out, tokens, width, eps,   \
                       s);                                                    \
    else                                                                      \
      sandwich_v<T, 1>(x, y, inv, wts, top, wb, w, out, tokens, width, eps,   \
                       s);                                                    \
  } while (0)
  if (f32) SN_T(float); else SN_T(__hip_bfloat16);
#undef SN_T
}

}  // extern "C"
