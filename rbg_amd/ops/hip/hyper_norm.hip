// f32 residual streams of designs with hyper-connections and dynamic tanh norms.
// A sublayer reads a weighed sum of the streams and writes to all of them:
//     x_t  = sum_s mix[s, t] x_s + mult * out[t] * y      (all from the old x)
//     h    = tanh(alpha * sum_s read[s] x_s) * w + b
// in one pass, where y is a row of the sublayer's output plus, for experts, the
// weighed sum of the token's expert rows.  Nothing is reduced over the width: a
// thread takes V columns of a token through all streams.
#include "expert_rows.h"
#include "hyper_args.h"

namespace {

constexpr int NT = 256;

template <typename T, int V>
DEV_INLINE void pending_row(const HyperArgs& p, const size_t token,
                            const int i, float* y) {
  if (p.rows != nullptr) {
    load_vec<V>((const T*)p.rows + token * p.width + i, y);
  } else {
#pragma unroll
    for (int j = 0; j < V; ++j) y[j] = 0.f;
  }
  if (p.inv != nullptr)
    add_expert_rows<T, V>((const T*)p.experts, p.inv, p.weights, p.top,
                          (const T*)p.self, token, p.width, i, y);
}

template <typename T, int V>
DEV_INLINE void put_norm(const HyperArgs& p, const size_t token, const int i,
                         float* u) {
  float w[V], b[V];
  load_vec<V>(p.w + i, w);
  load_vec<V>(p.b + i, b);
  const float alpha = p.alpha[0];
#pragma unroll
  for (int j = 0; j < V; ++j) u[j] = tanhf(alpha * u[j]) * w[j] + b[j];
  store_vec<V>((T*)p.out + token * p.width + i, u);
}

template <typename T, int V, int S>
__global__ __launch_bounds__(NT) void hyper_norm_kernel(const HyperArgs p) {
  const unsigned per = p.width / V;
  const unsigned item = blockIdx.x * NT + threadIdx.x;
  const size_t token = item / per;
  if (token >= (size_t)p.tokens) return;
  const int i = (int)(item % per) * V;
  float* x = p.x + token * S * p.width + i;
  float a[S][V];
#pragma unroll
  for (int s = 0; s < S; ++s) load_vec<V>(x + (size_t)s * p.width, a[s]);
  float u[V];
#pragma unroll
  for (int j = 0; j < V; ++j) u[j] = 0.f;
  if (p.conn != nullptr) {
    float y[V];
    pending_row<T, V>(p, token, i, y);
#pragma unroll
    for (int t = 0; t < S; ++t) {
      const float c = p.mult * p.conn[S * S + t];
      const float r = p.w != nullptr ? p.read[t] : 0.f;
      float n[V];
#pragma unroll
      for (int j = 0; j < V; ++j) n[j] = c * y[j];
#pragma unroll
      for (int s = 0; s < S; ++s) {
        const float m = p.conn[s * S + t];
#pragma unroll
        for (int j = 0; j < V; ++j) n[j] += m * a[s][j];
      }
      store_vec<V>(x + (size_t)t * p.width, n);
#pragma unroll
      for (int j = 0; j < V; ++j) u[j] += r * n[j];
    }
  } else {
#pragma unroll
    for (int s = 0; s < S; ++s) {
      const float r = p.w != nullptr ? p.read[s] : 0.f;
#pragma unroll
      for (int j = 0; j < V; ++j) u[j] += r * a[s][j];
    }
  }
  if (p.w != nullptr) put_norm<T, V>(p, token, i, u);
}

// any number of streams: the old ones of a column wait in LDS
template <typename T>
__global__ __launch_bounds__(NT) void hyper_norm_any_kernel(
    const HyperArgs p) {
  extern __shared__ float old[];                // [streams][NT]
  const unsigned item = blockIdx.x * NT + threadIdx.x;
  const size_t token = item / (unsigned)p.width;
  if (token >= (size_t)p.tokens) return;        // no barrier below
  const int i = (int)(item % (unsigned)p.width), S = p.streams;
  float* x = p.x + token * S * p.width + i;
  float u = 0.f;
  for (int s = 0; s < S; ++s) {
    const float v = x[(size_t)s * p.width];
    old[s * NT + threadIdx.x] = v;
    if (p.conn == nullptr && p.w != nullptr) u += p.read[s] * v;
  }
  if (p.conn != nullptr) {
    float y;
    pending_row<T, 1>(p, token, i, &y);
    for (int t = 0; t < S; ++t) {
      float n = p.mult * p.conn[S * S + t] * y;
      for (int s = 0; s < S; ++s)
        n += p.conn[s * S + t] * old[s * NT + threadIdx.x];
      x[(size_t)t * p.width] = n;
      if (p.w != nullptr) u += p.read[t] * n;
    }
  }
  if (p.w != nullptr) put_norm<T, 1>(p, token, i, &u);
}

template <typename T, int V>
void hyper_norm_v(const HyperArgs& p, hipStream_t s) {
  const unsigned grid =
      (unsigned)(((long)p.tokens * (p.width / V) + NT - 1) / NT);
#define HN_GO(S) hyper_norm_kernel<T, V, S><<<grid, NT, 0, s>>>(p)
  switch (p.streams) {
    case 1: HN_GO(1); break;
    case 2: HN_GO(2); break;
    case 3: HN_GO(3); break;
    case 4: HN_GO(4); break;
    default: break;
  }
#undef HN_GO
}

template <typename T>
void hyper_norm_t(const HyperArgs& p, int vec, hipStream_t s) {
  if (p.streams > 4) {
    const unsigned grid =
        (unsigned)(((long)p.tokens * p.width + NT - 1) / NT);
    hyper_norm_any_kernel<T>
        <<<grid, NT, sizeof(float) * NT * p.streams, s>>>(p);
  } else if (vec) {
    // 8 columns a thread once the chip is full of them
    if ((long)p.tokens * p.width >= 8l * 256 * NT * 4)
      hyper_norm_v<T, 8>(p, s);
    else
      hyper_norm_v<T, 4>(p, s);
  } else {
    hyper_norm_v<T, 1>(p, s);
  }
}

}  // namespace

extern "C" {

int hyper_max_streams() { return 64; }        // 64 KB of LDS

void launch_hyper_norm(const HyperArgs* p, int f32, int vec, hipStream_t s) {
  if (f32) hyper_norm_t<float>(*p, vec, s);
  else hyper_norm_t<__hip_bfloat16>(*p, vec, s);
}

}  // extern "C"
