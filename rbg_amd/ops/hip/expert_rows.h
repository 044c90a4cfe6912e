// What a branch left for a token, for the kernels that add it to the stream.
#pragma once
#include "vec_io.h"

// y of one token: its row, or the weighed sum of its `top` expert rows
template <typename T, int V>
DEV_INLINE void branch_row(const T* __restrict__ y, const int* __restrict__ inv,
                           const float* __restrict__ wts, const int top,
                           const size_t token, const int width, const int i,
                           float* o) {
  if (inv == nullptr) {
    load_vec<V>(y + token * width + i, o);
    return;
  }
#pragma unroll
  for (int j = 0; j < V; ++j) o[j] = 0.f;
#pragma unroll 4
  for (int t = 0; t < top; ++t) {
    float r[V];
    load_vec<V>(y + (size_t)inv[token * top + t] * width + i, r);
    const float w = wts[token * top + t];
#pragma unroll
    for (int j = 0; j < V; ++j) o[j] += w * r[j];
  }
}
