// What a branch left for a token, for the kernels that add it to the stream.
#pragma once
#include "vec_io.h"

// o += the weighed sum of one token's `top` expert rows.  A choice whose inv is
// negative has no row: its expert returns its own input, row `self` of the token
// (null: such choices are left out, as are expert rows when y is null).
template <typename T, int V>
DEV_INLINE void add_expert_rows(const T* __restrict__ y,
                                const int* __restrict__ inv,
                                const float* __restrict__ wts, const int top,
                                const T* __restrict__ self, const size_t token,
                                const int width, const int i, float* o) {
  constexpr int UN = 4;                         // rows in flight
  for (int t0 = 0; t0 < top; t0 += UN) {
    float r[UN][V], w[UN];
    bool on[UN];
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const size_t at = token * top + min(t0 + u, top - 1);
      const int row = inv[at];
      const T* src = row < 0 ? self : y;
      on[u] = t0 + u < top && src != nullptr;
      w[u] = wts[at];
      if (src != nullptr)
        load_vec<V>(src + (row < 0 ? token : (size_t)row) * width + i, r[u]);
    }
#pragma unroll
    for (int u = 0; u < UN; ++u)
      if (on[u]) {
#pragma unroll
        for (int j = 0; j < V; ++j) o[j] += w[u] * r[u][j];
      }
  }
}

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
  add_expert_rows<T, V>(y, inv, wts, top, nullptr, token, width, i, o);
}
