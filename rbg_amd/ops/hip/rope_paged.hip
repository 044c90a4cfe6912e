// What stands between the fused query/key/value projection and attention over
// pages: biases (or none), rotary positions on the leading dimensions of queries and keys
// (rotate-half pairs, any rotated size, or none), and the paged store of keys and values,
// in 32-bit registers and one pass.  A thread takes V pairs, or V dimensions
// that do not rotate, of one head (a unit).
#include "moe_args.h"
#include "vec_io.h"

namespace {

template <int V>
DEV_INLINE void load_bias(const float* b, const int at, float* o) {
  if (b != nullptr) {
    load_vec<V>(b + at, o);
  } else {
#pragma unroll
    for (int j = 0; j < V; ++j) o[j] = 0.f;
  }
}

// R neighbouring rows, one unit of the row: the biases are read once, the rows'
// loads are all in flight together
template <typename T, int V, int R>
__global__ __launch_bounds__(256) void rope_paged_kernel(
    const RopePagedArgs p, const uint32_t items, const uint32_t units) {
  const uint32_t item = blockIdx.x * 256u + threadIdx.x;
  if (item >= items) return;
  const int row0 = (int)(item / units) * R;
  int u = (int)(item % units);
  const int half = p.rot / 2;
  const int pair_u = half / V, per_head = pair_u + (p.d - p.rot) / V;
  const bool own = p.k != nullptr;
  T* y[R];
  int page[R], at[R];
  bool on[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int row = min(row0 + r, p.rows - 1);
    const int slot = own ? p.slots[row] : -1;
    on[r] = row0 + r < p.rows;
    y[r] = (T*)p.proj + (size_t)row * p.stride;
    page[r] = slot >= 0 ? slot / p.page_size : -1;
    at[r] = slot >= 0 ? slot % p.page_size : 0;
  }
  const int qk_units = (p.heads + (own ? p.kv_heads : 0)) * per_head;
  if (u >= qk_units) {                  // values
    u -= qk_units;
    const int vu = p.dv / V, head = u / vu, d = (u % vu) * V;
    const int col = p.off_v + head * p.dv + d;
    float x[R][V], b[V];
    load_bias<V>(p.bias, col, b);
#pragma unroll
    for (int r = 0; r < R; ++r) load_vec<V>(y[r] + col, x[r]);
#pragma unroll
    for (int r = 0; r < R; ++r) {
#pragma unroll
      for (int j = 0; j < V; ++j) x[r][j] += b[j];
      if (on[r] && page[r] >= 0)
        store_vec<V>((T*)p.v + (((size_t)page[r] * p.kv_heads + head) *
                                    p.page_size + at[r]) * p.dv + d, x[r]);
    }
    return;
  }
  const int head = u / per_head, e = u % per_head;
  const bool is_q = head < p.heads;
  const int col = is_q ? p.off_q + head * p.d
                       : p.off_k + (head - p.heads) * p.d;
  auto target = [&](int r) -> T* {
    return is_q ? y[r] + col
                : (T*)p.k + (((size_t)page[r] * p.kv_heads + head - p.heads) *
                                 p.page_size + at[r]) * p.d;
  };
  if (e >= pair_u) {                    // dimensions that do not rotate
    const int d = p.rot + (e - pair_u) * V;
    float x[R][V], b[V];
    load_bias<V>(p.bias, col + d, b);
#pragma unroll
    for (int r = 0; r < R; ++r) load_vec<V>(y[r] + col + d, x[r]);
#pragma unroll
    for (int r = 0; r < R; ++r) {
#pragma unroll
      for (int j = 0; j < V; ++j) x[r][j] += b[j];
      if (on[r] && (is_q || page[r] >= 0)) store_vec<V>(target(r) + d, x[r]);
    }
    return;
  }
  const int d = e * V;
  float ba[V], bb[V];
  load_bias<V>(p.bias, col + d, ba);
  load_bias<V>(p.bias, col + half + d, bb);
  float a[R][V], b[R][V], c[R][V], s[R][V];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int row = min(row0 + r, p.rows - 1);
    const int pos = min(max(p.positions[row], 0), p.table_rows - 1);
    const float* cs = p.cos_sin + (size_t)pos * p.rot + d;
    load_vec<V>(y[r] + col + d, a[r]);
    load_vec<V>(y[r] + col + half + d, b[r]);
    load_vec<V>(cs, c[r]);
    load_vec<V>(cs + half, s[r]);
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
#pragma unroll
    for (int j = 0; j < V; ++j) {
      const float m = a[r][j] + ba[j], n = b[r][j] + bb[j];
      a[r][j] = m * c[r][j] - n * s[r][j];
      b[r][j] = n * c[r][j] + m * s[r][j];
    }
    if (on[r] && (is_q || page[r] >= 0)) {
      store_vec<V>(target(r) + d, a[r]);
      store_vec<V>(target(r) + half + d, b[r]);
    }
  }
}

template <typename T, int V, int R>
void rope_paged_r(const RopePagedArgs& p, int units, hipStream_t s) {
  const uint32_t items = (uint32_t)((p.rows + R - 1) / R) * units;
  rope_paged_kernel<T, V, R><<<(items + 255) / 256, 256, 0, s>>>(p, items,
                                                                 units);
}

template <typename T, int V>
void rope_paged_t(const RopePagedArgs& p, hipStream_t s) {
  const int per_head = p.rot / 2 / V + (p.d - p.rot) / V;
  const int units = p.k != nullptr
      ? (p.heads + p.kv_heads) * per_head + p.kv_heads * (p.dv / V)
      : p.heads * per_head;
  if (p.rows >= 1024) rope_paged_r<T, V, 2>(p, units, s);
  else rope_paged_r<T, V, 1>(p, units, s);
}

}  // namespace

extern "C" void launch_rope_paged(const RopePagedArgs* p, int f32, int vec,
                                  hipStream_t s) {
  if (f32) {
    if (vec) rope_paged_t<float, 8>(*p, s);
    else rope_paged_t<float, 1>(*p, s);
  } else {
    if (vec) rope_paged_t<__hip_bfloat16, 8>(*p, s);
    else rope_paged_t<__hip_bfloat16, 1>(*p, s);
  }
}
