// What stands between the fused query/key/value projection and attention over
// pages: biases, rotary positions on the leading dimensions of queries and keys
// (rotate-half pairs, any rotated size), and the paged store of keys and values,
// in 32-bit registers and one pass.  A thread takes V pairs, or V dimensions
// that do not rotate, of one head.
#include "moe_args.h"
#include "vec_io.h"

namespace {

template <typename T, int V>
DEV_INLINE void rope_unit(const RopePagedArgs& p, const int row, int u) {
  const int half = p.rot / 2;
  const int pair_u = half / V, per_head = pair_u + (p.d - p.rot) / V;
  const int slot = p.k != nullptr ? p.slots[row] : -1;
  const int page = slot >= 0 ? slot / p.page_size : 0;
  const int at = slot >= 0 ? slot % p.page_size : 0;
  T* y = (T*)p.proj + (size_t)row * p.stride;

  const int qk_units = (p.heads + (p.k != nullptr ? p.kv_heads : 0)) * per_head;
  if (u >= qk_units) {                  // values
    u -= qk_units;
    const int vu = p.dv / V, head = u / vu, d = (u % vu) * V;
    const int col = p.off_v + head * p.dv + d;
    float x[V], b[V];
    load_vec<V>(y + col, x);
    load_vec<V>(p.bias + col, b);
#pragma unroll
    for (int j = 0; j < V; ++j) x[j] += b[j];
    if (slot >= 0)
      store_vec<V>((T*)p.v + (((size_t)page * p.kv_heads + head) *
                                  p.page_size + at) * p.dv + d, x);
    return;
  }
  const int head = u / per_head, e = u % per_head;
  const bool is_q = head < p.heads;
  const int col0 = is_q ? p.off_q + head * p.d
                        : p.off_k + (head - p.heads) * p.d;
  T* dst = is_q ? y + col0
                : (T*)p.k + (((size_t)page * p.kv_heads + head - p.heads) *
                                 p.page_size + at) * p.d;
  const bool write = is_q || slot >= 0;
  if (e >= pair_u) {
    const int d = p.rot + (e - pair_u) * V;
    float x[V], b[V];
    load_vec<V>(y + col0 + d, x);
    load_vec<V>(p.bias + col0 + d, b);
#pragma unroll
    for (int j = 0; j < V; ++j) x[j] += b[j];
    if (write) store_vec<V>(dst + d, x);
    return;
  }
  const int d = e * V;
  const int pos = min(max(p.positions[row], 0), p.table_rows - 1);
  const float* cs = p.cos_sin + (size_t)pos * p.rot + d;
  float a[V], b[V], ba[V], bb[V], c[V], s[V];
  load_vec<V>(y + col0 + d, a);
  load_vec<V>(y + col0 + half + d, b);
  load_vec<V>(p.bias + col0 + d, ba);
  load_vec<V>(p.bias + col0 + half + d, bb);
  load_vec<V>(cs, c);
  load_vec<V>(cs + half, s);
#pragma unroll
  for (int j = 0; j < V; ++j) {
    const float m = a[j] + ba[j], n = b[j] + bb[j];
    a[j] = m * c[j] - n * s[j];
    b[j] = n * c[j] + m * s[j];
  }
  if (write) {
    store_vec<V>(dst + d, a);
    store_vec<V>(dst + half + d, b);
  }
}

// TPR threads per row
template <typename T, int V, int TPR>
__global__ __launch_bounds__(256) void rope_paged_kernel(
    const RopePagedArgs p, const int units) {
  const int row = blockIdx.x * (256 / TPR) + threadIdx.x / TPR;
  if (row >= p.rows) return;
  for (int u = threadIdx.x % TPR; u < units; u += TPR)
    rope_unit<T, V>(p, row, u);
}

template <typename T, int V>
void rope_paged_t(const RopePagedArgs& p, hipStream_t s) {
  const int per_head = p.rot / 2 / V + (p.d - p.rot) / V;
  const int units = p.k != nullptr
      ? (p.heads + p.kv_heads) * per_head + p.kv_heads * (p.dv / V)
      : p.heads * per_head;
  // long prompts: a wave per row; short steps: more waves, to hide latency
  if (p.rows >= 1024) {
    rope_paged_kernel<T, V, 64><<<(p.rows + 3) / 4, 256, 0, s>>>(p, units);
  } else {
    rope_paged_kernel<T, V, 256><<<p.rows, 256, 0, s>>>(p, units);
  }
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
