// Short causal depthwise convolution with silu over portions of sequences
// (gfx950), on a column slice of a projection.
//
// A sequence's past inputs are kept in its state slot as a ring: position p's
// input at p % taps, one place more than the convolution looks back.  So a
// decode step may read the past in one workgroup while another stores the
// present (gated_delta.hip), and nothing is ever shifted.  Before position 0 the
// input is zero, whatever the slot holds.
//
// A thread walks a tile of tokens for V channels with the last inputs in
// registers.  Only a sequence's first tile reads the ring (the host keeps tile
// >= taps - 1), and that same thread stores the portion's last inputs.
#include "gated_args.h"
#include "vec_io.h"

namespace {

constexpr int NT = 256;

DEV_INLINE float silu_f(float z) { return z * sigmoid_f(z); }

// TAPS 0: any number, rows read again for every tap
template <typename T, int V, int TAPS>
__global__ __launch_bounds__(NT) void short_conv_kernel(const ShortConvArgs p) {
  const int seq = p.tiles[blockIdx.x * 2], t0 = p.tiles[blockIdx.x * 2 + 1];
  const int row0 = p.cu[seq], len = p.cu[seq + 1] - row0;
  const int i = (blockIdx.y * NT + threadIdx.x) * V;
  if (i >= p.width) return;
  const int taps = TAPS > 0 ? TAPS : p.taps, start = p.starts[seq];
  T* ring = (T*)p.ring + (size_t)p.slots[seq] * taps * p.width + i;
  const T* xs = (const T*)p.x + (size_t)row0 * p.x_row + i;
  T* out = (T*)p.out + (size_t)row0 * p.width + i;
  const int t1 = min(t0 + p.tile, len);
  auto input = [&](int t, float* v) {
    if (t >= 0) {
      load_vec<V>(xs + (size_t)t * p.x_row, v);
    } else if (start + t >= 0) {
      load_vec<V>(ring + (size_t)((start + t) % taps) * p.width, v);
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = 0.f;
    }
  };
  if constexpr (TAPS > 0) {
    float cw[TAPS][V], win[TAPS][V];
#pragma unroll
    for (int k = 0; k < TAPS; ++k)
      load_vec<V>(p.w + (size_t)k * p.width + i, cw[k]);
#pragma unroll
    for (int k = 1; k < TAPS; ++k) input(t0 - TAPS + k, win[k]);
#pragma unroll 4
    for (int t = t0; t < t1; ++t) {
#pragma unroll
      for (int k = 1; k < TAPS; ++k)
#pragma unroll
        for (int j = 0; j < V; ++j) win[k - 1][j] = win[k][j];
      load_vec<V>(xs + (size_t)t * p.x_row, win[TAPS - 1]);
      float h[V];
#pragma unroll
      for (int j = 0; j < V; ++j) {
        h[j] = 0.f;
#pragma unroll
        for (int k = 0; k < TAPS; ++k) h[j] += cw[k][j] * win[k][j];
        h[j] = silu_f(h[j]);
      }
      store_vec<V>(out + (size_t)t * p.width, h);
    }
  } else {
    for (int t = t0; t < t1; ++t) {
      float h[V], cw[V], v[V];
#pragma unroll
      for (int j = 0; j < V; ++j) h[j] = 0.f;
      for (int k = 0; k < taps; ++k) {
        input(t - taps + 1 + k, v);
        load_vec<V>(p.w + (size_t)k * p.width + i, cw);
#pragma unroll
        for (int j = 0; j < V; ++j) h[j] += cw[j] * v[j];
      }
#pragma unroll
      for (int j = 0; j < V; ++j) h[j] = silu_f(h[j]);
      store_vec<V>(out + (size_t)t * p.width, h);
    }
  }
  if (t0 == 0 && taps > 1) {
    for (int t = max(0, len - taps + 1); t < len; ++t) {
      float v[V];
      load_vec<V>(xs + (size_t)t * p.x_row, v);
      store_vec<V>(ring + (size_t)((start + t) % taps) * p.width, v);
    }
  }
}

}  // namespace

extern "C" void launch_short_conv(const ShortConvArgs* p, int f32, int vec,
                                  hipStream_t s) {
  const int v = vec ? 8 : 1;
  const dim3 grid(p->n_tiles, (p->width / v + NT - 1) / NT);
#define SC_GO(T, V, N) short_conv_kernel<T, V, N><<<grid, NT, 0, s>>>(*p)
#define SC_V(T)                                                               \
  do {                                                                        \
    if (!vec) { SC_GO(T, 1, 0); }                                             \
    else if (p->taps == 2) { SC_GO(T, 8, 2); }                                \
    else if (p->taps == 3) { SC_GO(T, 8, 3); }                                \
    else if (p->taps == 4) { SC_GO(T, 8, 4); }                                \
    else { SC_GO(T, 8, 0); }                                                  \
  } while (0)
  if (f32) { SC_V(float); } else { SC_V(__hip_bfloat16); }
#undef SC_V
#undef SC_GO
}
