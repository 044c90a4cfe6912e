// f32 residual stream: residual add, grouped RMS norm under one or two weights,
// and the causal input convolution.
//
// The stream x [T, W] stays f32 end to end; what the projections read is
// written in the activation dtype (bf16 or f32).  One workgroup per token row:
// the row is added, kept in LDS, reduced per group and written under both
// norms, so the stream is read and written once per layer.  In decode the
// convolution of the mixer's input rides in the same kernel: a thread owns its
// channels, reads their taps-1 past inputs from the sequence's state slot and
// writes the shifted history back.  In prefill the neighbours' rows must exist
// first, so the convolution is a kernel of its own over 16-token tiles.
#include "vec_io.h"

namespace {

constexpr int NT = 256;

// CONV: n1 becomes n1 + conv(n1) with the history of state slot slots[row]
// (all zeros at position 0), and the history moves on by one token.
template <typename T, int V, bool CONV, int NT>
__global__ __launch_bounds__(NT) void stream_norm_kernel(
    float* __restrict__ x, const T* __restrict__ delta,
    const float* __restrict__ w1, const float* __restrict__ w2,
    T* __restrict__ n1, T* __restrict__ n2, const int width, const int groups,
    const float eps, const float* __restrict__ conv_w,
    T* __restrict__ conv_state, const int* __restrict__ slots,
    const int* __restrict__ positions, const int taps) {
  constexpr int NW = NT / 64;
  extern __shared__ float smem[];
  const int sub = groups >= NW ? 1 : (NW + groups - 1) / groups;
  float* row = smem;                    // [width]
  float* part = smem + width;           // [groups * sub]
  float* inv = part + groups * sub;     // [groups]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const size_t base = (size_t)blockIdx.x * width;
  const int gs = width / groups;

  for (int i = tid * V; i < width; i += NT * V) {
    float v[V];
    load_vec<V>(x + base + i, v);
    if (delta != nullptr) {
      float d[V];
      load_vec<V>(delta + base + i, d);
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] += d[j];
      store_vec<V>(x + base + i, v);
    }
#pragma unroll
    for (int j = 0; j < V; ++j) row[i + j] = v[j];
  }
  __syncthreads();
  const int seg = (gs + sub - 1) / sub;
  for (int it = wave; it < groups * sub; it += NW) {
    const int g = it / sub, s = it % sub;
    const int lo = g * gs + s * seg, hi = min(lo + seg, (g + 1) * gs);
    float ss = 0.f;
    for (int i = lo + lane; i < hi; i += 64) ss += row[i] * row[i];
    ss = wave_sum(ss);
    if (lane == 0) part[it] = ss;
  }
  __syncthreads();
  for (int g = tid; g < groups; g += NT) {
    float ss = 0.f;
    for (int s = 0; s < sub; ++s) ss += part[g * sub + s];
    inv[g] = 1.f / sqrtf(ss / gs + eps);
  }
  __syncthreads();

  const size_t hist =
      CONV ? (size_t)slots[blockIdx.x] * (taps - 1) * width : 0;
  const bool fresh = CONV ? positions[blockIdx.x] == 0 : false;
  for (int i = tid * V; i < width; i += NT * V) {
    float y[V], wv[V];
    const float sc = inv[i / gs];        // V divides gs
    load_vec<V>(w1 + i, wv);
#pragma unroll
    for (int j = 0; j < V; ++j) y[j] = row[i + j] * sc * wv[j];
    if (CONV) {
      float h[V], cw[V];
#pragma unroll
      for (int j = 0; j < V; ++j) h[j] = y[j] = round_to<T>(y[j]);
      load_vec<V>(conv_w + (size_t)(taps - 1) * width + i, cw);
#pragma unroll
      for (int j = 0; j < V; ++j) h[j] += cw[j] * y[j];
      for (int p = 0; p < taps - 1; ++p) {
        float past[V];
        T* st = conv_state + hist + (size_t)p * width + i;
        if (fresh) {
#pragma unroll
          for (int j = 0; j < V; ++j) past[j] = 0.f;
        } else {
          load_vec<V>(st, past);
        }
        load_vec<V>(conv_w + (size_t)p * width + i, cw);
#pragma unroll
        for (int j = 0; j < V; ++j) h[j] += cw[j] * past[j];
        if (p > 0) store_vec<V>(st - width, past);
      }
      if (taps > 1)
        store_vec<V>(conv_state + hist + (size_t)(taps - 2) * width + i, y);
      store_vec<V>(n1 + base + i, h);
    } else {
      store_vec<V>(n1 + base + i, y);
    }
    if (w2 != nullptr) {
      load_vec<V>(w2 + i, wv);
#pragma unroll
      for (int j = 0; j < V; ++j) y[j] = row[i + j] * sc * wv[j];
      store_vec<V>(n2 + base + i, y);
    }
  }
}

// h = x + conv(x) over varlen sequences.  tiles [n, 2] = (sequence, first
// token of the tile inside the sequence's rows).  Only a sequence's first
// tile reads its history (the host keeps tile >= taps - 1), and that same
// thread writes the new history afterwards, so no other workgroup races it.
// TAPS > 0: the taps' weights and the last inputs live in registers, so that a
// row is read once; 0: any number of taps.
template <typename T, int V, int TAPS>
__global__ __launch_bounds__(NT) void causal_conv_kernel(
    T* __restrict__ out, const T* __restrict__ x,
    const float* __restrict__ w, T* __restrict__ state,
    const int* __restrict__ tiles, const int* __restrict__ cu,
    const int* __restrict__ starts, const int* __restrict__ slots,
    const int tile, const int width, const int taps) {
  const int seq = tiles[blockIdx.x * 2], t0 = tiles[blockIdx.x * 2 + 1];
  const int row0 = cu[seq], len = cu[seq + 1] - row0;
  const int i = (blockIdx.y * NT + threadIdx.x) * V;
  if (i >= width) return;
  const bool fresh = starts[seq] == 0;
  T* hist = state + (size_t)slots[seq] * (taps - 1) * width + i;
  const T* xs = x + (size_t)row0 * width + i;
  const int t1 = min(t0 + tile, len);
  // input at row src of this step; before it the history, or zeros
  auto past = [&](int src, float* v) {
    if (src >= 0) {
      load_vec<V>(xs + (size_t)src * width, v);
    } else if (fresh) {
#pragma unroll
      for (int j = 0; j < V; ++j) v[j] = 0.f;
    } else {
      load_vec<V>(hist + (size_t)(src + taps - 1) * width, v);
    }
  };
  if constexpr (TAPS > 0) {
    float cw[TAPS][V], win[TAPS][V];
#pragma unroll
    for (int p = 0; p < TAPS; ++p)
      load_vec<V>(w + (size_t)p * width + i, cw[p]);
#pragma unroll
    for (int p = 1; p < TAPS; ++p) past(t0 - TAPS + p, win[p]);
#pragma unroll 4
    for (int t = t0; t < t1; ++t) {
#pragma unroll
      for (int p = 1; p < TAPS; ++p)
#pragma unroll
        for (int j = 0; j < V; ++j) win[p - 1][j] = win[p][j];
      load_vec<V>(xs + (size_t)t * width, win[TAPS - 1]);
      float h[V];
#pragma unroll
      for (int j = 0; j < V; ++j) {
        h[j] = win[TAPS - 1][j];
#pragma unroll
        for (int p = 0; p < TAPS; ++p) h[j] += cw[p][j] * win[p][j];
      }
      store_vec<V>(out + ((size_t)row0 + t) * width + i, h);
    }
  } else {
    for (int t = t0; t < t1; ++t) {
      float h[V], cw[V], v[V];
      load_vec<V>(xs + (size_t)t * width, h);
      for (int p = 0; p < taps; ++p) {
        past(t - taps + 1 + p, v);
        load_vec<V>(w + (size_t)p * width + i, cw);
#pragma unroll
        for (int j = 0; j < V; ++j) h[j] += cw[j] * v[j];
      }
      store_vec<V>(out + ((size_t)row0 + t) * width + i, h);
    }
  }
  if (t0 == 0) {
    // ascending order: entry p is read (as p + len) no later than overwritten
    for (int p = 0; p < taps - 1; ++p) {
      float v[V];
      past(len - (taps - 1) + p, v);
      store_vec<V>(hist + (size_t)p * width, v);
    }
  }
}

template <typename T>
void stream_norm_t(float* x, const void* delta, const float* w1,
                   const float* w2, void* n1, void* n2, int tokens, int width,
                   int groups, float eps, const float* conv_w, void* state,
                   const int* slots, const int* positions, int taps,
                   hipStream_t s) {
  const int nt = width >= 4096 ? 512 : 256, nw = nt / 64;
  const int sub = groups >= nw ? 1 : (nw + groups - 1) / groups;
  const size_t lds = sizeof(float) * (width + groups * sub + groups);
  const bool vec = (width / groups) % 8 == 0;
#define SN_GO(V, C, N)                                                        \
  stream_norm_kernel<T, V, C, N><<<tokens, N, lds, s>>>(                      \
      x, (const T*)delta, w1, w2, (T*)n1, (T*)n2, width, groups, eps, conv_w, \
      (T*)state, slots, positions, taps)
#define SN_VC(V, C)                                                           \
  do {                                                                        \
    if (nt == 512) { SN_GO(V, C, 512); } else { SN_GO(V, C, 256); }           \
  } while (0)
  if (conv_w != nullptr) {
    if (vec) SN_VC(8, true); else SN_VC(1, true);
  } else {
    if (vec) SN_VC(8, false); else SN_VC(1, false);
  }
#undef SN_GO
#undef SN_VC
}

}  // namespace

extern "C" {

void launch_stream_norm(float* x, const void* delta, const float* w1,
                        const float* w2, void* n1, void* n2, int tokens,
                        int width, int groups, float eps, const float* conv_w,
                        void* state, const int* slots, const int* positions,
                        int taps, int f32, hipStream_t s) {
  if (f32)
    stream_norm_t<float>(x, delta, w1, w2, n1, n2, tokens, width, groups, eps,
                         conv_w, state, slots, positions, taps, s);
  else
    stream_norm_t<__hip_bfloat16>(x, delta, w1, w2, n1, n2, tokens, width,
                                  groups, eps, conv_w, state, slots, positions,
                                  taps, s);
}

void launch_causal_conv(void* out, const void* x, const float* w, void* state,
                        const int* tiles, const int* cu, const int* starts,
                        const int* slots, int n_tiles, int tile, int width,
                        int taps, int f32, hipStream_t s) {
  const int v = width % 8 == 0 ? 8 : 1;
  const dim3 grid(n_tiles, (width / v + NT - 1) / NT);
#define CC_GO(T, V, N) causal_conv_kernel<T, V, N><<<grid, NT, 0, s>>>(       \
      (T*)out, (const T*)x, w, (T*)state, tiles, cu, starts, slots, tile,     \
      width, taps)
#define CC_V(T)                                                               \
  do {                                                                        \
    if (v == 1) { CC_GO(T, 1, 0); }                                           \
    else if (taps == 2) { CC_GO(T, 8, 2); }                                   \
    else if (taps == 3) { CC_GO(T, 8, 3); }                                   \
    else if (taps == 4) { CC_GO(T, 8, 4); }                                   \
    else { CC_GO(T, 8, 0); }                                                  \
  } while (0)
  if (f32) { CC_V(float); } else { CC_V(__hip_bfloat16); }
#undef CC_V
#undef CC_GO
}

}  // extern "C"
