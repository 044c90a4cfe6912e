// What the chunked delta rules share: the record a chunk leaves for the scan, the
// scan over chunks, and the head norm with its gate.
//
// A rule is brought to the form (S before the chunk, V its values)
//   P  = TU S + TM V
//   O  = R S + QB P           (DIRECT: + QK V)
//   S' = DC S + BT P          (DIRECT: + KT V)
// with everything but S, P and O formed beforehand, per chunk and head, by a
// rule's own prep kernel.
#pragma once
#include "mfma_util.h"
#include "vec_io.h"

struct DeltaScanArgs {
  const void* v;          // + row*v_row + head*dv
  float* state;           // [slots, heads, dk, dv]
  const int* slots;       // [seqs]
  const int* cu;          // [seqs+1] rows
  const int* starts;      // [seqs] position of the first row
  const int* chunk_cu;    // [seqs+1] chunks
  const float* ws;        // [chunks, heads] records
  float* o;               // [rows, heads*dv]
  long v_row;
  int heads, dk, dv;
};

struct DeltaOutArgs {
  const float* o;         // [rows, heads*dv]
  const void* gate;       // + row*g_row + head*dv
  const float* norm_w;    // + head*w_head
  void* out;              // + row*o_row + head*dv
  long g_row, o_row;
  int heads, dv, w_head;
  int silu;               // gate: silu, else sigmoid
  float eps;
};

namespace {

constexpr int C = 16;                   // tokens per chunk
constexpr int SP = C + 4;               // row pitch of [.][16] arrays

// one chunk-head's record in the workspace, in floats: the image that the scan
// keeps in LDS, row pitches included
template <int DP, bool DIRECT> struct Rec {
  static constexpr int PP = DP + 4;               // pitch of [16][DP] arrays
  static constexpr int TU = 0;                    // [16][DP]
  static constexpr int R = TU + C * PP;           // [16][DP]
  static constexpr int BT = R + C * PP;           // [DP][16]
  static constexpr int TM = BT + DP * SP;         // [16][16]
  static constexpr int QB = TM + C * SP;          // [16][16]
  static constexpr int DC = QB + C * SP;          // [DP]
  static constexpr int KT = DC + DP;              // [DP][16], DIRECT only
  static constexpr int QK = KT + DP * SP;         // [16][16], DIRECT only
  static constexpr int SIZE = DIRECT ? QK + C * SP : KT;
};

// grid (heads, seqs, column groups).  A workgroup is NC column groups of 16
// value columns by KS parts of the key rows: wave (kp, cg) keeps its rows of
// its columns of S.  With KS = 2 the parts' shares of P and O meet in LDS.
// A record's loads fly under two chunks' MFMAs and land in the other half of
// LDS.
template <typename T, int DP, int KS, int NC, bool DIRECT>
__global__ __launch_bounds__(KS * NC * 64) void delta_scan_kernel(
    const DeltaScanArgs p) {
  typedef Rec<DP, DIRECT> W;
  constexpr int PP = W::PP, NT = KS * NC * 64, TT = DP / 16 / KS;
  constexpr int V4 = W::SIZE / 4, PER = (V4 + NT - 1) / NT;
  extern __shared__ __attribute__((aligned(16))) float smem[];
  f32x4* xch = reinterpret_cast<f32x4*>(smem + 2 * W::SIZE);  // [2][KS*NC*64]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int cg = wave % NC, kp = wave / NC;
  const int head = blockIdx.x, seq = blockIdx.y;
  const int D = p.dk, DV = p.dv, HD = p.heads * DV;
  const int vcol = (blockIdx.z * NC + cg) * 16 + gl;
  const bool vlive = vcol < DV;
  const int vc = min(vcol, DV - 1);
  const int row0 = p.cu[seq], len = p.cu[seq + 1] - row0;
  const int ch0 = p.chunk_cu[seq], nch = p.chunk_cu[seq + 1] - ch0;
  const bool fresh = p.starts[seq] == 0;
  float* S = p.state + ((size_t)p.slots[seq] * p.heads + head) * D * DV;
  const int k0 = kp * TT * 16;                  // this wave's key rows

  f32x4 s[TT];
#pragma unroll
  for (int t = 0; t < TT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int kr = k0 + t * 16 + gs * 4 + r;
      s[t][r] = !fresh && vlive && kr < D ? S[(size_t)kr * DV + vcol] : 0.f;
    }

  f32x4 stage[2][PER];
  float v[4], vn[2][4];
#define DC_FETCH(c, h)                                                        \
  do {                                                                        \
    const f32x4* src = reinterpret_cast<const f32x4*>(                        \
        p.ws + ((size_t)(ch0 + (c)) * p.heads + head) * W::SIZE);             \
    _Pragma("unroll") for (int i = 0; i < PER; ++i)                           \
      stage[h][i] = src[min(tid + i * NT, V4 - 1)];                           \
    _Pragma("unroll") for (int r = 0; r < 4; ++r) {                           \
      const int t = (c) * C + gs * 4 + r;                                     \
      vn[h][r] = to_f(((const T*)p.v)[                                        \
          (size_t)(row0 + min(t, len - 1)) * p.v_row + head * DV + vc]);      \
      if (t >= len || !vlive) vn[h][r] = 0.f;                                 \
    }                                                                         \
  } while (0)
#define DC_LAND(half)                                                         \
  do {                                                                        \
    f32x4* dst = reinterpret_cast<f32x4*>(smem + (half) * W::SIZE);           \
    _Pragma("unroll") for (int i = 0; i < PER; ++i)                           \
      if (tid + i * NT < V4) dst[tid + i * NT] = stage[half][i];              \
    _Pragma("unroll") for (int r = 0; r < 4; ++r) v[r] = vn[half][r];         \
  } while (0)
  DC_FETCH(0, 0);
  DC_LAND(0);
  DC_FETCH(min(1, nch - 1), 1);
  __syncthreads();
  for (int cc = 0; cc < nch; cc += 2)
#pragma unroll
  for (int h = 0; h < 2; ++h) {
    const int c = cc + h;
    if (c >= nch) break;
    const float* rec = smem + h * W::SIZE;
    // always: a skipped load would make the waits below drain every load
    DC_FETCH(min(c + 2, nch - 1), h);

    // P and O over the old state, two products side by side
    f32x4 pa = {0.f, 0.f, 0.f, 0.f}, oa = pa;
    if (kp == 0) {
      float x[4], y[4];
      load_vec<4>(rec + W::TM + gl * SP + gs * 4, x);
      if constexpr (DIRECT) load_vec<4>(rec + W::QK + gl * SP + gs * 4, y);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        pa = mfma_f32_k4(x[r], v[r], pa);
        if constexpr (DIRECT) oa = mfma_f32_k4(y[r], v[r], oa);
      }
    }
#pragma unroll
    for (int t = 0; t < TT; ++t) {
      float x[4], y[4];
      load_vec<4>(rec + W::TU + gl * PP + k0 + t * 16 + gs * 4, x);
      load_vec<4>(rec + W::R + gl * PP + k0 + t * 16 + gs * 4, y);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        pa = mfma_f32_k4(x[r], s[t][r], pa);
        oa = mfma_f32_k4(y[r], s[t][r], oa);
      }
    }
    if constexpr (KS == 2) {
      xch[wave * 64 + lane] = pa;
      if (kp == 1) xch[(KS * NC + cg) * 64 + lane] = oa;
    }
    // the decay and k v^T parts do not wait for P
#pragma unroll
    for (int t = 0; t < TT; ++t) {
      float x[4], d[4];
      load_vec<4>(rec + W::DC + k0 + t * 16 + gs * 4, d);
#pragma unroll
      for (int r = 0; r < 4; ++r) s[t][r] *= d[r];
      if constexpr (DIRECT) {
        load_vec<4>(rec + W::KT + (k0 + t * 16 + gl) * SP + gs * 4, x);
#pragma unroll
        for (int r = 0; r < 4; ++r) s[t] = mfma_f32_k4(x[r], v[r], s[t]);
      }
    }
    if constexpr (KS == 2) {
      __syncthreads();
      const f32x4 p0 = xch[cg * 64 + lane], p1 = xch[(NC + cg) * 64 + lane];
      pa = p0 + p1;
      if (kp == 0) oa += xch[(KS * NC + cg) * 64 + lane];
    }
#pragma unroll
    for (int t = 0; t < TT; ++t) {
      float y[4];
      load_vec<4>(rec + W::BT + (k0 + t * 16 + gl) * SP + gs * 4, y);
#pragma unroll
      for (int r = 0; r < 4; ++r) s[t] = mfma_f32_k4(y[r], pa[r], s[t]);
    }
    if (kp == 0) {
      float y[4];
      load_vec<4>(rec + W::QB + gl * SP + gs * 4, y);
#pragma unroll
      for (int r = 0; r < 4; ++r) oa = mfma_f32_k4(y[r], pa[r], oa);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = c * C + gs * 4 + r;
        if (t < len && vlive)
          p.o[(size_t)(row0 + t) * HD + head * DV + vcol] = oa[r];
      }
    }
    DC_LAND(1 - h);
    __syncthreads();
  }
#undef DC_FETCH
#undef DC_LAND
#pragma unroll
  for (int t = 0; t < TT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int kr = k0 + t * 16 + gs * 4 + r;
      if (vlive && kr < D) S[(size_t)kr * DV + vcol] = s[t][r];
    }
}

DEV_INLINE float delta_gate(float z, int silu) {
  const float s = sigmoid_f(z);
  return silu ? z * s : s;
}

// out = o / rms(o) * norm_w * gate.  vec: dv is 4 * LPI for a power of two LPI,
// and LPI lanes take a row of a head; else one wave does.
template <typename T, int LPI>
__global__ __launch_bounds__(256) void delta_out_vec_kernel(
    const DeltaOutArgs p, const long items) {
  const int lane = threadIdx.x & 63;
  const long item = (blockIdx.x * 4L + (threadIdx.x >> 6)) * (64 / LPI) +
                    lane / LPI;
  const int d = (lane % LPI) * 4;
  const long it = item < items ? item : items - 1;
  const int head = (int)(it % p.heads);
  const long row = it / p.heads;
  float x[4], w[4];
  load_vec<4>(p.o + it * (LPI * 4) + d, x);
  float ss = 0.f;
#pragma unroll
  for (int r = 0; r < 4; ++r) ss += x[r] * x[r];
#pragma unroll
  for (int off = LPI / 2; off >= 1; off >>= 1) ss += __shfl_xor(ss, off, 64);
  const float inv = 1.f / sqrtf(ss / (LPI * 4) + p.eps);
  const int col = head * LPI * 4 + d;
  load_vec<4>(p.norm_w + head * p.w_head + d, w);
  if (item >= items) return;
  const T* g = (const T*)p.gate + row * p.g_row + col;
  T* out = (T*)p.out + row * p.o_row + col;
  if constexpr (sizeof(T) == 2) {
    union { uint2 u; __hip_bfloat16 e[4]; } gv, ov;
    gv.u = *reinterpret_cast<const uint2*>(g);
#pragma unroll
    for (int r = 0; r < 4; ++r)
      ov.e[r] = f2bf(x[r] * inv * w[r] * delta_gate(bf2f(gv.e[r]), p.silu));
    *reinterpret_cast<uint2*>(out) = ov.u;
  } else {
    float gv[4];
    load_vec<4>((const float*)g, gv);
#pragma unroll
    for (int r = 0; r < 4; ++r)
      gv[r] = x[r] * inv * w[r] * delta_gate(gv[r], p.silu);
    store_vec<4>((float*)out, gv);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void delta_out_kernel(
    const DeltaOutArgs p, const long items) {
  const long item = blockIdx.x * 4L + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (item >= items) return;
  const int head = (int)(item % p.heads);
  const long row = item / p.heads;
  const int D = p.dv;
  const float* src = p.o + item * D;
  float ss = 0.f;
  for (int d = lane; d < D; d += 64) ss += src[d] * src[d];
  const float inv = 1.f / sqrtf(wave_sum(ss) / D + p.eps);
  const T* g = (const T*)p.gate + row * p.g_row + head * D;
  T* out = (T*)p.out + row * p.o_row + head * D;
  for (int d = lane; d < D; d += 64)
    out[d] = from_f<T>(src[d] * inv * p.norm_w[head * p.w_head + d] *
                       delta_gate(to_f(g[d]), p.silu));
}

template <typename T, int DP, int KS, int NC, bool DIRECT>
void delta_scan(const DeltaScanArgs& p, int seqs, hipStream_t s) {
  constexpr int NT = KS * NC * 64;
  const int zs = (p.dv + NC * 16 - 1) / (NC * 16);
  const size_t lds = 2 * Rec<DP, DIRECT>::SIZE * sizeof(float) +
                     (KS == 2 ? (size_t)(KS + 1) * NC * 64 * 16 : 0);
  static bool once = false;
  if (!once) {
    (void)hipFuncSetAttribute(
        (const void*)delta_scan_kernel<T, DP, KS, NC, DIRECT>,
        hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    once = true;
  }
  hipLaunchKernelGGL((delta_scan_kernel<T, DP, KS, NC, DIRECT>),
                     dim3(p.heads, seqs, zs), NT, lds, s, p);
}

template <typename T>
void delta_out(const DeltaOutArgs& p, long rows, hipStream_t s) {
  const long items = rows * p.heads;
  const bool vec = p.g_row % 4 == 0 && p.o_row % 4 == 0 &&
                   ((uintptr_t)p.gate & (4 * sizeof(T) - 1)) == 0 &&
                   ((uintptr_t)p.out & (4 * sizeof(T) - 1)) == 0;
#define DO_GO(DV)                                                             \
  do {                                                                        \
    const long per = 4L * (64 / (DV / 4));                                    \
    hipLaunchKernelGGL((delta_out_vec_kernel<T, DV / 4>),                     \
                       (int)((items + per - 1) / per), 256, 0, s, p, items);  \
  } while (0)
  if (vec && p.dv == 32) DO_GO(32);
  else if (vec && p.dv == 64) DO_GO(64);
  else if (vec && p.dv == 128) DO_GO(128);
  else if (vec && p.dv == 256) DO_GO(256);
  else
    hipLaunchKernelGGL((delta_out_kernel<T>), (int)((items + 3) / 4), 256, 0, s,
                       p, items);
#undef DO_GO
}

}  // namespace
