// Rows of two bf16 operands straight from global memory into LDS.
//
// A stage is 64 k of every row: 128 bytes, as 8 pieces of 16.  One wave
// instruction brings 8 rows (lane = row * 8 + place); the piece stored at place p
// of row r is p ^ (r & 7), so that the 16 rows of an MFMA fragment are read from
// different banks.
#pragma once
#include "mfma_util.h"

constexpr int BK = 64;

// 16 bytes per lane from base + off to 16 * lane past the wave's LDS address.
// Not the compiler's builtin: it would wait for the data before any LDS read.
DEV_INLINE void load_lds16(const uint32_t off, const void* base,
                           const uint32_t lds) {
  asm volatile("s_mov_b32 m0, %2\n\ts_nop 0\n\t"
               "global_load_lds_dwordx4 %0, %1"
               :: "v"(off), "s"(base), "s"(lds) : "memory", "m0");
}

// All but this wave's N youngest loads are in LDS, and every wave is here.
template <int N>
DEV_INLINE void landed_barrier() {
  asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)\n\ts_barrier"
               :: "n"(N) : "memory");
}

DEV_INLINE int stage_piece() {          // this lane's piece of its rows
  const int lane = threadIdx.x & 63;
  return (lane & 7) ^ (lane >> 3);
}

// elements from a fragment row's start to its pieces for half h of the stage
DEV_INLINE int stage_at(const int h) {
  const int lane = threadIdx.x & 63;
  return ((h * 4 + (lane >> 4)) ^ (lane & 7)) * 8;
}

// how far (bytes) the last, partial stage steps back so that no piece passes
// the row's end; what it repeats is masked
DEV_INLINE uint32_t tail_back(const int rest) {
  return (uint32_t)max(stage_piece() * 8 - (rest - 8), 0) * 2;
}

// BM rows of x against 64 rows of w by 4 waves, NB stages deep: each wave gets
// 16 rows of w (registers: 4 neighbours of them, lane & 15: row of x).  For
// products that stream w: few rows of x, all of memory's latency in flight.
//   xo[c], wo[c]  byte offset, from xb or wb, of row c * 32 + stream_row() at
//                 this lane's piece
//   start         stage to begin with: workgroups that start apart do not ask
//                 the same memory channels at once
//   live          16-row tiles of x that exist
template <int BM, int NB>
struct LdsStream {
  static constexpr int XI = BM / 32, L = XI + 2, TM = BM / 16;
  static constexpr int STAGE = (BM + 64) * BK;          // elements
  static constexpr int BYTES = NB * STAGE * 2;

  static DEV_INLINE int row() {
    return (threadIdx.x >> 6) * 8 + ((threadIdx.x & 63) >> 3);
  }

  static DEV_INLINE void run(const void* xb, const uint32_t (&xo)[XI],
                             const void* wb, const uint32_t (&wo)[2],
                             const int k, const int start, const int live,
                             char* smem, f32x4 (&acc)[TM]) {
    const __hip_bfloat16* lds = (const __hip_bfloat16*)smem;
    const int gl = threadIdx.x & 15, gs = (threadIdx.x & 63) >> 4;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const uint32_t to = __builtin_amdgcn_readfirstlane(
        (uint32_t)(uintptr_t)smem + wave * 1024);
    const int rest = k % BK, n = k / BK + (rest ? 1 : 0);
    const uint32_t back = rest ? tail_back(rest) : 0;
    auto stage = [&](int i) {
      const int s = i + start;
      return s >= n ? s - n : s;
    };
    auto issue = [&](int i) {
      const int s = stage(i);
      const uint32_t at = to + (i % NB) * STAGE * 2;
      const uint32_t less = rest && s == n - 1 ? back : 0;
#pragma unroll
      for (int c = 0; c < XI; ++c)
        load_lds16(xo[c] - less, (const char*)xb + s * BK * 2, at + c * 4096);
#pragma unroll
      for (int c = 0; c < 2; ++c)
        load_lds16(wo[c] - less, (const char*)wb + s * BK * 2,
                   at + BM * BK * 2 + c * 4096);
    };
#pragma unroll
    for (int j = 0; j < TM; ++j) acc[j] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NB - 1; ++i)
      if (i < n) issue(i);
    for (int i = 0; i < n; ++i) {
      if (i + NB - 2 < n) landed_barrier<L * (NB - 2)>();
      else landed_barrier<0>();
      // the buffer of stage i - 1 is read: the barrier is behind it
      if (i + NB - 1 < n) issue(i + NB - 1);
      const __hip_bfloat16* xs = lds + (i % NB) * STAGE + gl * BK;
      const __hip_bfloat16* ws = lds + (i % NB) * STAGE +
                                 (BM + wave * 16 + gl) * BK;
      mf_bf8 a[2], b[2][TM];
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        a[h] = frag8(ws + stage_at(h));
#pragma unroll
        for (int j = 0; j < TM; ++j)
          if (j < live) b[h][j] = frag8(xs + j * 16 * BK + stage_at(h));
      }
      if (rest && stage(i) == n - 1) {
        const mf_bf8 z = {};
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          const bool on = h * 32 + gs * 8 < rest;
          a[h] = on ? a[h] : z;
#pragma unroll
          for (int j = 0; j < TM; ++j) b[h][j] = on ? b[h][j] : z;
        }
      }
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int j = 0; j < TM; ++j)
          if (j < live) acc[j] = mfma_bf16_k32(a[h], b[h][j], acc[j]);
    }
  }
};
