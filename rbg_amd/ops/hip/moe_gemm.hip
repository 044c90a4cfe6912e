// Grouped products of a step's (token, choice) rows with their experts' weights
// (gfx950): out[row, n] = sum_k x[row, k] w[expert, n, k], rows in expert order,
// a tile of rows per expert (moe_route.hip).  The number of tiles is on the
// device; launches cover the most there can be and the rest leaves at once.
//
//   tiled   128 rows x 128 or 192 columns, 64 k a step, both operands straight
//           from global memory into LDS (rows may be gathered: every lane brings
//           its own address).  One buffer: the other workgroups of the CU, three
//           or four of them, compute while one waits, which measured better than
//           two buffers with half the workgroups.  16-byte pieces of a row are
//           stored swizzled by the row: fragment reads are free of conflicts.
//   skinny  decode: 16 * MT rows against 16 * NN weight rows, whose fragments go
//           from global memory into the MFMAs; waves split K and meet in LDS.
//   rows    any sizes, bf16 or f32: a thread per column, up to 16 rows at once.
#include "mfma_util.h"
#include "moe_args.h"
#include "vec_io.h"

namespace {

DEV_INLINE float relu2_f(float x) {
  x = fmaxf(x, 0.f);
  return x * x;
}

// four neighbouring columns of one row
DEV_INLINE void put4(const MoeGemmArgs& p, const size_t row, const int n,
                     f32x4 v) {
  union { uint2 u; __hip_bfloat16 e[4]; } o;
#pragma unroll
  for (int r = 0; r < 4; ++r) o.e[r] = f2bf(p.relu2 ? relu2_f(v[r]) : v[r]);
  *reinterpret_cast<uint2*>((__hip_bfloat16*)p.out + row * p.n + n) = o.u;
}

constexpr int BM = 128, BK = 64, GT = 256;

// 16 bytes per lane from base + off to 16 * lane past the wave's LDS address.
// Not the compiler's builtin: it would wait for the data before any LDS read.
DEV_INLINE void load_lds16(const uint32_t off, const void* base,
                           const uint32_t lds) {
  asm volatile("s_mov_b32 m0, %2\n\ts_nop 0\n\t"
               "global_load_lds_dwordx4 %0, %1"
               :: "v"(off), "s"(base), "s"(lds) : "memory", "m0");
}

// what this wave asked for is in LDS, and every wave is here
DEV_INLINE void landed_barrier() {
  asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory");
}

// 4 waves of 64 rows x BN / 2 columns
template <int BN, int OCC>
__global__ __launch_bounds__(GT, OCC)
void moe_tiled_kernel(const MoeGemmArgs p) {
  constexpr int TN = BN / 32, XI = BM / 32, WI = BN / 32;
  __shared__ __attribute__((aligned(16)))
  __hip_bfloat16 lds[(BM + BN) * BK];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int gl = lane & 15, gs = lane >> 4;

  // each XCD takes a run of tiles; inside it, up to 4 row tiles share the
  // weight columns they walk together
  const int n_tiles = *p.count, nb = (p.n + BN - 1) / BN;
  const int total = n_tiles * nb, per = (total + 7) / 8;
  const int idx = blockIdx.x >> 3, work = (blockIdx.x & 7) * per + idx;
  if (idx >= per || work >= total) return;
  const int g0 = work / (4 * nb) * 4, gn = min(4, n_tiles - g0);
  const int in = work - g0 * nb;
  const int* tile = p.tiles + (size_t)(g0 + in % gn) * 3;
  const int n0 = in / gn * BN;
  const int expert = tile[0], row0 = tile[1], rows = tile[2];

  // wave-instruction c brings rows c*32 + wave*8 .. +7, 8 pieces of 16 bytes
  // each; a lane's row is fixed modulo 8, so its piece number is too
  const int lr = lane >> 3, piece = (lane & 7) ^ lr;
  uint32_t xo[XI], wo[WI];                      // bytes; the host checks sizes
#pragma unroll
  for (int c = 0; c < XI; ++c) {
    const int at = row0 + min(c * 32 + wave * 8 + lr, rows - 1);
    xo[c] = ((uint32_t)(p.rows != nullptr ? p.rows[at] : at) * p.k +
             piece * 8) * 2;
  }
#pragma unroll
  for (int c = 0; c < WI; ++c)
    wo[c] = ((uint32_t)min(n0 + c * 32 + wave * 8 + lr, p.n - 1) * p.k +
             piece * 8) * 2;
  const char* xb = (const char*)p.x;
  const char* wb = (const char*)p.w + (size_t)expert * p.n * p.k * 2;
  const uint32_t to = __builtin_amdgcn_readfirstlane(
      (uint32_t)(uintptr_t)lds + wave * 1024);
  auto issue = [&](int kt) {
#pragma unroll
    for (int c = 0; c < XI; ++c)
      load_lds16(xo[c], xb + kt * BK * 2, to + c * 4096);
#pragma unroll
    for (int c = 0; c < WI; ++c)
      load_lds16(wo[c], wb + kt * BK * 2, to + BM * BK * 2 + c * 4096);
  };
  const int wm = (wave >> 1) * 64, wn = (wave & 1) * (BN / 2);
  f32x4 acc[TN][4];
#pragma unroll
  for (int i = 0; i < TN; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = {0.f, 0.f, 0.f, 0.f};
  const __hip_bfloat16* xs = lds + (wm + gl) * BK;
  const __hip_bfloat16* ws = lds + (BM + wn + gl) * BK;
  auto compute = [&](int k_left) {
    const mf_bf8 z = {};
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      const int at = ((h * 4 + gs) ^ (gl & 7)) * 8;
      mf_bf8 a[TN], b[4];
#pragma unroll
      for (int i = 0; i < TN; ++i) a[i] = frag8(ws + i * 16 * BK + at);
#pragma unroll
      for (int j = 0; j < 4; ++j) b[j] = frag8(xs + j * 16 * BK + at);
      if (k_left < BK) {
        const bool on = h * 32 + gs * 8 < k_left;
#pragma unroll
        for (int i = 0; i < TN; ++i) a[i] = on ? a[i] : z;
#pragma unroll
        for (int j = 0; j < 4; ++j) b[j] = on ? b[j] : z;
      }
      __builtin_amdgcn_s_setprio(1);
#pragma unroll
      for (int i = 0; i < TN; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[i][j] = mfma_bf16_k32(a[i], b[j], acc[i][j]);
      __builtin_amdgcn_s_setprio(0);
    }
  };
  const int nk = p.k / BK, rest = p.k % BK;
  for (int kt = 0; kt < nk; ++kt) {
    issue(kt);
    landed_barrier();
    compute(BK);
    landed_barrier();                           // everyone has read
  }
  if (rest) {                                   // pieces past the end: the last
    const int back = max(piece * 8 - (rest - 8), 0) * 2;
#pragma unroll
    for (int c = 0; c < XI; ++c) xo[c] -= back;
#pragma unroll
    for (int c = 0; c < WI; ++c) wo[c] -= back;
    issue(nk);
    landed_barrier();
    compute(rest);
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = wm + j * 16 + gl;
    if (r >= rows) continue;
#pragma unroll
    for (int i = 0; i < TN; ++i) {
      const int n = n0 + wn + i * 16 + gs * 4;
      if (n < p.n) put4(p, row0 + r, n, acc[i][j]);
    }
  }
}

template <int BN, int OCC>
void moe_tiled(const MoeGemmArgs& p, hipStream_t s) {
  const int nb = (p.n + BN - 1) / BN;
  moe_tiled_kernel<BN, OCC><<<8 * ((p.max_tiles * nb + 7) / 8), GT, 0, s>>>(p);
}

constexpr int SW = 4;                           // waves of a skinny workgroup
constexpr int UN = 4;                           // 32-k steps in flight

template <int MT, int NN>
__global__ __launch_bounds__(SW * 64) void moe_skinny_kernel(
    const MoeGemmArgs p) {
  __shared__ f32x4 red[SW][NN * MT][64];
  if ((int)blockIdx.y >= *p.count) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int* tile = p.tiles + (size_t)blockIdx.y * 3;
  const int expert = tile[0], row0 = tile[1], rows = tile[2];
  const int n0 = blockIdx.x * 16 * NN;
  const __hip_bfloat16* wr[NN];
#pragma unroll
  for (int n = 0; n < NN; ++n)
    wr[n] = (const __hip_bfloat16*)p.w +
            ((size_t)expert * p.n + min(n0 + n * 16 + gl, p.n - 1)) * p.k;
  const __hip_bfloat16* xr[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int r = row0 + min(t * 16 + gl, rows - 1);
    xr[t] = (const __hip_bfloat16*)p.x +
            (size_t)(p.rows != nullptr ? p.rows[r] : r) * p.k;
  }
  f32x4 acc[NN][MT];
#pragma unroll
  for (int n = 0; n < NN; ++n)
#pragma unroll
    for (int t = 0; t < MT; ++t) acc[n][t] = {0.f, 0.f, 0.f, 0.f};
  const int per = ((p.k + SW * 32 - 1) / (SW * 32)) * 32;
  const int kb = wave * per, ke = min(kb + per, p.k);
  for (int k0 = kb; k0 < ke; k0 += 32 * UN) {
    // unconditional clamped loads, all before the first product: a guard would
    // serialise them
    mf_bf8 wf[UN][NN], xf[UN][MT];
    const mf_bf8 z = {};
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const int kc = min(k0 + u * 32 + gs * 8, p.k - 8);
#pragma unroll
      for (int n = 0; n < NN; ++n) wf[u][n] = frag8(wr[n] + kc);
#pragma unroll
      for (int t = 0; t < MT; ++t) xf[u][t] = frag8(xr[t] + kc);
    }
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const bool on = k0 + u * 32 + gs * 8 < ke;
#pragma unroll
      for (int n = 0; n < NN; ++n) {
        const mf_bf8 w = on ? wf[u][n] : z;
#pragma unroll
        for (int t = 0; t < MT; ++t)
          acc[n][t] = mfma_bf16_k32(w, xf[u][t], acc[n][t]);
      }
    }
  }
#pragma unroll
  for (int n = 0; n < NN; ++n)
#pragma unroll
    for (int t = 0; t < MT; ++t) red[wave][n * MT + t][lane] = acc[n][t];
  __syncthreads();
  for (int i = threadIdx.x; i < NN * MT * 64; i += SW * 64) {
    const int u = i >> 6, ln = i & 63;
    f32x4 s = red[0][u][ln];
#pragma unroll
    for (int wv = 1; wv < SW; ++wv) s += red[wv][u][ln];
    const int r = (u % MT) * 16 + (ln & 15);
    const int n = n0 + (u / MT) * 16 + (ln >> 4) * 4;
    if (r < rows && n < p.n) put4(p, row0 + r, n, s);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void moe_rows_kernel(const MoeGemmArgs p) {
  if ((int)blockIdx.y >= *p.count) return;
  const int* tile = p.tiles + (size_t)blockIdx.y * 3;
  const int expert = tile[0], row0 = tile[1], rows = tile[2];
  const int n = blockIdx.x * 256 + threadIdx.x;
  if (n >= p.n) return;
  const T* w = (const T*)p.w + ((size_t)expert * p.n + n) * p.k;
  const T* x[16];
  float acc[16];
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int at = row0 + min(r, rows - 1);
    x[r] = (const T*)p.x + (size_t)(p.rows != nullptr ? p.rows[at] : at) * p.k;
    acc[r] = 0.f;
  }
  for (int k = 0; k < p.k; ++k) {
    const float wv = to_f(w[k]);
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] += wv * to_f(x[r][k]);
  }
#pragma unroll
  for (int r = 0; r < 16; ++r)
    if (r < rows)
      ((T*)p.out)[(size_t)(row0 + r) * p.n + n] =
          from_f<T>(p.relu2 ? relu2_f(acc[r]) : acc[r]);
}

}  // namespace

extern "C" void launch_moe_gemm(const MoeGemmArgs* p, int f32, int vec,
                                hipStream_t s) {
  if (!vec) {                                   // tile <= 16
    const dim3 grid((p->n + 255) / 256, p->max_tiles);
    if (f32) {
      moe_rows_kernel<float><<<grid, 256, 0, s>>>(*p);
    } else {
      moe_rows_kernel<__hip_bfloat16><<<grid, 256, 0, s>>>(*p);
    }
  } else if (p->tile <= 16) {
    // wide workgroups once the experts alone fill the chip
    if (p->max_tiles >= 32) {
      moe_skinny_kernel<1, 2><<<dim3((p->n + 31) / 32, p->max_tiles), SW * 64,
                                0, s>>>(*p);
    } else {
      moe_skinny_kernel<1, 1><<<dim3((p->n + 15) / 16, p->max_tiles), SW * 64,
                                0, s>>>(*p);
    }
  } else if (p->tile <= 32) {
    moe_skinny_kernel<2, 2><<<dim3((p->n + 31) / 32, p->max_tiles), SW * 64, 0,
                              s>>>(*p);
  } else {
    // the wide form is 1.08 times as fast per column
    const long wide = (p->n + 191) / 192 * 192L, slim = (p->n + 127) / 128 * 128L;
    if (wide * 100 <= slim * 108) moe_tiled<192, 3>(*p, s);
    else moe_tiled<128, 4>(*p, s);
  }
}
