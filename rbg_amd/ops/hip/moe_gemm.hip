// Grouped products of a step's (token, choice) rows with their experts' weights
// (gfx950): out[row, n] = sum_k x[row, k] w[expert, n, k], rows in expert order,
// a tile of rows per expert (moe_route.hip).  The number of tiles is on the
// device; launches cover the most there can be and the rest leaves at once.
//
//   tiled   128 rows x 128 columns, 64 k a step, both operands straight from
//           global memory into double-buffered LDS (rows may be gathered: every
//           lane brings its own address).  16-byte pieces of a row are stored
//           swizzled by the row, which keeps fragment reads free of conflicts.
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

constexpr int BM = 128, BN = 128, BK = 64, GT = 256;
constexpr int STAGE = (BM + BN) * BK;           // elements of one buffer

DEV_INLINE void load_lds16(const __hip_bfloat16* g, __hip_bfloat16* l) {
  typedef __attribute__((address_space(1))) const void gvoid;
  typedef __attribute__((address_space(3))) void lvoid;
  __builtin_amdgcn_global_load_lds((gvoid*)(uintptr_t)g,
                                   (lvoid*)(uint32_t)(uintptr_t)l, 16, 0, 0);
}

__global__ __launch_bounds__(GT, 2) void moe_tiled_kernel(const MoeGemmArgs p) {
  extern __shared__ __attribute__((aligned(16))) char gemm_smem[];
  __hip_bfloat16* lds = (__hip_bfloat16*)gemm_smem;
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
  // each; lane's row is fixed modulo 8, so its piece number is too
  const int lr = lane >> 3, piece = (lane & 7) ^ lr;
  const __hip_bfloat16* xp[4];
  const __hip_bfloat16* wp[4];
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    const int r = c * 32 + wave * 8 + lr;
    const int xr = row0 + min(r, rows - 1);
    xp[c] = (const __hip_bfloat16*)p.x +
            (size_t)(p.rows != nullptr ? p.rows[xr] : xr) * p.k;
    wp[c] = (const __hip_bfloat16*)p.w +
            ((size_t)expert * p.n + min(n0 + r, p.n - 1)) * p.k;
  }
  auto issue = [&](int kt, int buf) {
    // columns past the end repeat the last ones; compute() masks them
    const int col = min(kt * BK + piece * 8, p.k - 8);
    __hip_bfloat16* to = lds + buf * STAGE + wave * 8 * BK;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      load_lds16(xp[c] + col, to + c * 32 * BK);
      load_lds16(wp[c] + col, to + BM * BK + c * 32 * BK);
    }
  };
  const int wm = (wave >> 1) * 64, wn = (wave & 1) * 64;
  f32x4 acc[4][4];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) acc[i][j] = {0.f, 0.f, 0.f, 0.f};
  auto compute = [&](int buf, int k_left) {
    const __hip_bfloat16* xs = lds + buf * STAGE;
    const __hip_bfloat16* ws = xs + BM * BK;
    const mf_bf8 z = {};
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      const int at = ((h * 4 + gs) ^ (gl & 7)) * 8;
      const bool on = h * 32 + gs * 8 < k_left;
      mf_bf8 a[4], b[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        a[i] = frag8(ws + (wn + i * 16 + gl) * BK + at);
        b[i] = frag8(xs + (wm + i * 16 + gl) * BK + at);
      }
      if (k_left < BK) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          a[i] = on ? a[i] : z;
          b[i] = on ? b[i] : z;
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          acc[i][j] = mfma_bf16_k32(a[i], b[j], acc[i][j]);
    }
  };
  const int nk = (p.k + BK - 1) / BK;
  issue(0, 0);
  for (int kt = 0; kt < nk; ++kt) {
    // this step's pieces have landed, and the other buffer is read
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (kt + 1 < nk) issue(kt + 1, (kt + 1) & 1);
    compute(kt & 1, p.k - kt * BK);
  }
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int r = wm + j * 16 + gl;
    if (r >= rows) continue;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int n = n0 + wn + i * 16 + gs * 4;
      if (n < p.n) put4(p, row0 + r, n, acc[i][j]);
    }
  }
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
    static bool once = false;
    if (!once) {
      (void)hipFuncSetAttribute((const void*)moe_tiled_kernel,
                                hipFuncAttributeMaxDynamicSharedMemorySize,
                                2 * STAGE * 2);
      once = true;
    }
    const int nb = (p->n + BN - 1) / BN;
    moe_tiled_kernel<<<8 * ((p->max_tiles * nb + 7) / 8), GT, 2 * STAGE * 2,
                       s>>>(*p);
  }
}
