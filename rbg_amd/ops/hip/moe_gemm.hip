// Grouped products of a step's (token, choice) rows with their experts' weights
// (gfx950): out[row, n] = sum_k x[row, k] w[expert, n, k], rows in expert order,
// a tile of rows per expert (moe_route.hip).  The number of tiles is on the
// device; launches cover the most there can be and the rest leaves at once.
//
//   tiled   128 rows x 128 or 192 columns, 64 k a step, both operands straight
//           from global memory into LDS (rows may be gathered: every lane brings
//           its own address).  One buffer: the other workgroups of the CU, three
//           or four of them, compute while one waits, which measured better than
//           two buffers with half the workgroups.
//   stream  32 or 64 rows x 64 columns, several stages of LDS deep: decode
//           batches, whose time is the weights' way from memory.
//   skinny  up to 16 rows x 16 columns, weight fragments from global memory into
//           the MFMAs, waves split K and meet in LDS: batches whose experts do
//           not fill the chip otherwise.
//   rows    any sizes, bf16 or f32: a thread per column, up to 16 rows at once.
// A squared relu, or a gated unit of interleaved rows, rides on the way out.
#include "lds_stream.h"
#include "expert_args.h"
#include "act.h"
#include "vec_io.h"

namespace {

DEV_INLINE float relu2_f(float x) {
  x = fmaxf(x, 0.f);
  return x * x;
}

DEV_INLINE bool gated(const MoeGemmArgs& p) { return p.act >= EXPERT_SILU_GLU; }

DEV_INLINE float glu_f(const MoeGemmArgs& p, float g, float u) {
  return p.act == EXPERT_CLAMPED_GLU ? clamped_glu_f(g, u, p.limit)
                                     : silu_glu_f(g, u);
}

// four neighbouring columns of one row
DEV_INLINE void put4(const MoeGemmArgs& p, const size_t row, const int n,
                     f32x4 v) {
  if (gated(p)) {                               // gate, gate, up, up
    union { uint32_t u; __hip_bfloat16 e[2]; } o;
    o.e[0] = f2bf(glu_f(p, v[0], v[2]));
    o.e[1] = f2bf(glu_f(p, v[1], v[3]));
    *reinterpret_cast<uint32_t*>((__hip_bfloat16*)p.out + row * (p.n / 2) +
                                 n / 2) = o.u;
    return;
  }
  union { uint2 u; __hip_bfloat16 e[4]; } o;
#pragma unroll
  for (int r = 0; r < 4; ++r) o.e[r] = f2bf(p.act == EXPERT_RELU2 ? relu2_f(v[r]) : v[r]);
  *reinterpret_cast<uint2*>((__hip_bfloat16*)p.out + row * p.n + n) = o.u;
}

constexpr int BM = 128, GT = 256;

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

  // wave instruction c brings rows c*32 + wave*8 .. +7
  const int lr = lane >> 3, piece = stage_piece();
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
      const int at = stage_at(h);
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
    landed_barrier<0>();
    compute(BK);
    landed_barrier<0>();                           // everyone has read
  }
  if (rest) {                                   // pieces past the end: the last
    const uint32_t back = tail_back(rest);
#pragma unroll
    for (int c = 0; c < XI; ++c) xo[c] -= back;
#pragma unroll
    for (int c = 0; c < WI; ++c) wo[c] -= back;
    issue(nk);
    landed_barrier<0>();
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

template <int SM, int NB>
__global__ __launch_bounds__(256) void moe_stream_kernel(const MoeGemmArgs p) {
  using Stream = LdsStream<SM, NB>;
  extern __shared__ __attribute__((aligned(16))) char stream_smem[];
  if ((int)blockIdx.y >= *p.count) return;
  const int* tile = p.tiles + (size_t)blockIdx.y * 3;
  const int expert = tile[0], row0 = tile[1], rows = tile[2];
  const int n0 = blockIdx.x * 64, piece = stage_piece();
  uint32_t xo[Stream::XI], wo[2];
#pragma unroll
  for (int c = 0; c < Stream::XI; ++c) {
    const int at = row0 + min(c * 32 + Stream::row(), rows - 1);
    xo[c] = ((uint32_t)(p.rows != nullptr ? p.rows[at] : at) * p.k +
             piece * 8) * 2;
  }
#pragma unroll
  for (int c = 0; c < 2; ++c)
    wo[c] = ((uint32_t)min(n0 + c * 32 + Stream::row(), p.n - 1) * p.k +
             piece * 8) * 2;
  f32x4 acc[Stream::TM];
  Stream::run(p.x, xo, (const char*)p.w + (size_t)expert * p.n * p.k * 2, wo,
              p.k, (blockIdx.x + 5 * blockIdx.y) % ((p.k + BK - 1) / BK),
              (rows + 15) / 16, stream_smem, acc);
  const int n = n0 + (threadIdx.x >> 6) * 16 + ((threadIdx.x & 63) >> 4) * 4;
#pragma unroll
  for (int j = 0; j < Stream::TM; ++j) {
    const int r = j * 16 + (threadIdx.x & 15);
    if (r < rows && n < p.n) put4(p, row0 + r, n, acc[j]);
  }
}

template <int SM, int NB>
void moe_stream(const MoeGemmArgs& p, hipStream_t s) {
  constexpr int lds = LdsStream<SM, NB>::BYTES;
  static bool once = false;
  if (!once) {
    (void)hipFuncSetAttribute((const void*)moe_stream_kernel<SM, NB>,
                              hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    once = true;
  }
  const dim3 grid((p.n + 63) / 64, p.max_tiles);
  moe_stream_kernel<SM, NB><<<grid, 256, lds, s>>>(p);
}

constexpr int SW = 4;                           // waves of a skinny workgroup
constexpr int UN = 4;                           // 32-k steps in flight

__global__ __launch_bounds__(SW * 64) void moe_skinny_kernel(
    const MoeGemmArgs p) {
  __shared__ f32x4 red[SW][64];
  if ((int)blockIdx.y >= *p.count) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int* tile = p.tiles + (size_t)blockIdx.y * 3;
  const int expert = tile[0], row0 = tile[1], rows = tile[2];
  const int n0 = blockIdx.x * 16, at = row0 + min(gl, rows - 1);
  const __hip_bfloat16* wr = (const __hip_bfloat16*)p.w +
      ((size_t)expert * p.n + min(n0 + gl, p.n - 1)) * p.k;
  const __hip_bfloat16* xr = (const __hip_bfloat16*)p.x +
      (size_t)(p.rows != nullptr ? p.rows[at] : at) * p.k;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  const int per = ((p.k + SW * 32 - 1) / (SW * 32)) * 32;
  const int kb = wave * per, ke = min(kb + per, p.k);
  for (int k0 = kb; k0 < ke; k0 += 32 * UN) {
    // unconditional clamped loads, all before the first product: a guard would
    // serialise them
    mf_bf8 wf[UN], xf[UN];
    const mf_bf8 z = {};
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const int kc = min(k0 + u * 32 + gs * 8, p.k - 8);
      wf[u] = frag8(wr + kc);
      xf[u] = frag8(xr + kc);
    }
#pragma unroll
    for (int u = 0; u < UN; ++u)
      acc = mfma_bf16_k32(k0 + u * 32 + gs * 8 < ke ? wf[u] : z, xf[u], acc);
  }
  red[wave][lane] = acc;
  __syncthreads();
  if (wave > 0) return;
#pragma unroll
  for (int wv = 1; wv < SW; ++wv) acc += red[wv][lane];
  const int n = n0 + gs * 4;
  if (gl < rows && n < p.n) put4(p, row0 + gl, n, acc);
}

// GLU: a thread per column of the result, from two rows of w
template <typename T, bool GLU>
__global__ __launch_bounds__(256) void moe_rows_kernel(const MoeGemmArgs p) {
  if ((int)blockIdx.y >= *p.count) return;
  const int* tile = p.tiles + (size_t)blockIdx.y * 3;
  const int expert = tile[0], row0 = tile[1], rows = tile[2];
  const int c = blockIdx.x * 256 + threadIdx.x, cols = GLU ? p.n / 2 : p.n;
  if (c >= cols) return;
  const int n = GLU ? c / 2 * 4 + c % 2 : c;
  const T* w = (const T*)p.w + ((size_t)expert * p.n + n) * p.k;
  const T* x[16];
  float acc[16], up[GLU ? 16 : 1];
#pragma unroll
  for (int r = 0; r < 16; ++r) {
    const int at = row0 + min(r, rows - 1);
    x[r] = (const T*)p.x + (size_t)(p.rows != nullptr ? p.rows[at] : at) * p.k;
    acc[r] = 0.f;
    if (GLU) up[r] = 0.f;
  }
  for (int k = 0; k < p.k; ++k) {
    const float wv = to_f(w[k]), wu = GLU ? to_f(w[2 * (size_t)p.k + k]) : 0.f;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      const float xv = to_f(x[r][k]);
      acc[r] += wv * xv;
      if (GLU) up[r] += wu * xv;
    }
  }
#pragma unroll
  for (int r = 0; r < 16; ++r)
    if (r < rows)
      ((T*)p.out)[(size_t)(row0 + r) * cols + c] = from_f<T>(
          GLU                       ? glu_f(p, acc[r], up[r])
          : p.act == EXPERT_RELU2 ? relu2_f(acc[r])
                                  : acc[r]);
}

template <typename T>
void moe_rows(const MoeGemmArgs& p, hipStream_t s) {
  const bool glu = p.act >= EXPERT_SILU_GLU;
  const dim3 grid(((glu ? p.n / 2 : p.n) + 255) / 256, p.max_tiles);
  if (glu) {
    moe_rows_kernel<T, true><<<grid, 256, 0, s>>>(p);
  } else {
    moe_rows_kernel<T, false><<<grid, 256, 0, s>>>(p);
  }
}

}  // namespace

extern "C" void launch_moe_gemm(const MoeGemmArgs* p, int f32, int vec,
                                hipStream_t s) {
  if (!vec) {                                   // tile <= 16
    if (f32) moe_rows<float>(*p, s);
    else moe_rows<__hip_bfloat16>(*p, s);
  } else if (p->tile <= 16) {
    moe_skinny_kernel<<<dim3((p->n + 15) / 16, p->max_tiles), SW * 64, 0,
                        s>>>(*p);
  } else if (p->tile <= 32) {
    moe_stream<32, 4>(*p, s);
  } else if (p->tile <= 64) {
    moe_stream<64, 4>(*p, s);
  } else {
    // the wide form is 1.08 times as fast per column
    const long wide = (p->n + 191) / 192 * 192L, slim = (p->n + 127) / 128 * 128L;
    if (wide * 100 <= slim * 108) moe_tiled<192, 3>(*p, s);
    else moe_tiled<128, 4>(*p, s);
  }
}
