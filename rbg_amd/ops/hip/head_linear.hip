// Per-head linear maps of a decode batch: every head multiplies its own weight
// [n, k] (the absorbed key and value expansions of latent attention), with an
// optional sigmoid output gate, straight into a column slice.  Behind a head's
// columns may follow the rotated dims of its query: the absorbed query of latent
// attention is then ready.
//
// Decode-shaped: few rows, so the time is the weights' stream.  bf16: a wave
// owns 16 output columns of a head for 16 * MT rows; weight rows are MFMA A
// fragments loaded from global memory (16 bytes per lane, each byte used by
// exactly one wave), the rows are B fragments from L2.  The result's lanes are
// rows and its registers four neighbouring columns.  f32 (and sizes that are
// not multiples of 8): one thread per output.
#include "latent_args.h"
#include "mfma_util.h"
#include "rotary.h"
#include "vec_io.h"

namespace {

// rows [s0, s1) of a head's tail, pieces (pairs) from `at` on in steps of `step`
__host__ DEV_INLINE int tail_pieces(const HeadLinearArgs& p) {
  return p.tail_vec ? rotary_vecs(p.rot) : p.rot.dims / 2;
}

DEV_INLINE void rotate_tail_vec(const HeadLinearArgs& p, const int head,
                                const int s0, const int s1, const int at,
                                const int step) {
  const int per = rotary_vecs(p.rot);
  for (int e = at; e < (s1 - s0) * per; e += step) {
    const int s = s0 + e / per;
    rotate_vec(p.rot, rotary_row(p.rot, s), e % per,
               (const __hip_bfloat16*)p.tail + (size_t)s * p.t_row +
                   head * p.t_head,
               (__hip_bfloat16*)p.out + (size_t)s * p.o_row +
                   head * p.o_head + p.n);
  }
}

template <typename T>
DEV_INLINE void rotate_tail(const HeadLinearArgs& p, const int head,
                            const int s0, const int s1, const int at,
                            const int step) {
  const int half = p.rot.dims / 2;
  for (int e = at; e < (s1 - s0) * half; e += step) {
    const int s = s0 + e / half;
    rotate_pair(p.rot, rotary_row(p.rot, s), e % half,
                (const T*)p.tail + (size_t)s * p.t_row + head * p.t_head,
                (T*)p.out + (size_t)s * p.o_row + head * p.o_head + p.n);
  }
}

template <int MT>
__global__ __launch_bounds__(256) void head_linear_kernel(
    const HeadLinearArgs p) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int head = blockIdx.y;
  const int n0 = (blockIdx.x * 4 + wave) * 16;
  const int s0 = blockIdx.z * 16 * MT;
  const int nb = (p.n + 63) / 64;
  if ((int)blockIdx.x >= nb) {                  // workgroups behind the last
    const int s1 = min(s0 + 16 * MT, p.rows);
    const int at = (blockIdx.x - nb) * 256 + threadIdx.x;
    const int step = (gridDim.x - nb) * 256;
    if (p.tail_vec) rotate_tail_vec(p, head, s0, s1, at, step);
    else rotate_tail<__hip_bfloat16>(p, head, s0, s1, at, step);
    return;
  }
  if (n0 >= p.n) return;
  const __hip_bfloat16* w = (const __hip_bfloat16*)p.w +
      ((size_t)head * p.n + min(n0 + gl, p.n - 1)) * p.k;
  const __hip_bfloat16* x[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t)
    x[t] = (const __hip_bfloat16*)p.x +
           (size_t)min(s0 + t * 16 + gl, p.rows - 1) * p.x_row +
           (size_t)head * p.x_head;
  f32x4 acc[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) acc[t] = {0.f, 0.f, 0.f, 0.f};
  constexpr int UN = 4;                         // 32-k steps in flight
  for (int k0 = 0; k0 < p.k; k0 += 32 * UN) {
    // unconditional clamped loads, all before the first product: a guard would
    // serialise them
    mf_bf8 wf[UN], xf[UN][MT];
    const mf_bf8 z = {};
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const int kc = min(k0 + u * 32 + gs * 8, p.k - 8);
      wf[u] = frag8(w + kc);
#pragma unroll
      for (int t = 0; t < MT; ++t) xf[u][t] = frag8(x[t] + kc);
    }
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const mf_bf8 wu = k0 + u * 32 + gs * 8 < p.k ? wf[u] : z;
#pragma unroll
      for (int t = 0; t < MT; ++t) acc[t] = mfma_bf16_k32(wu, xf[u][t], acc[t]);
    }
  }
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int s = s0 + t * 16 + gl;
    if (s >= p.rows) continue;
    if (p.pack) {                       // four columns as one 8-byte access
      const int n = n0 + gs * 4;
      if (n >= p.n) continue;
      union { uint2 u; __hip_bfloat16 e[4]; } ov, gv;
      if (p.gate != nullptr)
        gv.u = *reinterpret_cast<const uint2*>(
            (const __hip_bfloat16*)p.gate + (size_t)s * p.g_row +
            (size_t)head * p.n + n);
#pragma unroll
      for (int r = 0; r < 4; ++r)
        ov.e[r] = f2bf(p.gate != nullptr
                           ? acc[t][r] * sigmoid_f(bf2f(gv.e[r]))
                           : acc[t][r]);
      *reinterpret_cast<uint2*>((__hip_bfloat16*)p.out + (size_t)s * p.o_row +
                                head * p.o_head + n) = ov.u;
      continue;
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int n = n0 + gs * 4 + r;
      if (n >= p.n) continue;
      float o = acc[t][r];
      if (p.gate != nullptr)
        o *= sigmoid_f(bf2f(((const __hip_bfloat16*)p.gate)[
            (size_t)s * p.g_row + (size_t)head * p.n + n]));
      ((__hip_bfloat16*)p.out)[(size_t)s * p.o_row + head * p.o_head + n] =
          f2bf(o);
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void head_linear_rows_kernel(
    const HeadLinearArgs p, const long total) {
  const long i = blockIdx.x * 256L + threadIdx.x;
  const long main = (total + 255) / 256;
  if (blockIdx.x >= main) {                     // one (row, head) each
    const int at = (int)(blockIdx.x - main), s = at / p.heads;
    rotate_tail<T>(p, at % p.heads, s, s + 1, threadIdx.x, 256);
    return;
  }
  if (i >= total) return;
  const int n = (int)(i % p.n), head = (int)(i / p.n % p.heads);
  const long s = i / ((long)p.n * p.heads);
  const T* w = (const T*)p.w + ((size_t)head * p.n + n) * p.k;
  const T* x = (const T*)p.x + s * p.x_row + head * p.x_head;
  float o = 0.f;
  for (int k = 0; k < p.k; ++k) o += to_f(x[k]) * to_f(w[k]);
  if (p.gate != nullptr)
    o *= sigmoid_f(
        to_f(((const T*)p.gate)[s * p.g_row + (long)head * p.n + n]));
  ((T*)p.out)[s * p.o_row + head * p.o_head + n] = from_f<T>(o);
}

}  // namespace

extern "C" void launch_head_linear(const HeadLinearArgs* p, int f32, int vec,
                                   hipStream_t s) {
  const long total = (long)p->rows * p->heads * p->n;
  const bool tail = p->rot.dims > 0;
  const int grid = (int)((total + 255) / 256) +
                   (tail ? p->rows * p->heads : 0);
  if (f32) {
    head_linear_rows_kernel<float><<<grid, 256, 0, s>>>(*p, total);
  } else if (!vec) {
    head_linear_rows_kernel<__hip_bfloat16><<<grid, 256, 0, s>>>(*p, total);
  } else {
    // one piece of the tail a thread
    const int most = p->rows <= 16 ? 16 : p->rows <= 32 ? 32 : 64;
    const int nb = (p->n + 63) / 64 +
        (tail ? (min(p->rows, most) * tail_pieces(*p) + 255) / 256 : 0);
    if (p->rows <= 16) {
      head_linear_kernel<1><<<dim3(nb, p->heads, 1), 256, 0, s>>>(*p);
    } else if (p->rows <= 32) {
      head_linear_kernel<2><<<dim3(nb, p->heads, 1), 256, 0, s>>>(*p);
    } else {
      head_linear_kernel<4><<<dim3(nb, p->heads, (p->rows + 63) / 64), 256, 0,
                              s>>>(*p);
    }
  }
}
