// Per-head linear maps of a decode batch: every head multiplies its own weight
// [n, k] (the absorbed key and value expansions of latent attention), with an
// optional sigmoid output gate, straight into a column slice.
//
// Decode-shaped: few rows, so the time is the weights' stream.  bf16: a wave
// owns 16 output columns of a head for 16 * MT rows; weight rows are MFMA A
// fragments loaded from global memory (16 bytes per lane, each byte used by
// exactly one wave), the rows are B fragments from L2.  The result's lanes are
// rows and its registers four neighbouring columns.  f32 (and sizes that are
// not multiples of 8): one thread per output.
#include "mfma_util.h"
#include "latent_args.h"
#include "vec_io.h"

namespace {

template <int MT>
__global__ __launch_bounds__(256) void head_linear_kernel(
    const HeadLinearArgs p) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int head = blockIdx.y;
  const int n0 = (blockIdx.x * 4 + wave) * 16;
  const int s0 = blockIdx.z * 16 * MT;
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
#pragma unroll 4
  for (int k0 = 0; k0 < p.k; k0 += 32) {
    const int k = k0 + gs * 8;
    // unconditional clamped loads: a guard would serialise them
    const int kc = min(k, p.k - 8);
    mf_bf8 wf = frag8(w + kc);
    const mf_bf8 z = {};
    wf = k < p.k ? wf : z;
#pragma unroll
    for (int t = 0; t < MT; ++t) {
      const mf_bf8 xf = frag8(x[t] + kc);
      acc[t] = mfma_bf16_k32(wf, xf, acc[t]);
    }
  }
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    const int s = s0 + t * 16 + gl;
    if (s >= p.rows) continue;
    if (p.pack) {                       // four columns as one 8-byte access
      const int n = n0 + gs * 4;
      if (n >= p.n) continue;
      const size_t col = (size_t)head * p.n + n;
      union { uint2 u; __hip_bfloat16 e[4]; } ov, gv;
      if (p.gate != nullptr)
        gv.u = *reinterpret_cast<const uint2*>(
            (const __hip_bfloat16*)p.gate + (size_t)s * p.g_row + col);
#pragma unroll
      for (int r = 0; r < 4; ++r)
        ov.e[r] = f2bf(p.gate != nullptr
                           ? acc[t][r] * sigmoid_f(bf2f(gv.e[r]))
                           : acc[t][r]);
      *reinterpret_cast<uint2*>((__hip_bfloat16*)p.out + (size_t)s * p.o_row +
                                col) = ov.u;
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
      ((__hip_bfloat16*)p.out)[(size_t)s * p.o_row + (size_t)head * p.n + n] =
          f2bf(o);
    }
  }
}

template <typename T>
__global__ __launch_bounds__(256) void head_linear_rows_kernel(
    const HeadLinearArgs p, const long total) {
  const long i = blockIdx.x * 256L + threadIdx.x;
  if (i >= total) return;
  const int n = (int)(i % p.n), head = (int)(i / p.n % p.heads);
  const long s = i / ((long)p.n * p.heads);
  const T* w = (const T*)p.w + ((size_t)head * p.n + n) * p.k;
  const T* x = (const T*)p.x + s * p.x_row + head * p.x_head;
  float o = 0.f;
  for (int k = 0; k < p.k; ++k) o += to_f(x[k]) * to_f(w[k]);
  const long col = (long)head * p.n + n;
  if (p.gate != nullptr)
    o *= sigmoid_f(to_f(((const T*)p.gate)[s * p.g_row + col]));
  ((T*)p.out)[s * p.o_row + col] = from_f<T>(o);
}

}  // namespace

extern "C" void launch_head_linear(const HeadLinearArgs* p, int f32, int vec,
                                   hipStream_t s) {
  const long total = (long)p->rows * p->heads * p->n;
  if (f32) {
    head_linear_rows_kernel<float>
        <<<(int)((total + 255) / 256), 256, 0, s>>>(*p, total);
  } else if (!vec) {
    head_linear_rows_kernel<__hip_bfloat16>
        <<<(int)((total + 255) / 256), 256, 0, s>>>(*p, total);
  } else {
    const int nb = (p->n + 63) / 64;
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
