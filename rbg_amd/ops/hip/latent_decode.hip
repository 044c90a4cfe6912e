// Decode attention over paged latents (gfx950, bf16): absorbed queries, one
// token per sequence, the latent as key and value at once, window-limited.  A key
// may be longer than its value (a rotated part behind the latent).
//
// A workgroup takes one sequence, 16 heads and one split of the visible keys,
// 64 keys a step (4 chunks of 16: a chunk is part of one page, so contiguous):
//   stage    wave w brings chunk w: global -> registers, a step ahead -> LDS
//   S^T = C Q^T    wave w scores its chunk: A = latent rows, B = the heads'
//            queries in registers; a head is a lane column
//   softmax  running max shared through LDS; the weights go to LDS as two bf16
//            (hi + lo), so that they keep 16 bits
//   O^T += C^T P^T wave w owns a quarter of the rank for all 64 keys: A = the
//            same LDS rows read transposed, B = the weights
// The accumulators are split over the waves, so nothing is merged at the end
// but the sum of the weights.  Splits of the keys meet in latent_combine.  The
// second tile of 16 heads finds the latents in L2.
#include "mfma_util.h"
#include "latent_args.h"

namespace {

constexpr int NW = 4;

// RK: value columns, DK: key columns
template <int RK, int DK>
__global__ __launch_bounds__(NW * 64, 2) void latent_decode_kernel(
    const LatentDecodeArgs p) {
  constexpr int PITCH = DK + 16;              // 8 banks per row
  // 16-byte loads per chunk: whole value rows, then what the keys have more
  constexpr int LPV = 16 * RK / 8 / 64, LPC = 16 * DK / 8 / 64;
  constexpr int VL = RK / 8, XL = DK > RK ? (DK - RK) / 8 : 1;
  constexpr int DT = RK / 16 / NW;            // 16-column tiles per wave
  static_assert(DT >= 1 && LPC >= 1, "rank tile too small");
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __hip_bfloat16* cs = (__hip_bfloat16*)smem; // [64][PITCH]
  // weights by chunk, lane group and head: 4 keys each
  mf_bf4* ph = (mf_bf4*)(cs + 64 * PITCH);    // [4][4][16]
  mf_bf4* pl = ph + 256;
  float* mx_s = (float*)(pl + 256);           // [NW][16]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int split = blockIdx.x, seq = blockIdx.y, h0 = blockIdx.z * 16;
  const int pos = p.ctx[seq] - 1;
  const int lo = p.window > 0 ? max(0, pos - p.window + 1) : 0;
  const int c_lo = lo >> 4, c_n = (pos >> 4) - c_lo + 1;
  // this split's chunks, whole steps of NW
  const int steps = (c_n + NW - 1) / NW;
  const int per = (steps + p.splits - 1) / p.splits * NW;
  const int c_beg = c_lo + split * per;
  const int c_end = min(c_beg + per, c_lo + c_n);
  const int* table = p.tables + (size_t)seq * p.max_pages;
  const __hip_bfloat16* cache = (const __hip_bfloat16*)p.cache;
  const int cpp = p.page_size >> 4;           // chunks per page
  const bool full = p.d == DK;

  const int head = min(h0 + gl, p.heads - 1);
  const __hip_bfloat16* q = (const __hip_bfloat16*)p.q +
                            (size_t)seq * p.q_row + (size_t)head * p.q_head;
  mf_bf8 qf[DK / 32];
#pragma unroll
  for (int s = 0; s < DK / 32; ++s) {
    const int d = s * 32 + gs * 8;
    mf_bf8 z = {};
    qf[s] = d < p.d ? frag8(q + d) : z;
  }

  float m = MASKED, l = 0.f;
  if (p.sink != nullptr && split == 0) {      // counts once
    m = p.sink[head] * LOG2E;
    l = wave == 0 && gs == 0 ? 1.f : 0.f;
  }
  f32x4 acc[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d) acc[d] = {0.f, 0.f, 0.f, 0.f};
  const float sl2 = p.scale * LOG2E;

  u32x4 reg[LPC];
  const u32x4 zero4 = {0, 0, 0, 0};
  // load i of a chunk brings key k(i), columns d(i) ..; both are one lane's
  // constant plus one of i, so that addresses are too
  const int vk = lane / VL, vd = lane % VL * 8;
  const int xk = lane / XL, xd = RK + lane % XL * 8;
  auto key_of = [&](int i) {
    return i < LPV ? vk + i * (64 / VL)
                   : xk + (i - LPV) * (64 / XL);
  };
  auto dim_of = [&](int i) { return i < LPV ? vd : xd; };
  // a chunk past the end re-reads the last one, as zeros
  auto fetch = [&](const int c) {
    const int cc = min(c, c_end - 1);
    const __hip_bfloat16* src =
        cache + ((size_t)table[cc / cpp] * p.page_size + (cc % cpp) * 16) * p.d;
#pragma unroll
    for (int i = 0; i < LPC; ++i)
      reg[i] = full || dim_of(i) < p.d
          ? *reinterpret_cast<const u32x4*>(src + key_of(i) * p.d + dim_of(i))
          : zero4;
  };

  if (c_beg < c_end) fetch(c_beg + wave);
  for (int c0 = c_beg; c0 < c_end; c0 += NW) {
    const int c = c0 + wave;
    __hip_bfloat16* mine = cs + wave * 16 * PITCH;
    // rows outside the window are stored as zeros: their weight is zero, but
    // a row nobody has written yet may hold anything
    const int c_hi = min(pos, c_end * 16 - 1);
#pragma unroll
    for (int i = 0; i < LPC; ++i) {
      const int j = c * 16 + key_of(i);
      *reinterpret_cast<u32x4*>(&mine[key_of(i) * PITCH + dim_of(i)]) =
          j >= lo && j <= c_hi ? reg[i] : zero4;
    }
    if (c0 + NW < c_end) fetch(c + NW);
    f32x4 s = {0.f, 0.f, 0.f, 0.f}, s2 = s;
#pragma unroll
    for (int st = 0; st < DK / 32; st += 2) {
      s = mfma_bf16_k32(frag8(&mine[gl * PITCH + st * 32 + gs * 8]), qf[st],
                        s);
      s2 = mfma_bf16_k32(frag8(&mine[gl * PITCH + st * 32 + 32 + gs * 8]),
                         qf[st + 1], s2);
    }
    s += s2;
    float x[4], mx = MASKED;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int j = c * 16 + gs * 4 + r;
      x[r] = j >= lo && j <= c_hi ? s[r] * sl2 : MASKED;
      mx = fmaxf(mx, x[r]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    if (gs == 0) mx_s[wave * 16 + gl] = mx;
    __syncthreads();
    float mn = m;
#pragma unroll
    for (int w = 0; w < NW; ++w) mn = fmaxf(mn, mx_s[w * 16 + gl]);
    const float corr = exp2_fast(m - mn);
    m = mn;
    float sum = 0.f;
    mf_bf4 hi, lw;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float e = x[r] > MASKED ? exp2_fast(x[r] - mn) : 0.f;
      sum += e;
      __bf16 a, b;
      split_bf16(e, a, b);
      hi[r] = a;
      lw[r] = b;
    }
    ph[(wave * 4 + gs) * 16 + gl] = hi;
    pl[(wave * 4 + gs) * 16 + gl] = lw;
    l = l * corr + sum;                       // this wave's keys
#pragma unroll
    for (int d = 0; d < DT; ++d) acc[d] *= corr;
    __syncthreads();
#pragma unroll
    for (int st = 0; st < 2; ++st) {
      const mf_bf4 h0v = ph[(st * 8 + gs) * 16 + gl];
      const mf_bf4 h1v = ph[(st * 8 + 4 + gs) * 16 + gl];
      const mf_bf4 l0v = pl[(st * 8 + gs) * 16 + gl];
      const mf_bf4 l1v = pl[(st * 8 + 4 + gs) * 16 + gl];
      const mf_bf8 hv = {h0v[0], h0v[1], h0v[2], h0v[3],
                         h1v[0], h1v[1], h1v[2], h1v[3]};
      const mf_bf8 lv = {l0v[0], l0v[1], l0v[2], l0v[3],
                         l1v[0], l1v[1], l1v[2], l1v[3]};
#pragma unroll
      for (int d = 0; d < DT; ++d) {
        const __hip_bfloat16* b = &cs[(st * 32 + gs * 4 + (gl >> 2)) * PITCH +
                                      (wave * DT + d) * 16 + (gl & 3) * 4];
        const mf_bf4 v0 = tr_read4(b), v1 = tr_read4(b + 16 * PITCH);
        const mf_bf8 vf = {v0[0], v0[1], v0[2], v0[3],
                           v1[0], v1[1], v1[2], v1[3]};
        acc[d] = mfma_bf16_k32(vf, hv, acc[d]);
        acc[d] = mfma_bf16_k32(vf, lv, acc[d]);
      }
    }
    __syncthreads();                          // LDS is free again
  }

  // sum of the weights over lane groups and waves
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (gs == 0) mx_s[wave * 16 + gl] = l;
  __syncthreads();
  float L = 0.f;
#pragma unroll
  for (int w = 0; w < NW; ++w) L += mx_s[w * 16 + gl];
  if (h0 + gl >= p.heads) return;
  const size_t row = (size_t)seq * p.heads + h0 + gl;
  if (p.splits > 1) {
    const size_t part = (size_t)split * p.seqs * p.heads + row;
    if (wave == 0 && gs == 0) {
      p.part_ml[part * 2] = m;
      p.part_ml[part * 2 + 1] = L;
    }
#pragma unroll
    for (int d = 0; d < DT; ++d) {
      const int c = (wave * DT + d) * 16 + gs * 4;
      if (c < p.rank)
        *reinterpret_cast<f32x4*>(&p.part_o[part * p.rank + c]) = acc[d];
    }
  } else {
    const float inv = 1.f / L;
#pragma unroll
    for (int d = 0; d < DT; ++d) {
      const int c = (wave * DT + d) * 16 + gs * 4;
      if (c >= p.rank) continue;
      union { uint2 u; __hip_bfloat16 e[4]; } o;
#pragma unroll
      for (int r = 0; r < 4; ++r) o.e[r] = f2bf(acc[d][r] * inv);
      *reinterpret_cast<uint2*>(
          &((__hip_bfloat16*)p.out)[row * p.rank + c]) = o.u;
    }
  }
}

// one workgroup per (sequence, head): sum of the splits' partials
__global__ __launch_bounds__(128) void latent_combine_kernel(
    const LatentDecodeArgs p) {
  __shared__ float f[64];                     // splits <= 64
  const size_t row = blockIdx.x;              // seq * heads + head
  const size_t rows = (size_t)p.seqs * p.heads;
  const int tid = threadIdx.x;
  if (tid < 64) {
    const bool on = tid < p.splits;
    const float m = on ? p.part_ml[(tid * rows + row) * 2] : MASKED;
    const float l = on ? p.part_ml[(tid * rows + row) * 2 + 1] : 0.f;
    const float M = wave_max(m);
    const float w = on ? exp2_fast(m - M) : 0.f;
    f[tid] = w / wave_sum(l * w);
  }
  __syncthreads();
  for (int d = tid * 4; d < p.rank; d += 512) {
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (int s = 0; s < p.splits; ++s)
      o += *reinterpret_cast<const f32x4*>(
               &p.part_o[(s * rows + row) * p.rank + d]) * f[s];
    union { uint2 u; __hip_bfloat16 e[4]; } ov;
#pragma unroll
    for (int r = 0; r < 4; ++r) ov.e[r] = f2bf(o[r]);
    *reinterpret_cast<uint2*>(&((__hip_bfloat16*)p.out)[row * p.rank + d]) =
        ov.u;
  }
}

template <int RK, int DK>
void latent_decode_go(const LatentDecodeArgs& p, hipStream_t s) {
  const size_t lds = (size_t)64 * (DK + 16) * 2 + 2 * 256 * 8 + NW * 16 * 4;
  static bool once = false;
  if (!once) {
    (void)hipFuncSetAttribute((const void*)latent_decode_kernel<RK, DK>,
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              (int)lds);
    once = true;
  }
  const dim3 grid(p.splits, p.seqs, (p.heads + 15) / 16);
  latent_decode_kernel<RK, DK><<<grid, NW * 64, lds, s>>>(p);
}

template <int RK>
void latent_decode_t(const LatentDecodeArgs& p, hipStream_t s) {
  if (p.d <= RK) latent_decode_go<RK, RK>(p, s);
  else if (p.d <= RK + 64) latent_decode_go<RK, RK + 64>(p, s);
  else latent_decode_go<RK, RK + 128>(p, s);
}

int value_columns(int rank) {
  return rank <= 64 ? 64 : rank <= 128 ? 128 : rank <= 256 ? 256 : 512;
}

}  // namespace

extern "C" {

// whether there is a form for these sizes
int latent_decode_fits(int d, int rank) {
  return rank <= 512 && d >= rank && d <= value_columns(rank) + 128;
}

void launch_latent_decode(const LatentDecodeArgs* p, hipStream_t s) {
  switch (value_columns(p->rank)) {
    case 64: latent_decode_t<64>(*p, s); break;
    case 128: latent_decode_t<128>(*p, s); break;
    case 256: latent_decode_t<256>(*p, s); break;
    default: latent_decode_t<512>(*p, s); break;
  }
  if (p->splits > 1)
    latent_combine_kernel<<<p->seqs * p->heads, 128, 0, s>>>(*p);
}

}  // extern "C"
