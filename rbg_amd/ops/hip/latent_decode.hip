// Decode attention over paged latents (gfx950, bf16): absorbed queries, one
// token per sequence, the latent as key and value at once, window-limited.
//
// A workgroup takes one sequence, 16 heads and one split of the visible keys;
// its 4 waves walk 16-key chunks (a part of one page: contiguous memory)
// independently of each other:
//   global -> registers, two chunks ahead -> wave-private LDS
//   S^T = C Q^T    A = latent rows, B = the 16 heads' queries in registers
//   softmax        a head is a lane column; max and sum take two shuffles
//   O^T += C^T P^T B = the weights' registers, split in two bf16 so that they
//                  keep 16 bits; A = the same LDS rows read transposed
// No barrier inside the loop.  The waves' (m, l, O) merge through LDS, the
// splits' in latent_combine.  Latents are read once per 16 heads, which the
// second head tile finds in L2.
#include "mfma_util.h"
#include "mix_args.h"

namespace {

constexpr int NW = 4;

template <int RK>
__global__ __launch_bounds__(NW * 64, 1) void latent_decode_kernel(
    const LatentDecodeArgs p) {
  constexpr int PITCH = RK + 16;              // 8 banks per row
  constexpr int LPC = 16 * RK / 8 / 64;       // 16-byte loads per chunk
  constexpr int DT = RK / 16;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  __hip_bfloat16* cs = (__hip_bfloat16*)smem +
                       (threadIdx.x >> 6) * 16 * PITCH;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int split = blockIdx.x, seq = blockIdx.y, h0 = blockIdx.z * 16;
  const int pos = p.ctx[seq] - 1;
  const int lo = p.window > 0 ? max(0, pos - p.window + 1) : 0;
  const int c_lo = lo >> 4, c_n = (pos >> 4) - c_lo + 1;
  // this split's chunks; the waves take every NW-th
  const int per = (c_n + p.splits - 1) / p.splits;
  const int c_beg = c_lo + split * per;
  const int c_end = min(c_beg + per, c_lo + c_n);
  const int* table = p.tables + (size_t)seq * p.max_pages;
  const __hip_bfloat16* cache = (const __hip_bfloat16*)p.cache;
  const int cpp = p.page_size >> 4;           // chunks per page
  const bool full = p.rank == RK;

  const int head = min(h0 + gl, p.heads - 1);
  const __hip_bfloat16* q = (const __hip_bfloat16*)p.q +
                            (size_t)seq * p.q_row + (size_t)head * p.q_head;
  mf_bf8 qf[RK / 32];
#pragma unroll
  for (int s = 0; s < RK / 32; ++s) {
    const int d = s * 32 + gs * 8;
    mf_bf8 z = {};
    qf[s] = d < p.rank ? frag8(q + d) : z;
  }

  float m = MASKED, l = 0.f;
  f32x4 acc[DT];
#pragma unroll
  for (int d = 0; d < DT; ++d) acc[d] = {0.f, 0.f, 0.f, 0.f};
  const float sl2 = p.scale * LOG2E;

  u32x4 ra[LPC], rb[LPC];
  const u32x4 zero4 = {0, 0, 0, 0};
  // a chunk past the end re-reads the last one; it is never used
#define LD_FETCH(reg, c)                                                      \
  do {                                                                        \
    const int cc = min((c), c_end - 1);                                       \
    const __hip_bfloat16* src =                                               \
        cache + ((size_t)table[cc / cpp] * p.page_size + (cc % cpp) * 16) *   \
                    p.rank;                                                   \
    _Pragma("unroll") for (int i = 0; i < LPC; ++i) {                         \
      const int e = i * 64 + lane, key = e / (RK / 8), d = (e % (RK / 8)) * 8;\
      reg[i] = full || d < p.rank                                             \
          ? *reinterpret_cast<const u32x4*>(src + key * p.rank + d) : zero4;  \
    }                                                                         \
  } while (0)
  // rows outside the window are stored as zeros: their weight is zero, but a
  // row nobody has written yet may hold anything
#define LD_LAND(reg, c)                                                       \
  do {                                                                        \
    _Pragma("unroll") for (int i = 0; i < LPC; ++i) {                         \
      const int e = i * 64 + lane, key = e / (RK / 8), d = (e % (RK / 8)) * 8;\
      const int j = (c) * 16 + key;                                           \
      *reinterpret_cast<u32x4*>(&cs[key * PITCH + d]) =                       \
          j >= lo && j <= pos ? reg[i] : zero4;                               \
    }                                                                         \
  } while (0)

  auto chunk = [&](int c) {
    f32x4 s = {0.f, 0.f, 0.f, 0.f}, s2 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int st = 0; st < RK / 32; st += 2) {
      s = mfma_bf16_k32(frag8(&cs[gl * PITCH + st * 32 + gs * 8]), qf[st], s);
      if (st + 1 < RK / 32)
        s2 = mfma_bf16_k32(frag8(&cs[gl * PITCH + st * 32 + 32 + gs * 8]),
                           qf[st + 1], s2);
    }
    s += s2;
    float x[4], mx = MASKED;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int j = c * 16 + gs * 4 + r;
      x[r] = j >= lo && j <= pos ? s[r] * sl2 : MASKED;
      mx = fmaxf(mx, x[r]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m, mx), corr = exp2_fast(m - mn);
    m = mn;
    mf_bf4 ph, pl;
    float sum = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float e = x[r] > MASKED ? exp2_fast(x[r] - mn) : 0.f;
      sum += e;
      __bf16 h, w;
      split_bf16(e, h, w);
      ph[r] = h;
      pl[r] = w;
    }
    l = l * corr + sum;
    const bool rescale = __any(corr != 1.f);
#pragma unroll
    for (int d = 0; d < DT; ++d) {
      const mf_bf4 vf =
          tr_read4(&cs[(gs * 4 + (gl >> 2)) * PITCH + d * 16 + (gl & 3) * 4]);
      if (rescale) acc[d] *= corr;
      acc[d] = mfma_bf16_k16(vf, ph, acc[d]);
      acc[d] = mfma_bf16_k16(vf, pl, acc[d]);
    }
  };

  int c = c_beg + wave;
  if (c < c_end) {
    LD_FETCH(ra, c);
    LD_FETCH(rb, c + NW);
    for (; c < c_end; c += 2 * NW) {
      LD_LAND(ra, c);
      LD_FETCH(ra, c + 2 * NW);
      __builtin_amdgcn_wave_barrier();
      chunk(c);
      __builtin_amdgcn_wave_barrier();
      if (c + NW >= c_end) break;
      LD_LAND(rb, c + NW);
      LD_FETCH(rb, c + 3 * NW);
      __builtin_amdgcn_wave_barrier();
      chunk(c + NW);
      __builtin_amdgcn_wave_barrier();
    }
  }
#undef LD_FETCH
#undef LD_LAND

  // merge the waves: [RK][17] sums and [NW][16] (m, l) in LDS
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  __syncthreads();                            // staging is free now
  float* osum = (float*)smem;
  float* ml = osum + RK * 17;
  if (gs == 0) {
    ml[(wave * 16 + gl) * 2] = m;
    ml[(wave * 16 + gl) * 2 + 1] = l;
  }
  __syncthreads();
  float M = MASKED, L = 0.f;
#pragma unroll
  for (int w = 0; w < NW; ++w) M = fmaxf(M, ml[(w * 16 + gl) * 2]);
#pragma unroll
  for (int w = 0; w < NW; ++w)
    L += ml[(w * 16 + gl) * 2 + 1] * exp2_fast(ml[(w * 16 + gl) * 2] - M);
  const float f = exp2_fast(m - M);
  for (int w = 0; w < NW; ++w) {
    if (wave == w) {
#pragma unroll
      for (int d = 0; d < DT; ++d)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float* o = &osum[(d * 16 + gs * 4 + r) * 17 + gl];
          *o = (w == 0 ? 0.f : *o) + acc[d][r] * f;
        }
    }
    __syncthreads();
  }
  float* lm = ml + NW * 32;                   // [16] L for the writers below
  if (tid < 16) {
    lm[tid] = L;
    if (p.splits > 1 && h0 + tid < p.heads) {
      float* o = p.part_ml +
                 (((size_t)split * p.seqs + seq) * p.heads + h0 + tid) * 2;
      o[0] = M;
      o[1] = L;
    }
  }
  __syncthreads();
  for (int i = tid; i < 16 * p.rank; i += NW * 64) {
    const int h = i / p.rank, d = i % p.rank;
    if (h0 + h >= p.heads) break;
    const float o = osum[d * 17 + h];
    if (p.splits > 1)
      p.part_o[(((size_t)split * p.seqs + seq) * p.heads + h0 + h) * p.rank +
               d] = o;
    else
      ((__hip_bfloat16*)p.out)[((size_t)seq * p.heads + h0 + h) * p.rank + d] =
          f2bf(o / lm[h]);
  }
}

// one workgroup per (sequence, head): sum of the splits' partials
__global__ __launch_bounds__(256) void latent_combine_kernel(
    const LatentDecodeArgs p) {
  const size_t row = blockIdx.x;              // seq * heads + head
  const size_t rows = (size_t)p.seqs * p.heads;
  float M = MASKED, L = 0.f;
  for (int s = 0; s < p.splits; ++s)
    M = fmaxf(M, p.part_ml[(s * rows + row) * 2]);
  for (int s = 0; s < p.splits; ++s)
    L += p.part_ml[(s * rows + row) * 2 + 1] *
         exp2_fast(p.part_ml[(s * rows + row) * 2] - M);
  const float inv = 1.f / L;
  for (int d = threadIdx.x; d < p.rank; d += 256) {
    float o = 0.f;
    for (int s = 0; s < p.splits; ++s)
      o += p.part_o[(s * rows + row) * p.rank + d] *
           exp2_fast(p.part_ml[(s * rows + row) * 2] - M);
    ((__hip_bfloat16*)p.out)[row * p.rank + d] = f2bf(o * inv);
  }
}

template <int RK>
void latent_decode_t(const LatentDecodeArgs& p, hipStream_t s) {
  const size_t stage = (size_t)NW * 16 * (RK + 16) * 2;
  const size_t merge = (size_t)(RK * 17 + NW * 32 + 16) * 4;
  const size_t lds = stage > merge ? stage : merge;
  static bool once = false;
  if (!once) {
    (void)hipFuncSetAttribute((const void*)latent_decode_kernel<RK>,
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              (int)lds);
    once = true;
  }
  const dim3 grid(p.splits, p.seqs, (p.heads + 15) / 16);
  latent_decode_kernel<RK><<<grid, NW * 64, lds, s>>>(p);
}

}  // namespace

extern "C" void launch_latent_decode(const LatentDecodeArgs* p,
                                     hipStream_t s) {
  if (p->rank <= 64) {
    latent_decode_t<64>(*p, s);
  } else if (p->rank <= 128) {
    latent_decode_t<128>(*p, s);
  } else if (p->rank <= 256) {
    latent_decode_t<256>(*p, s);
  } else {
    latent_decode_t<512>(*p, s);
  }
  if (p->splits > 1)
    latent_combine_kernel<<<p->seqs * p->heads, 256, 0, s>>>(*p);
}
