// Causal window attention over contiguous keys and values (gfx950, bf16):
// varlen prefill of any head sizes up to 256, with an optional sigmoid output
// gate, an optional key part that all heads share, and an optional sink per head.  A query at position i sees keys j with 0 <= i - j < window.
//
// A workgroup takes 128 query rows of one head (NW waves x QT x 16) and walks the
// 64-key tiles between its first row's window edge and its last row.  Per tile
//   S^T = K Q^T      A = K rows from LDS, B = Q rows held in registers
//   softmax          a query is a lane column: row max and sum are in-lane
//                    plus two shuffles, and the rescale is one scalar
//   O^T += V^T P^T   B = the softmax registers themselves (see mfma_util.h),
//                    split in two bf16 so the weights keep 16 bits; A = V read
//                    from row-major LDS through the transposing read
// so the weights never touch LDS.  The next tile's global loads fly under the
// current tile's MFMAs.  Row pitch is dim + 16 elements: 8 banks per row, which
// keeps both read patterns conflict-free.
//
// Head sizes of whole 64s take a form whose tiles go straight from global memory
// to LDS: without staging registers two workgroups fit a CU at 192 key dims too.
// The tile of the next keys is brought while this one's softmax and second
// product run; V has two buffers, K is free by then.
#include "latent_args.h"
#include "lds_stream.h"
#include "mfma_util.h"
#include "vec_io.h"

namespace {

constexpr int KT = 64;

// query r of its sequence: sums over the lane groups, division, gate, store
template <int DV>
DEV_INLINE void finish_row(const WindowAttnArgs& p, const int head,
                           const int r, const int qrow0, const int qlen,
                           float sum, const f32x4 (&acc)[DV / 16]) {
  const int gs = (threadIdx.x & 63) >> 4;
  sum += __shfl_xor(sum, 16, 64);
  sum += __shfl_xor(sum, 32, 64);
  if (r >= qlen) return;
  const float inv = 1.f / sum;
  const size_t row = qrow0 + r;
  __hip_bfloat16* o = (__hip_bfloat16*)p.out + row * p.o_row +
                      (size_t)head * p.dv;
  const __hip_bfloat16* g =
      p.gate ? (const __hip_bfloat16*)p.gate + row * p.g_row +
                   (size_t)head * p.dv
             : nullptr;
#pragma unroll
  for (int d = 0; d < DV / 16; ++d) {
    const int c = d * 16 + gs * 4;
    if (c >= p.dv) continue;
    union { uint2 u; __hip_bfloat16 e[4]; } ov, gv;
    if (g) gv.u = *reinterpret_cast<const uint2*>(g + c);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float x = acc[d][e] * inv;
      if (g) x *= sigmoid_f(bf2f(gv.e[e]));
      ov.e[e] = f2bf(x);
    }
    *reinterpret_cast<uint2*>(o + c) = ov.u;
  }
}

template <int DK, int DV, int NW, int QT>
__global__ __launch_bounds__(NW * 64, (DK + DV) > 320 ? 1 : 2)
void window_attn_kernel(const WindowAttnArgs p) {
  constexpr int KP = DK + 16, VP = DV + 16;
  constexpr int ROWS = NW * QT * 16;          // 128
  constexpr int NT = NW * 64;
  constexpr int KPC = KT * DK / 8 / NT, VPC = KT * DV / 8 / NT;
  __shared__ __hip_bfloat16 ks[KT * KP];
  __shared__ __hip_bfloat16 vs[KT * VP];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int gl = lane & 15, gs = lane >> 4;

  // workgroups go round the 8 XCDs: give each XCD whole heads, so that the
  // query tiles of a head share its keys and values in one L2
  const int items = p.n_blocks * p.heads, per = (items + 7) / 8;
  const int work = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  if ((blockIdx.x >> 3) >= per || work >= items) return;
  const int head = work / p.n_blocks;
  const int* bi = p.blocks + (p.n_blocks - 1 - work % p.n_blocks) * 2;
  const int* si = p.seq_info + bi[0] * 4;
  const int qrow0 = si[0], qlen = si[1], krow0 = si[2], qoff = si[3];
  const int t0 = bi[1];                       // first query of the block
  const int klen = qoff + qlen;

  const __hip_bfloat16* q = (const __hip_bfloat16*)p.q + head * p.q_head;
  const __hip_bfloat16* k = (const __hip_bfloat16*)p.k + head * p.k_head;
  const __hip_bfloat16* k2 = (const __hip_bfloat16*)p.k2 - p.d1;
  const __hip_bfloat16* v = (const __hip_bfloat16*)p.v + head * p.v_head;

  // Q as B operand: column = query, 8 dims per lane
  mf_bf8 qf[QT][DK / 32];
  int qpos[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int r = t0 + (wave * QT + t) * 16 + gl;
    qpos[t] = qoff + r;                       // may lie past the end: unused
    const __hip_bfloat16* qr = q + (size_t)(qrow0 + min(r, qlen - 1)) * p.q_row;
#pragma unroll
    for (int s = 0; s < DK / 32; ++s) {
      const int d = s * 32 + gs * 8;
      mf_bf8 z = {};
      qf[t][s] = d < p.d ? frag8(qr + d) : z;
    }
  }

  const int last = min(qoff + t0 + ROWS - 1, klen - 1);
  const int first = p.window > 0 ? max(0, qoff + t0 - p.window + 1) : 0;
  const int wlo = p.window > 0
      ? max(0, qoff + t0 + wave * QT * 16 - p.window + 1) : 0;
  const int whi = min(qoff + t0 + (wave + 1) * QT * 16 - 1, klen - 1);

  u32x4 kr[KPC], vr[VPC];
  const u32x4 zero4 = {0, 0, 0, 0};
  auto fetch = [&](int kt) {
#pragma unroll
    for (int i = 0; i < KPC; ++i) {
      const int e = tid + i * NT, key = e / (DK / 8), c = (e % (DK / 8)) * 8;
      const size_t row = krow0 + min(kt * KT + key, klen - 1);
      const __hip_bfloat16* src =
          c < p.d1 ? k + row * p.k_row : k2 + row * p.k2_row;
      kr[i] = c < p.d ? *reinterpret_cast<const u32x4*>(src + c) : zero4;
    }
#pragma unroll
    for (int i = 0; i < VPC; ++i) {
      const int e = tid + i * NT, key = e / (DV / 8), c = (e % (DV / 8)) * 8;
      const size_t row = krow0 + min(kt * KT + key, klen - 1);
      vr[i] = c < p.dv ? *reinterpret_cast<const u32x4*>(v + row * p.v_row + c)
                       : zero4;
    }
  };
  auto land = [&]() {
#pragma unroll
    for (int i = 0; i < KPC; ++i) {
      const int e = tid + i * NT, key = e / (DK / 8), c = (e % (DK / 8)) * 8;
      *reinterpret_cast<u32x4*>(&ks[key * KP + c]) = kr[i];
    }
#pragma unroll
    for (int i = 0; i < VPC; ++i) {
      const int e = tid + i * NT, key = e / (DV / 8), c = (e % (DV / 8)) * 8;
      *reinterpret_cast<u32x4*>(&vs[key * VP + c]) = vr[i];
    }
  };

  float m[QT], l[QT];
  f32x4 acc[QT][DV / 16];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    // a sink is the first maximum and one more term of the sum
    m[t] = p.sink != nullptr ? p.sink[head] * LOG2E : MASKED;
    l[t] = p.sink != nullptr && gs == 0 ? 1.f : 0.f;
#pragma unroll
    for (int d = 0; d < DV / 16; ++d) acc[t][d] = {0.f, 0.f, 0.f, 0.f};
  }
  const float sl2 = p.scale * LOG2E;
  const int kt1 = last / KT;
  fetch(first / KT);
  for (int kt = first / KT; kt <= kt1; ++kt) {
    __syncthreads();                          // the tile before is read
    land();
    __syncthreads();
    if (kt < kt1) fetch(kt + 1);
    const int k0 = kt * KT;
    if (k0 > whi || k0 + KT <= wlo) continue;  // barriers stay uniform

    f32x4 s[QT][4];
#pragma unroll
    for (int t = 0; t < QT; ++t)
#pragma unroll
      for (int c = 0; c < 4; ++c) s[t][c] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < 4; ++c)
#pragma unroll
      for (int st = 0; st < DK / 32; ++st) {
        const mf_bf8 kf = frag8(&ks[(c * 16 + gl) * KP + st * 32 + gs * 8]);
#pragma unroll
        for (int t = 0; t < QT; ++t)
          s[t][c] = mfma_bf16_k32(kf, qf[t][st], s[t][c]);
      }
    mf_bf8 ph[QT][2], pl[QT][2];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      const int hi = qpos[t], lo = p.window > 0 ? hi - p.window + 1 : 0;
      float mx = MASKED;
#pragma unroll
      for (int c = 0; c < 4; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = k0 + c * 16 + gs * 4 + r;
          const float x = j <= hi && j >= lo ? s[t][c][r] * sl2 : MASKED;
          s[t][c][r] = x;
          mx = fmaxf(mx, x);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m[t], mx);
      const float corr = exp2_fast(m[t] - mn);
      m[t] = mn;
      float sum = 0.f;
#pragma unroll
      for (int c = 0; c < 4; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float x = s[t][c][r];
          const float e = x > MASKED ? exp2_fast(x - mn) : 0.f;
          sum += e;
          __bf16 h, lw;
          split_bf16(e, h, lw);
          ph[t][c >> 1][(c & 1) * 4 + r] = h;
          pl[t][c >> 1][(c & 1) * 4 + r] = lw;
        }
      l[t] = l[t] * corr + sum;               // per lane; summed at the end
#pragma unroll
      for (int d = 0; d < DV / 16; ++d) acc[t][d] *= corr;
    }
#pragma unroll
    for (int st = 0; st < 2; ++st)
#pragma unroll
      for (int d = 0; d < DV / 16; ++d) {
        const __hip_bfloat16* b =
            &vs[(st * 32 + gs * 4 + (gl >> 2)) * VP + d * 16 + (gl & 3) * 4];
        const mf_bf4 v0 = tr_read4(b), v1 = tr_read4(b + 16 * VP);
        const mf_bf8 vf = {v0[0], v0[1], v0[2], v0[3],
                           v1[0], v1[1], v1[2], v1[3]};
#pragma unroll
        for (int t = 0; t < QT; ++t) {
          acc[t][d] = mfma_bf16_k32(vf, ph[t][st], acc[t][d]);
          acc[t][d] = mfma_bf16_k32(vf, pl[t][st], acc[t][d]);
        }
      }
  }

#pragma unroll
  for (int t = 0; t < QT; ++t)
    finish_row<DV>(p, head, t0 + (wave * QT + t) * 16 + gl, qrow0, qlen, l[t],
                   acc[t]);
}

// One workgroup: 4 waves of 32 queries.  G, VG: key and value dims / 64, the tile
// in LDS as [G or VG][64 rows][8 pieces of 16 bytes].  Piece p of key row r lies
// at p ^ (r / 2 % 8), so that the 16 rows of a fragment spread over the banks; of
// value row r at p ^ (r / 2 % 4 * 2), which keeps pairs of pieces together for the
// transposing read.
template <int G, int VG>
__global__ __launch_bounds__(256, 2)
void window_direct_kernel(const WindowAttnArgs p) {
  constexpr int QT = 2, ROWS = 4 * QT * 16, PART = KT * 64;
  __shared__ __attribute__((aligned(16)))
  __hip_bfloat16 lds[(G + 2 * VG) * PART];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int gl = lane & 15, gs = lane >> 4;

  // whole heads to an XCD, as above
  const int items = p.n_blocks * p.heads, per = (items + 7) / 8;
  const int work = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  if ((blockIdx.x >> 3) >= per || work >= items) return;
  const int head = work / p.n_blocks;
  const int* bi = p.blocks + (p.n_blocks - 1 - work % p.n_blocks) * 2;
  const int* si = p.seq_info + bi[0] * 4;
  const int qrow0 = si[0], qlen = si[1], krow0 = si[2], qoff = si[3];
  const int t0 = bi[1], klen = qoff + qlen;

  const __hip_bfloat16* q = (const __hip_bfloat16*)p.q + head * p.q_head;
  mf_bf8 qf[QT][2 * G];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int r = t0 + (wave * QT + t) * 16 + gl;
    const __hip_bfloat16* qr = q + (size_t)(qrow0 + min(r, qlen - 1)) * p.q_row;
#pragma unroll
    for (int s = 0; s < 2 * G; ++s) qf[t][s] = frag8(qr + s * 32 + gs * 8);
  }
  const int q0 = qoff + t0 + wave * QT * 16;  // this wave's first position
  const int last = min(qoff + t0 + ROWS - 1, klen - 1);
  const int first = p.window > 0 ? max(0, qoff + t0 - p.window + 1) : 0;
  const int wlo = p.window > 0 ? max(0, q0 - p.window + 1) : 0;
  const int whi = min(q0 + QT * 16 - 1, klen - 1);

  // a wave brings rows wave * 16 .. + 15 of every part, 8 at a time
  const int row = wave * 16 + (lane >> 3), place = lane & 7;
  const uint32_t base = __builtin_amdgcn_readfirstlane(
      (uint32_t)(uintptr_t)lds + wave * 2048);
  const __hip_bfloat16* k = (const __hip_bfloat16*)p.k + head * p.k_head +
                            krow0 * p.k_row;
  const __hip_bfloat16* k2 = (const __hip_bfloat16*)p.k2 + krow0 * p.k2_row;
  const __hip_bfloat16* v = (const __hip_bfloat16*)p.v + head * p.v_head +
                            krow0 * p.v_row;
  const int own = p.d1 / 64;                  // parts that are the head's own
  auto issue = [&](const int kt) {
    const long r0 = (long)kt * KT;
    const int left = klen - 1 - kt * KT;      // later rows repeat the last one
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int r = min(row + j * 8, left);
      const uint32_t kp = (uint32_t)(place ^ (j * 4 + (lane >> 4))) * 16;
      const uint32_t vp = (uint32_t)(place ^ ((lane >> 4) * 2)) * 16;
      const uint32_t ko = (uint32_t)(r * (int)p.k_row) * 2 + kp;
      const uint32_t k2o = (uint32_t)(r * (int)p.k2_row) * 2 + kp;
      const uint32_t vo = (uint32_t)(r * (int)p.v_row) * 2 + vp;
#pragma unroll
      for (int g = 0; g < G; ++g) {
        const uint32_t to = base + (g * PART + j * 512) * 2;
        if (g < own) load_lds16(ko, k + r0 * p.k_row + g * 64, to);
        else load_lds16(k2o, k2 + r0 * p.k2_row + (g - own) * 64, to);
      }
#pragma unroll
      for (int g = 0; g < VG; ++g)
        load_lds16(vo, v + r0 * p.v_row + g * 64,
                   base + ((G + (kt & 1) * VG + g) * PART + j * 512) * 2);
    }
  };

  float m[QT], l[QT];
  f32x4 acc[QT][VG * 4];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    // a sink is the first maximum and one more term of the sum
    m[t] = p.sink != nullptr ? p.sink[head] * LOG2E : MASKED;
    l[t] = p.sink != nullptr && gs == 0 ? 1.f : 0.f;
#pragma unroll
    for (int d = 0; d < VG * 4; ++d) acc[t][d] = {0.f, 0.f, 0.f, 0.f};
  }
  const float sl2 = p.scale * LOG2E;
  const int kt1 = last / KT;
  // in the value tile: row gs * 4 + gl / 4, columns gl % 4 * 4
  const int vrow = gs * 4 + (gl >> 2), vsw = (vrow >> 1) & 3;
  const int vat = vrow * 64 + (gl & 3) * 4;
  const __hip_bfloat16* kb = lds + gl * 64;
  const int ksw = gl >> 1;
  issue(first / KT);
  for (int kt = first / KT; kt <= kt1; ++kt) {
    landed_barrier<0>();                      // the tile is here, and whole
    const int k0 = kt * KT;
    const bool on = k0 <= whi && k0 + KT > wlo;
    f32x4 s[QT][4];
#pragma unroll
    for (int t = 0; t < QT; ++t)
#pragma unroll
      for (int c = 0; c < 4; ++c) s[t][c] = {0.f, 0.f, 0.f, 0.f};
    if (on) {
      __builtin_amdgcn_s_setprio(1);
#pragma unroll
      for (int g = 0; g < G; ++g)
#pragma unroll
        for (int h = 0; h < 2; ++h)
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            const mf_bf8 kf = frag8(kb + g * PART + c * 16 * 64 +
                                    ((h * 4 + gs) ^ ksw) * 8);
#pragma unroll
            for (int t = 0; t < QT; ++t)
              s[t][c] = mfma_bf16_k32(kf, qf[t][g * 2 + h], s[t][c]);
          }
      __builtin_amdgcn_s_setprio(0);
    }
    landed_barrier<0>();                      // the keys are read
    if (kt < kt1) issue(kt + 1);
    if (!on) continue;
    // every key seen by every query of the wave
    const bool whole = k0 + KT - 1 <= q0 && whi >= q0 + QT * 16 - 1 &&
                       (p.window <= 0 || k0 >= q0 + QT * 16 - p.window);
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      const int hi = q0 + t * 16 + gl;        // may lie past the end: unused
      const int lo = p.window > 0 ? hi - p.window + 1 : 0;
      float mx = MASKED;
#pragma unroll
      for (int c = 0; c < 4; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          float x = s[t][c][r] * sl2;
          if (!whole) {
            const int j = k0 + c * 16 + gs * 4 + r;
            x = j <= hi && j >= lo ? x : MASKED;
          }
          s[t][c][r] = x;
          mx = fmaxf(mx, x);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m[t], mx);
      if (__any(mn > m[t])) {                 // else nothing to rescale
        const float corr = exp2_fast(m[t] - mn);
        l[t] *= corr;
        m[t] = mn;
#pragma unroll
        for (int d = 0; d < VG * 4; ++d) acc[t][d] *= corr;
      }
    }
    const __hip_bfloat16* vb = lds + (G + (kt & 1) * VG) * PART + vat;
#pragma unroll
    for (int st = 0; st < 2; ++st) {
      mf_bf8 ph[QT], pl[QT];
#pragma unroll
      for (int t = 0; t < QT; ++t) {
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const float x = s[t][st * 2 + (i >> 2)][i & 3];
          float e = exp2_fast(x - m[t]);
          // a query that has seen no key yet has no maximum either
          if (!whole) e = x > MASKED ? e : 0.f;
          sum += e;
          __bf16 h, lw;
          split_bf16(e, h, lw);
          ph[t][i] = h;
          pl[t][i] = lw;
        }
        l[t] += sum;                          // per lane; summed at the end
      }
      __builtin_amdgcn_s_setprio(1);
#pragma unroll
      for (int d = 0; d < VG * 4; ++d) {
        const __hip_bfloat16* b = vb + (d >> 2) * PART + st * 32 * 64 +
                                  ((d & 3) ^ vsw) * 16;
        const mf_bf4 v0 = tr_read4(b), v1 = tr_read4(b + 16 * 64);
        const mf_bf8 vf = {v0[0], v0[1], v0[2], v0[3],
                           v1[0], v1[1], v1[2], v1[3]};
#pragma unroll
        for (int t = 0; t < QT; ++t) {
          acc[t][d] = mfma_bf16_k32(vf, ph[t], acc[t][d]);
          acc[t][d] = mfma_bf16_k32(vf, pl[t], acc[t][d]);
        }
      }
      __builtin_amdgcn_s_setprio(0);
    }
  }
#pragma unroll
  for (int t = 0; t < QT; ++t)
    finish_row<VG * 64>(p, head, t0 + (wave * QT + t) * 16 + gl, qrow0, qlen,
                        l[t], acc[t]);
}

template <int G>
void go_direct(const WindowAttnArgs& p, hipStream_t s) {
  const int grid = 8 * ((p.n_blocks * p.heads + 7) / 8);
  if (p.dv == 64) {
    window_direct_kernel<G, 1><<<grid, 256, 0, s>>>(p);
  } else {
    window_direct_kernel<G, 2><<<grid, 256, 0, s>>>(p);
  }
}

template <int DK>
void go_dv(const WindowAttnArgs& p, hipStream_t s) {
  const int grid = 8 * ((p.n_blocks * p.heads + 7) / 8);
#define WA_GO(DV, NW, QT)                                                     \
  window_attn_kernel<DK, DV, NW, QT><<<grid, NW * 64, 0, s>>>(p)
  if (p.dv <= 64) {
    WA_GO(64, 4, 2);
  } else if (p.dv <= 128) {
    WA_GO(128, 4, 2);
  } else {
    WA_GO(256, 8, 1);
  }
#undef WA_GO
}

}  // namespace

extern "C" {

int window_attn_rows() { return 128; }        // query rows per block

void launch_window_attn(const WindowAttnArgs* p, hipStream_t s) {
  const bool direct = p->d % 64 == 0 && p->d1 % 64 == 0 && p->d <= 192 &&
                      (p->dv == 64 || p->dv == 128) &&
                      // 32-bit offsets within a tile
                      p->k_row < (1 << 23) && p->k2_row < (1 << 23) &&
                      p->v_row < (1 << 23);
  if (direct) {
    if (p->d == 64) go_direct<1>(*p, s);
    else if (p->d == 128) go_direct<2>(*p, s);
    else go_direct<3>(*p, s);
    return;
  }
  if (p->d <= 64) go_dv<64>(*p, s);
  else if (p->d <= 128) go_dv<128>(*p, s);
  else if (p->d <= 192) go_dv<192>(*p, s);
  else go_dv<256>(*p, s);
}

}  // extern "C"
