// Causal attention over paged keys and values (gfx950): grouped heads, key and
// value sizes of their own, soft-capped scores, a silent key of score zero (a
// sink), a sliding window, and differential heads.  Pages are [page, kv head,
// row, size]: a head's 16 rows are one contiguous piece.
//
// A differential head (MAPS 2) has two queries and two keys side by side, whose
// softmaxes weigh the same values; its output is o1 - lam o2, divided by its
// root mean square.  Prompts keep both maps' sums in one wave, so values are read
// once; decode takes the maps as two query heads whose queries are zero in each
// other's half of the key.
//
//   prompt   128 query rows of one head per workgroup over 64-key tiles.  S^T =
//            K Q^T, so a query is a lane column and the softmax registers are
//            the next product's B operand, O^T += V^T P^T, with V read from LDS
//            through the transposing read.  Page numbers run two tiles ahead and
//            rows one tile ahead of the products.
//   decode   a workgroup takes one sequence, one kv head with up to 16 of its
//            query heads, and one split of the keys; every wave walks its own 32
//            keys a step, without barriers: key rows go from global memory
//            straight into MFMA operands, value rows through a wave's own LDS
//            strip.  The waves meet at the end, the splits in a second kernel.
//   rows     one wave per (query row, head), any sizes, bf16 or f32.
//
// A window starts the walk over keys at the first one that a row sees.
//
// A soft cap bounds the scores; when its exponentials fit f32 with room (BOUND),
// nothing has to be subtracted, and the running maximum and every rescaling go.
//
// Scores and weights are f32.  Weights enter the second product as two bf16
// (hi + lo), which keeps 16 bits of them.  The sink is the running maximum's
// first value (zero) and one more term of the final sum.
#include "mfma_util.h"
#include "moe_args.h"
#include "vec_io.h"

namespace {

// score * log2(e) of a raw product x
struct ScoreMap {
  float scale, cap, turn;     // cap 0: scale only
  DEV_INLINE explicit ScoreMap(const PagedAttnArgs& p) {
    if (p.softcap > 0.f) {
      cap = p.softcap * LOG2E;
      turn = 2.f * LOG2E * p.scale / p.softcap;
      scale = 0.f;
    } else {
      cap = turn = 0.f;
      scale = p.scale * LOG2E;
    }
  }
  DEV_INLINE float operator()(float x) const {
    if (cap == 0.f) return x * scale;
    // tanh(z) = 1 - 2 / (1 + e^2z)
    return cap - 2.f * cap * rcp_f(1.f + exp2_fast(x * turn));
  }
};

// largest |score| * log2(e) whose exponential may be summed as it is
constexpr float BOUND_LOG2 = 100.f;

constexpr int KT = 64;

// A wave keeps QT sums: of QT query tiles, or (MAPS 2) of one tile's two maps.
// SPLIT (MAPS 2, QT 1): one tile's two maps are a pair of waves, which meet in
// LDS at the end.
template <int DK, int DV, int NW, int QT, bool BOUND, int MAPS = 1>
__global__ __launch_bounds__(NW * 64, (DK + DV) > 256 ? 1 : 2)
void paged_prefill_kernel(const PagedAttnArgs p) {
  static_assert(MAPS == 1 || (MAPS == 2 && QT <= 2 && !BOUND), "maps");
  constexpr bool SPLIT = MAPS == 2 && QT == 1;
  constexpr int DKM = DK * MAPS;              // a key row, maps side by side
  constexpr int KP = DKM + 16, VP = DV + 16;  // 8 banks per row
  constexpr int SM = SPLIT ? 1 : MAPS;        // maps of a wave
  constexpr int WR = QT / SM * 16;            // query rows of a wave
  constexpr int ROWS = SPLIT ? NW / 2 * WR : NW * WR;   // or SUB pieces of 128
  constexpr int SUB = 128 / ROWS;
  constexpr int NT = NW * 64;
  constexpr int KPC = KT * DKM / 8 / NT, VPC = (KT * DV / 8 + NT - 1) / NT;
  constexpr bool VFULL = VPC * NT * 8 == KT * DV;
  static_assert(KPC * NT * 8 == KT * DKM, "tile");
  constexpr int TILE = KT * (KP + VP), MEET = SPLIT ? NW / 2 * DV * 32 : 0;
  __shared__ __attribute__((aligned(16)))
  __hip_bfloat16 ks[TILE > MEET ? TILE : MEET];
  __hip_bfloat16* vs = ks + KT * KP;
  const int tid = threadIdx.x, lane = tid & 63;
  const int own = SPLIT ? (tid >> 6) & 1 : 0; // SPLIT: the wave's map
  const int wave = SPLIT ? tid >> 7 : tid >> 6;
  const int gl = lane & 15, gs = lane >> 4;

  // workgroups go round the 8 XCDs: give each XCD whole heads, so that the
  // query tiles of a head (and of its neighbours with the same keys) share L2
  const int nb = p.n_blocks * SUB;
  const int items = nb * p.heads, per = (items + 7) / 8;
  const int work = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
  if ((blockIdx.x >> 3) >= per || work >= items) return;
  const int head = work / nb, kvh = head / (p.heads / p.kv_heads);
  const int piece = nb - 1 - work % nb;
  const int* bi = p.blocks + piece / SUB * 2;
  const int* si = p.seq_info + bi[0] * 3;
  const int qrow0 = si[0], qlen = si[1], qoff = si[2];
  const int t0 = bi[1] + piece % SUB * ROWS;  // first query of the piece
  if (SUB > 1 && t0 >= qlen) return;
  const int klen = qoff + qlen;
  const int* table = p.tables + (size_t)bi[0] * p.max_pages;

  const __hip_bfloat16* q = (const __hip_bfloat16*)p.q + head * p.q_head;
  const __hip_bfloat16* k = (const __hip_bfloat16*)p.k +
                            (size_t)kvh * p.page_size * p.d * MAPS;
  const __hip_bfloat16* v = (const __hip_bfloat16*)p.v +
                            (size_t)kvh * p.page_size * p.dv;
  const size_t k_page = (size_t)p.kv_heads * p.page_size * p.d * MAPS;
  const size_t v_page = (size_t)p.kv_heads * p.page_size * p.dv;

  mf_bf8 qf[QT][DK / 32];
  int qpos[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    const int r = t0 + wave * WR + t / SM * 16 + gl;
    qpos[t] = qoff + r;                       // may lie past the end: unused
    const __hip_bfloat16* qr = q + (size_t)(qrow0 + min(r, qlen - 1)) * p.q_row +
                               (own + t % SM) * p.d;
#pragma unroll
    for (int s = 0; s < DK / 32; ++s) {
      const int d = s * 32 + gs * 8;
      mf_bf8 z = {};
      qf[t][s] = d < p.d ? frag8(qr + d) : z;
    }
  }
  const int last = min(qoff + t0 + ROWS - 1, klen - 1);
  const int whi = min(qoff + t0 + (wave + 1) * WR - 1, klen - 1);
  const int kt1 = last / KT;
  // keys before a window; a bounded score's form has none
  const int behind = !BOUND && p.window > 0 ? p.window : 1 << 30;
  const int wlo = qoff + t0 + wave * WR - behind + 1;
  const int kt0 = max(qoff + t0 - behind + 1, 0) / KT;

  // keys past the end repeat the last one, so every row read is a written one
  int kpg[KPC], vpg[VPC];
  auto pages = [&](int kt) {
#pragma unroll
    for (int i = 0; i < KPC; ++i)
      kpg[i] = table[min(kt * KT + (tid + i * NT) / (DKM / 8), klen - 1) >>
                     p.page_shift];
#pragma unroll
    for (int i = 0; i < VPC; ++i)
      vpg[i] = table[min(kt * KT + (tid + i * NT) / (DV / 8), klen - 1) >>
                     p.page_shift];
  };
  u32x4 kr[KPC], vr[VPC];
  const u32x4 zero4 = {0, 0, 0, 0};
  auto fetch = [&](int kt) {
#pragma unroll
    for (int i = 0; i < KPC; ++i) {
      const int e = tid + i * NT, cm = (e % (DKM / 8)) * 8;
      const int map = MAPS == 1 ? 0 : cm / DK, c = cm - map * DK;
      const int at = min(kt * KT + e / (DKM / 8), klen - 1) &
                     (p.page_size - 1);
      kr[i] = c < p.d ? *reinterpret_cast<const u32x4*>(
                            k + kpg[i] * k_page + (at * MAPS + map) * p.d + c)
                      : zero4;
    }
#pragma unroll
    for (int i = 0; i < VPC; ++i) {
      const int e = tid + i * NT, c = (e % (DV / 8)) * 8;
      const int at = min(kt * KT + e / (DV / 8), klen - 1) & (p.page_size - 1);
      vr[i] = c < p.dv ? *reinterpret_cast<const u32x4*>(
                             v + vpg[i] * v_page + at * p.dv + c)
                       : zero4;
    }
  };
  auto land = [&]() {
#pragma unroll
    for (int i = 0; i < KPC; ++i) {
      const int e = tid + i * NT, key = e / (DKM / 8);
      const int c = (e % (DKM / 8)) * 8;
      *reinterpret_cast<u32x4*>(&ks[key * KP + c]) = kr[i];
    }
#pragma unroll
    for (int i = 0; i < VPC; ++i) {
      const int e = tid + i * NT, key = e / (DV / 8), c = (e % (DV / 8)) * 8;
      if (VFULL || e < KT * DV / 8)
        *reinterpret_cast<u32x4*>(&vs[key * VP + c]) = vr[i];
    }
  };

  float m[QT], l[QT];
  f32x4 acc[QT][DV / 16];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    m[t] = BOUND || p.sink ? 0.f : MASKED;
    l[t] = 0.f;
#pragma unroll
    for (int d = 0; d < DV / 16; ++d) acc[t][d] = {0.f, 0.f, 0.f, 0.f};
  }
  const ScoreMap score(p);
  pages(kt0);
  fetch(kt0);
  pages(min(kt0 + 1, kt1));
  for (int kt = kt0; kt <= kt1; ++kt) {
    __syncthreads();                          // the tile before is read
    land();
    __syncthreads();
    if (kt < kt1) {
      fetch(kt + 1);
      pages(min(kt + 2, kt1));
    }
    const int k0 = kt * KT;
    // barriers stay uniform
    if (k0 > whi || k0 + KT - 1 < wlo) continue;

    f32x4 s[QT][4];
#pragma unroll
    for (int t = 0; t < QT; ++t)
#pragma unroll
      for (int c = 0; c < 4; ++c) s[t][c] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < 4; ++c)
#pragma unroll
      for (int st = 0; st < DK / 32; ++st)
#pragma unroll
        for (int map = 0; map < SM; ++map) {
          const mf_bf8 kf = frag8(
              &ks[(c * 16 + gl) * KP + (own + map) * DK + st * 32 + gs * 8]);
#pragma unroll
          for (int t = map; t < QT; t += SM)
            s[t][c] = mfma_bf16_k32(kf, qf[t][st], s[t][c]);
        }
    mf_bf8 ph[QT][2], pl[QT][2];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
      const int hi = qpos[t], lo = hi - behind;
      float mn = 0.f;
      if (!BOUND) {
        float mx = MASKED;
#pragma unroll
        for (int c = 0; c < 4; ++c)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int j = k0 + c * 16 + gs * 4 + r;
            const float x =
                j <= hi && j > lo ? score(s[t][c][r]) : MASKED;
            s[t][c][r] = x;
            mx = fmaxf(mx, x);
          }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
        mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        mn = fmaxf(m[t], mx);
        const float corr = exp2_fast(m[t] - mn);
        m[t] = mn;
        l[t] *= corr;
#pragma unroll
        for (int d = 0; d < DV / 16; ++d) acc[t][d] *= corr;
      }
      float sum = 0.f;
#pragma unroll
      for (int c = 0; c < 4; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = k0 + c * 16 + gs * 4 + r;
          const float x = BOUND ? score(s[t][c][r]) : s[t][c][r] - mn;
          const float e =
              j <= hi && (BOUND || j > lo) ? exp2_fast(x) : 0.f;
          sum += e;
          __bf16 h, lw;
          split_bf16(e, h, lw);
          ph[t][c >> 1][(c & 1) * 4 + r] = h;
          pl[t][c >> 1][(c & 1) * 4 + r] = lw;
        }
      l[t] += sum;                            // per lane; summed at the end
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

  float sums[QT];
#pragma unroll
  for (int t = 0; t < QT; ++t) {
    sums[t] = l[t];
    sums[t] += __shfl_xor(sums[t], 16, 64);
    sums[t] += __shfl_xor(sums[t], 32, 64);
    if (p.sink) sums[t] += exp2_fast(-m[t]);
  }
  if constexpr (MAPS == 2) {
    // the difference of the maps, over its root mean square, in acc[0]
    float f1 = 1.f / sums[0], f2 = p.lam[0];
    f32x4* meet = (f32x4*)ks + wave * DV * 4 + lane;
    if constexpr (SPLIT) {
      __syncthreads();                        // keys and values are read
      if (own) {
#pragma unroll
        for (int d = 0; d < DV / 16; ++d) meet[d * 64] = acc[0][d] * f1;
      }
      __syncthreads();
      if (own) return;
    } else {
      f2 /= sums[1];
    }
    float ss = 0.f;
#pragma unroll
    for (int d = 0; d < DV / 16; ++d) {
      f32x4 other;
      if constexpr (SPLIT) other = meet[d * 64];
      else other = acc[QT - 1][d];
      acc[0][d] = acc[0][d] * f1 - other * f2;
#pragma unroll
      for (int e = 0; e < 4; ++e) ss += acc[0][d][e] * acc[0][d][e];
    }
    ss += __shfl_xor(ss, 16, 64);
    ss += __shfl_xor(ss, 32, 64);
    sums[0] = sqrtf(ss / p.dv + p.out_eps) / p.out_scale;
  }
#pragma unroll
  for (int t = 0; t < QT / SM; ++t) {
    const int r = t0 + wave * WR + t * 16 + gl;
    if (r >= qlen) continue;
    const float inv = 1.f / sums[t];
    __hip_bfloat16* o = (__hip_bfloat16*)p.out + (size_t)(qrow0 + r) * p.o_row +
                        (size_t)head * p.dv;
#pragma unroll
    for (int d = 0; d < DV / 16; ++d) {
      const int c = d * 16 + gs * 4;
      if (c >= p.dv) continue;
      union { uint2 u; __hip_bfloat16 e[4]; } ov;
#pragma unroll
      for (int e = 0; e < 4; ++e) ov.e[e] = f2bf(acc[t][d][e] * inv);
      *reinterpret_cast<uint2*>(o + c) = ov.u;
    }
  }
}

constexpr int DW = 4;                         // waves of a decode workgroup

// DK: a key row, maps side by side
template <int DK, int DV, bool BOUND, int MAPS = 1>
__global__ __launch_bounds__(DW * 64, (DK + DV) > 256 ? 1 : 2)
void paged_decode_kernel(const PagedAttnArgs p) {
  constexpr int VP = DV + 16, VL = DV / 16;   // VL 16-byte loads of 32 rows
  constexpr int STRIP = 32 * VP * 2;          // bytes of a wave's value rows
  constexpr int ACC = DV * 16 * 4;            // bytes of a wave's sums
  constexpr int PER = STRIP > ACC ? STRIP : ACC;
  __shared__ __attribute__((aligned(16))) char smem[DW * PER];
  __shared__ float ml_s[2][DW][16];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int gl = lane & 15, gs = lane >> 4;
  const int split = blockIdx.x, seq = blockIdx.y;
  // (head, map) pairs of a kv head, 16 at a time
  const int ratio = p.heads / p.kv_heads * MAPS, tiles = (ratio + 15) / 16;
  const int kvh = blockIdx.z / tiles, r0 = (blockIdx.z % tiles) * 16;
  const int h0 = kvh * ratio + r0, nh = min(16, ratio - r0);
  const int kd = p.d * MAPS;
  const int pos = p.ctx[seq] - 1;
  const int lo = !BOUND && p.window > 0 ? max(pos - p.window + 1, 0) : 0;
  const int first = lo / (DW * 32);
  const int steps = pos / (DW * 32) + 1 - first;
  const int per = (steps + p.splits - 1) / p.splits;
  const int s_beg = first + split * per;
  const int s_end = min(s_beg + per, first + steps);
  const int* table = p.tables + (size_t)seq * p.max_pages;
  const size_t k_page = (size_t)p.kv_heads * p.page_size * kd;
  const size_t v_page = (size_t)p.kv_heads * p.page_size * p.dv;
  const __hip_bfloat16* k = (const __hip_bfloat16*)p.k +
                            (size_t)kvh * p.page_size * kd;
  const __hip_bfloat16* v = (const __hip_bfloat16*)p.v +
                            (size_t)kvh * p.page_size * p.dv;
  __hip_bfloat16* vs = (__hip_bfloat16*)(smem + wave * PER);

  const int qh = h0 + min(gl, nh - 1);
  const __hip_bfloat16* q = (const __hip_bfloat16*)p.q +
      (size_t)seq * p.q_row + (size_t)(qh / MAPS) * p.q_head;
  const int q_lo = qh % MAPS * p.d;           // its map's part of the key
  mf_bf8 qf[DK / 32];
#pragma unroll
  for (int s = 0; s < DK / 32; ++s) {
    const int d = s * 32 + gs * 8;
    mf_bf8 z = {};
    qf[s] = d >= q_lo && d < q_lo + p.d ? frag8(q + d) : z;
  }
  float m = BOUND || p.sink ? 0.f : MASKED, l = 0.f;
  f32x4 acc[DV / 16];
#pragma unroll
  for (int d = 0; d < DV / 16; ++d) acc[d] = {0.f, 0.f, 0.f, 0.f};
  const ScoreMap score(p);

  mf_bf8 kr[2][DK / 32];
  u32x4 vr[VL];
  const u32x4 zero4 = {0, 0, 0, 0};
  const mf_bf8 zero8 = {};
  // 16 keys are part of one page; pages past the last are the last again
  int pg0 = 0, pg1 = 0, at0 = 0, at1 = 0;
  auto pages = [&](int step) {
    const int j0 = step * (DW * 32) + wave * 32;
    const int a = min(j0, pos & ~15), b = min(j0 + 16, pos & ~15);
    pg0 = table[a >> p.page_shift];
    pg1 = table[b >> p.page_shift];
    at0 = a & (p.page_size - 1);
    at1 = b & (p.page_size - 1);
  };
  auto fetch = [&]() {
    const __hip_bfloat16* k0 = k + pg0 * k_page + (at0 + gl) * kd;
    const __hip_bfloat16* k1 = k + pg1 * k_page + (at1 + gl) * kd;
#pragma unroll
    for (int s = 0; s < DK / 32; ++s) {
      const int d = s * 32 + gs * 8;
      kr[0][s] = d < kd ? frag8(k0 + d) : zero8;
      kr[1][s] = d < kd ? frag8(k1 + d) : zero8;
    }
    const __hip_bfloat16* v0 = v + pg0 * v_page + at0 * p.dv;
    const __hip_bfloat16* v1 = v + pg1 * v_page + at1 * p.dv;
#pragma unroll
    for (int i = 0; i < VL; ++i) {
      const int e = i * 64 + lane, key = e / (DV / 8), d = (e % (DV / 8)) * 8;
      const __hip_bfloat16* row = (key < 16 ? v0 : v1) + (key & 15) * p.dv;
      vr[i] = d < p.dv ? *reinterpret_cast<const u32x4*>(row + d) : zero4;
    }
  };
  if (s_beg < s_end) {
    pages(s_beg);
    fetch();
    pages(min(s_beg + 1, s_end - 1));
  }
  for (int step = s_beg; step < s_end; ++step) {
    const int j0 = step * (DW * 32) + wave * 32;
    f32x4 s[2];
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      s[c] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int st = 0; st < DK / 32; ++st)
        s[c] = mfma_bf16_k32(kr[c][st], qf[st], s[c]);
    }
    // rows that hold no key of this sequence may hold anything
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
    for (int i = 0; i < VL; ++i) {
      const int e = i * 64 + lane, key = e / (DV / 8), d = (e % (DV / 8)) * 8;
      *reinterpret_cast<u32x4*>(&vs[key * VP + d]) =
          j0 + key <= pos ? vr[i] : zero4;
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    if (step + 1 < s_end) {
      fetch();
      pages(min(step + 2, s_end - 1));
    }
    float mn = 0.f;
    if (!BOUND) {
      float mx = MASKED;
#pragma unroll
      for (int c = 0; c < 2; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = j0 + c * 16 + gs * 4 + r;
          const float x = j <= pos && j >= lo ? score(s[c][r]) : MASKED;
          s[c][r] = x;
          mx = fmaxf(mx, x);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      mn = fmaxf(m, mx);
      const float corr = exp2_fast(m - mn);
      m = mn;
      l *= corr;
#pragma unroll
      for (int d = 0; d < DV / 16; ++d) acc[d] *= corr;
    }
    mf_bf8 ph, pl;
#pragma unroll
    for (int c = 0; c < 2; ++c)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = j0 + c * 16 + gs * 4 + r;
        const float x = BOUND ? score(s[c][r]) : s[c][r] - mn;
        const float e =
            j <= pos && (BOUND || j >= lo) ? exp2_fast(x) : 0.f;
        l += e;
        __bf16 h, lw;
        split_bf16(e, h, lw);
        ph[c * 4 + r] = h;
        pl[c * 4 + r] = lw;
      }
#pragma unroll
    for (int d = 0; d < DV / 16; ++d) {
      const __hip_bfloat16* b =
          &vs[(gs * 4 + (gl >> 2)) * VP + d * 16 + (gl & 3) * 4];
      const mf_bf4 v0 = tr_read4(b), v1 = tr_read4(b + 16 * VP);
      const mf_bf8 vf = {v0[0], v0[1], v0[2], v0[3],
                         v1[0], v1[1], v1[2], v1[3]};
      acc[d] = mfma_bf16_k32(vf, ph, acc[d]);
      acc[d] = mfma_bf16_k32(vf, pl, acc[d]);
    }
  }

  // the waves' sums on one scale, then added
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (gs == 0) {
    ml_s[0][wave][gl] = m;
    ml_s[1][wave][gl] = l;
  }
  __syncthreads();
  float M = m, L = 0.f;
#pragma unroll
  for (int w = 0; w < DW; ++w) M = fmaxf(M, ml_s[0][w][gl]);
#pragma unroll
  for (int w = 0; w < DW; ++w)
    L += ml_s[1][w][gl] * exp2_fast(ml_s[0][w][gl] - M);
  const float mine = exp2_fast(m - M);
  f32x4* sums = (f32x4*)(smem + wave * PER);
#pragma unroll
  for (int d = 0; d < DV / 16; ++d) sums[d * 64 + lane] = acc[d] * mine;
  __syncthreads();
  if (gl >= nh) return;
  const size_t row = (size_t)seq * p.heads * MAPS + h0 + gl;
  const size_t part = (size_t)split * p.rows * p.heads * MAPS + row;
  const bool parts = MAPS > 1 || p.splits > 1;
  if (parts && wave == 0 && gs == 0) {
    p.part_ml[part * 2] = M;
    p.part_ml[part * 2 + 1] = L;
  }
  const float inv = 1.f / (L + (p.sink ? exp2_fast(-M) : 0.f));
  for (int d = wave; d < DV / 16; d += DW) {
    const int c = d * 16 + gs * 4;
    if (c >= p.dv) continue;
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < DW; ++w)
      o += ((const f32x4*)(smem + w * PER))[d * 64 + lane];
    if (parts) {
      *reinterpret_cast<f32x4*>(&p.part_o[part * p.dv + c]) = o;
    } else {
      union { uint2 u; __hip_bfloat16 e[4]; } ov;
#pragma unroll
      for (int r = 0; r < 4; ++r) ov.e[r] = f2bf(o[r] * inv);
      *reinterpret_cast<uint2*>((__hip_bfloat16*)p.out + (size_t)seq * p.o_row +
                                (size_t)(h0 + gl) * p.dv + c) = ov.u;
    }
  }
}

// one wave per (sequence, head): sum of the splits' partials
__global__ __launch_bounds__(64) void paged_combine_kernel(
    const PagedAttnArgs p) {
  __shared__ float f[64];                     // splits <= 64
  const size_t row = blockIdx.x;              // seq * heads + head
  const size_t rows = (size_t)p.rows * p.heads;
  const int tid = threadIdx.x;
  const bool on = tid < p.splits;
  const float m = on ? p.part_ml[(tid * rows + row) * 2] : MASKED;
  const float l = on ? p.part_ml[(tid * rows + row) * 2 + 1] : 0.f;
  const float M = wave_max(m);
  const float w = on ? exp2_fast(m - M) : 0.f;
  f[tid] = w / (wave_sum(l * w) + (p.sink ? exp2_fast(-M) : 0.f));
  __syncthreads();
  __hip_bfloat16* out = (__hip_bfloat16*)p.out +
      (row / p.heads) * p.o_row + (row % p.heads) * p.dv;
  for (int d = tid * 4; d < p.dv; d += 256) {
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (int s = 0; s < p.splits; ++s)
      o += *reinterpret_cast<const f32x4*>(
               &p.part_o[(s * rows + row) * p.dv + d]) * f[s];
    union { uint2 u; __hip_bfloat16 e[4]; } ov;
#pragma unroll
    for (int r = 0; r < 4; ++r) ov.e[r] = f2bf(o[r]);
    *reinterpret_cast<uint2*>(out + d) = ov.u;
  }
}

// The same of a differential head's two maps, then their difference over its
// root mean square.  dv <= 256
__global__ __launch_bounds__(64) void paged_difference_kernel(
    const PagedAttnArgs p) {
  __shared__ float f[2][64];                  // splits <= 64
  const size_t row = blockIdx.x;              // seq * heads + head
  const size_t rows = (size_t)p.rows * p.heads * 2;
  const int tid = threadIdx.x;
  const bool on = tid < p.splits;
#pragma unroll
  for (int map = 0; map < 2; ++map) {
    const size_t at = tid * rows + row * 2 + map;
    const float m = on ? p.part_ml[at * 2] : MASKED;
    const float l = on ? p.part_ml[at * 2 + 1] : 0.f;
    const float M = p.sink ? fmaxf(wave_max(m), 0.f) : wave_max(m);
    const float w = on ? exp2_fast(m - M) : 0.f;
    f[map][tid] = w / (wave_sum(l * w) + (p.sink ? exp2_fast(-M) : 0.f)) *
                  (map ? -p.lam[0] : 1.f);
  }
  __syncthreads();
  const int d = tid * 4;
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  if (d < p.dv) {
#pragma unroll 4
    for (int s = 0; s < p.splits; ++s) {
      const float* at = &p.part_o[(s * rows + row * 2) * p.dv + d];
      o += *reinterpret_cast<const f32x4*>(at) * f[0][s];
      o += *reinterpret_cast<const f32x4*>(at + p.dv) * f[1][s];
    }
  }
  const float ss = wave_sum(o[0] * o[0] + o[1] * o[1] + o[2] * o[2] +
                            o[3] * o[3]);
  const float inv = p.out_scale / sqrtf(ss / p.dv + p.out_eps);
  if (d >= p.dv) return;
  union { uint2 u; __hip_bfloat16 e[4]; } ov;
#pragma unroll
  for (int r = 0; r < 4; ++r) ov.e[r] = f2bf(o[r] * inv);
  *reinterpret_cast<uint2*>((__hip_bfloat16*)p.out +
                            (row / p.heads) * p.o_row +
                            (row % p.heads) * p.dv + d) = ov.u;
}

// NACC: value dimensions per lane (dv <= 64 * NACC)
template <typename T, int NACC, int MAPS>
__global__ __launch_bounds__(256) void paged_rows_kernel(
    const PagedAttnArgs p) {
  extern __shared__ float rows_smem[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const long item = (long)blockIdx.x * 4 + wave;
  if (item >= (long)p.rows * p.heads) return;       // whole wave leaves
  const int row = (int)(item / p.heads), head = (int)(item % p.heads);
  const int kvh = head / (p.heads / p.kv_heads);
  const int kd = p.d * MAPS;
  float* q = rows_smem + wave * (kd + 64 * MAPS);
  float* pr = q + kd;
  const T* qp = (const T*)p.q + row * p.q_row + head * p.q_head;
  for (int i = lane; i < kd; i += 64) q[i] = to_f(qp[i]);
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
  const int seq = p.ctx != nullptr ? row : p.row_info[row * 2];
  const int pos = p.ctx != nullptr ? p.ctx[row] - 1 : p.row_info[row * 2 + 1];
  const int lo = p.window > 0 ? max(pos - p.window + 1, 0) : 0;
  const int* table = p.tables + (size_t)seq * p.max_pages;
  auto key_row = [&](int j) -> size_t {
    return ((size_t)table[j / p.page_size] * p.kv_heads + kvh) * p.page_size +
           j % p.page_size;
  };
  float m[MAPS], l[MAPS], acc[MAPS][NACC];
#pragma unroll
  for (int a = 0; a < MAPS; ++a) {
    m[a] = p.sink ? 0.f : -INFINITY;
    l[a] = p.sink ? 1.f : 0.f;
#pragma unroll
    for (int i = 0; i < NACC; ++i) acc[a][i] = 0.f;
  }

  for (int j0 = lo; j0 <= pos; j0 += 64) {
    const int j = j0 + lane;
#pragma unroll
    for (int a = 0; a < MAPS; ++a) {
      float s = -INFINITY;
      if (j <= pos) {
        const T* kr = (const T*)p.k + key_row(j) * kd + a * p.d;
        float dot = 0.f;
        for (int i = 0; i < p.d; ++i) dot += q[a * p.d + i] * to_f(kr[i]);
        s = dot * p.scale;
        if (p.softcap > 0.f) s = p.softcap * tanhf(s / p.softcap);
      }
      const float mn = fmaxf(m[a], wave_max(s));
      const float e = expf(s - mn);
      const float corr = expf(m[a] - mn);
      l[a] = l[a] * corr + wave_sum(e);
      m[a] = mn;
      pr[a * 64 + lane] = e;
#pragma unroll
      for (int i = 0; i < NACC; ++i) acc[a][i] *= corr;
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
    const int n = min(64, pos - j0 + 1);
    for (int t = 0; t < n; ++t) {
      const T* vr = (const T*)p.v + key_row(j0 + t) * p.dv;
#pragma unroll
      for (int i = 0; i < NACC; ++i) {
        const int d = i * 64 + lane;
        const float x = d < p.dv ? to_f(vr[d]) : 0.f;
#pragma unroll
        for (int a = 0; a < MAPS; ++a) acc[a][i] += pr[a * 64 + t] * x;
      }
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
  }
  T* op = (T*)p.out + row * p.o_row + (size_t)head * p.dv;
  float f = 1.f;
#pragma unroll
  for (int i = 0; i < NACC; ++i) acc[0][i] /= l[0];
  if constexpr (MAPS == 2) {
    float ss = 0.f;                             // dimensions past dv are zero
#pragma unroll
    for (int i = 0; i < NACC; ++i) {
      acc[0][i] -= p.lam[0] * (acc[1][i] / l[1]);
      ss += acc[0][i] * acc[0][i];
    }
    f = p.out_scale / sqrtf(wave_sum(ss) / p.dv + p.out_eps);
  }
#pragma unroll
  for (int i = 0; i < NACC; ++i) {
    const int d = i * 64 + lane;
    if (d < p.dv) op[d] = from_f<T>(acc[0][i] * f);
  }
}

bool bounded(const PagedAttnArgs& p) {
  return p.softcap > 0.f && p.softcap * LOG2E <= BOUND_LOG2 && p.window == 0;
}

template <int DK>
void prefill_dv(const PagedAttnArgs& p, hipStream_t s) {
  const int grid = 8 * ((p.n_blocks * p.heads + 7) / 8);
#define PP_GO(DV, NW, QT)                                                     \
  do {                                                                        \
    if (bounded(p))                                                           \
      paged_prefill_kernel<DK, DV, NW, QT, true><<<grid, NW * 64, 0, s>>>(p); \
    else                                                                      \
      paged_prefill_kernel<DK, DV, NW, QT, false><<<grid, NW * 64, 0, s>>>(p);\
  } while (0)
  if (p.dv <= 64) PP_GO(64, 4, 2);
  else if (p.dv <= 96) PP_GO(96, 4, 2);
  else if (p.dv <= 128) PP_GO(128, 4, 2);
  else PP_GO(256, 8, 1);
#undef PP_GO
}

// two maps: a wave's two sums are one query tile's; sums of 256 values take a
// wave each
template <int DK>
void prefill_maps(const PagedAttnArgs& p, hipStream_t s) {
#define PP_GO(DV, QT)                                                         \
  do {                                                                        \
    const int grid = 8 * ((p.n_blocks * (2 / QT) * p.heads + 7) / 8);         \
    paged_prefill_kernel<DK, DV, 8, QT, false, 2><<<grid, 512, 0, s>>>(p);    \
  } while (0)
  if (p.dv <= 64) PP_GO(64, 2);
  else if (p.dv <= 96) PP_GO(96, 2);
  else if (p.dv <= 128) PP_GO(128, 2);
  else PP_GO(256, 1);
#undef PP_GO
}

template <int DK, int MAPS = 1>
void decode_dv(const PagedAttnArgs& p, hipStream_t s) {
  const int tiles = (p.heads / p.kv_heads * MAPS + 15) / 16;
  const dim3 grid(p.splits, p.rows, p.kv_heads * tiles);
#define PD_GO(DV)                                                             \
  do {                                                                        \
    if constexpr (MAPS > 1)                                                   \
      paged_decode_kernel<DK, DV, false, MAPS><<<grid, DW * 64, 0, s>>>(p);   \
    else if (bounded(p))                                                      \
      paged_decode_kernel<DK, DV, true><<<grid, DW * 64, 0, s>>>(p);          \
    else                                                                      \
      paged_decode_kernel<DK, DV, false><<<grid, DW * 64, 0, s>>>(p);         \
  } while (0)
  if (p.dv <= 64) PD_GO(64);
  else if (p.dv <= 96) PD_GO(96);
  else if (p.dv <= 128) PD_GO(128);
  else PD_GO(256);
#undef PD_GO
}

template <typename T>
void paged_rows_t(const PagedAttnArgs& p, hipStream_t s) {
  const int grid = (int)(((long)p.rows * p.heads + 3) / 4);
  const size_t lds = sizeof(float) * 4 * p.maps * (p.d + 64);
#define PR_GO(N)                                                              \
  do {                                                                        \
    if (p.maps == 2) {                                                        \
      paged_rows_kernel<T, N, 2><<<grid, 256, lds, s>>>(p);                   \
    } else {                                                                  \
      paged_rows_kernel<T, N, 1><<<grid, 256, lds, s>>>(p);                   \
    }                                                                         \
  } while (0)
  if (p.dv <= 64) PR_GO(1);
  else if (p.dv <= 128) PR_GO(2);
  else if (p.dv <= 256) PR_GO(4);
  else if (p.dv <= 512) PR_GO(8);
  else PR_GO(16);
#undef PR_GO
}

}  // namespace

extern "C" {

int paged_block_rows() { return 128; }        // query rows per prompt block

void launch_paged_prefill(const PagedAttnArgs* p, hipStream_t s) {
  if (p->maps == 2) {
    if (p->d <= 64) prefill_maps<64>(*p, s);
    else prefill_maps<128>(*p, s);
    return;
  }
  if (p->d <= 64) prefill_dv<64>(*p, s);
  else if (p->d <= 128) prefill_dv<128>(*p, s);
  else prefill_dv<256>(*p, s);
}

void launch_paged_decode(const PagedAttnArgs* p, hipStream_t s) {
  if (p->maps == 2) {
    if (p->d <= 32) decode_dv<64, 2>(*p, s);
    else if (p->d <= 64) decode_dv<128, 2>(*p, s);
    else decode_dv<256, 2>(*p, s);
    paged_difference_kernel<<<p->rows * p->heads, 64, 0, s>>>(*p);
    return;
  }
  if (p->d <= 64) decode_dv<64>(*p, s);
  else if (p->d <= 128) decode_dv<128>(*p, s);
  else decode_dv<256>(*p, s);
  if (p->splits > 1) {
    paged_combine_kernel<<<p->rows * p->heads, 64, 0, s>>>(*p);
  }
}

void launch_paged_rows(const PagedAttnArgs* p, int f32, hipStream_t s) {
  if (f32) paged_rows_t<float>(*p, s);
  else paged_rows_t<__hip_bfloat16>(*p, s);
}

}  // extern "C"
