// Generalized delta rule over prompts, 16 tokens at a time (gfx950), in f32 on
// the matrix cores (v_mfma_f32_16x16x4_f32), any f32 or bf16 projections.
//
// Write c_t for the chunk's cumulative log decay and scale the vectors by it:
//   U_t = u_t e^{c_{t-1}}   R_t = r_t e^{c_t}   K_t = k_t e^{-c_t}
//   B_t = (a u)_t e^{-c_t}
// (e^{16 * decay_scale} bounds the factors, so f32 keeps every product to its
// own rounding).  With S the state before the chunk, p_t = u_t^T S_{t-1} obeys
//   (I + tril_(U B^T)) P = U S + tril_(U K^T) V         (tril_: strictly lower)
// so with T = (I + tril_(U B^T))^-1, from forward substitution,
//   P  = (T U) S + (T tril_(U K^T)) V
//   O  = R S + tril(R K^T) V - tril(R B^T) P
//   S' = e^{c_15} S + (e^{c_15} K)^T V - (e^{c_15} B)^T P
// delta_prep forms everything that does not need S, one workgroup per chunk
// and head; delta_scan walks a sequence's chunks with 16 value columns of S in
// each wave's registers; delta_out applies the head norm and the output gate.
// Missing tokens of a last chunk have u = k = r = 0 and no decay.
#include "mfma_util.h"
#include "mix_args.h"
#include "vec_io.h"

namespace {

constexpr int C = 16;                   // tokens per chunk
constexpr int SP = C + 4;               // row pitch of [.][16] arrays

// one chunk-head's record in the workspace, in floats: the image that the scan
// keeps in LDS, row pitches included
template <int DP> struct Rec {
  static constexpr int PP = DP + 4;               // pitch of [16][DP] arrays
  static constexpr int TU = 0;                    // [16][DP]
  static constexpr int R = TU + C * PP;           // [16][DP]
  static constexpr int KT = R + C * PP;           // [DP][16]
  static constexpr int BT = KT + DP * SP;         // [DP][16], negated
  static constexpr int TM = BT + DP * SP;         // [16][16]
  static constexpr int QK = TM + C * SP;          // [16][16]
  static constexpr int QB = QK + C * SP;          // [16][16], negated
  static constexpr int DC = QB + C * SP;          // [DP]
  static constexpr int SIZE = DC + DP;
};

template <typename T, int DP>
__global__ __launch_bounds__(256) void delta_prep_kernel(
    const DeltaArgs p, const int* __restrict__ tiles, float* __restrict__ ws) {
  typedef Rec<DP> W;
  constexpr int PP = W::PP;
  constexpr int GR = 256 / DP;          // token groups in the staging step
  constexpr int TPG = C / GR;           // tokens per group
  constexpr int NWV = (DP + 63) / 64;   // waves that share a token's channels
  __shared__ __attribute__((aligned(16))) float us[C * PP], rs[C * PP],
      ksh[C * PP], bs[C * PP];
  __shared__ __attribute__((aligned(16))) float ls[C * SP], ms[C * SP],
      ts[C * SP];
  __shared__ float csum[GR][DP], nrm[C][NWV == 1 ? 1 : NWV];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int tile = blockIdx.x, head = blockIdx.y;
  const int seq = tiles[tile * 2], t0 = tiles[tile * 2 + 1];
  const int row0 = p.cu[seq] + t0;
  const int n = min(C, p.cu[seq + 1] - row0);
  const int D = p.dim, HD = p.heads * D;
  float* rec = ws + ((size_t)tile * p.heads + head) * W::SIZE;

  // ---- channels x tokens: decay, unit keys, removal --------------------
  const int ch = tid % DP, grp = tid / DP;
  const bool live = ch < D;
  const int col = head * D + min(ch, D - 1);
  const float w0 = p.w0[col], ab = p.a_bias[col];
  float lw[TPG], kv[TPG], rv[TPG], av[TPG];
#pragma unroll
  for (int i = 0; i < TPG; ++i) {
    const int t = grp * TPG + i;
    const int row = row0 + min(t, n - 1);
    const T* pr = (const T*)p.proj + (size_t)row * p.proj_stride;
    const float z = to_f(((const T*)p.z)[(size_t)row * HD + col]);
    const float kk = to_f(pr[p.off_k + col]);
    const float rr = to_f(pr[p.off_r + col]);
    const float aa = to_f(pr[p.off_a + col]);
    const bool on = live && t < n;
    lw[i] = on ? -p.decay_scale * sigmoid_f(z + w0) : 0.f;
    kv[i] = on ? kk : 0.f;
    rv[i] = on ? rr : 0.f;
    av[i] = on ? sigmoid_f(aa + ab) : 0.f;
    // squared norm over channels: lanes of the same token
    float ss = kv[i] * kv[i];
#pragma unroll
    for (int off = (DP < 64 ? DP : 64) / 2; off >= 1; off >>= 1)
      ss += __shfl_xor(ss, off, 64);
    if ((ch & 63) == 0) nrm[t][ch >> 6] = ss;
    if (i) lw[i] += lw[i - 1];          // running within the group
  }
  csum[grp][ch] = lw[TPG - 1];
  __syncthreads();
  float base = 0.f, tot = 0.f;
#pragma unroll
  for (int g = 0; g < GR; ++g) {
    if (g < grp) base += csum[g][ch];
    tot += csum[g][ch];
  }
#pragma unroll
  for (int i = 0; i < TPG; ++i) {
    const int t = grp * TPG + i;
    float ss = 0.f;
#pragma unroll
    for (int w = 0; w < NWV; ++w) ss += nrm[t][w];
    const float u = kv[i] * rcp_f(sqrtf(ss + p.unit_eps));
    const float c1 = base + lw[i], c0 = i ? base + lw[i - 1] : base;
    const float e1 = __expf(-c1);
    us[t * PP + ch] = u * __expf(c0);
    rs[t * PP + ch] = rv[i] * __expf(c1);
    ksh[t * PP + ch] = kv[i] * e1;
    bs[t * PP + ch] = av[i] * u * e1;
  }
  if (grp == 0) rec[W::DC + ch] = __expf(tot);
  __syncthreads();

  // ---- the four token x token products, one per wave --------------------
  {
    const float* a = wave < 2 ? us : rs;
    const float* b = (wave & 1) ? ksh : bs;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f}, acc2 = acc;
#pragma unroll 4
    for (int d = 0; d < DP; d += 32) {
      float x[8], y[8];
      load_vec<4>(a + gl * PP + d + gs * 4, x);
      load_vec<4>(b + gl * PP + d + gs * 4, y);
      load_vec<4>(a + gl * PP + d + 16 + gs * 4, x + 4);
      load_vec<4>(b + gl * PP + d + 16 + gs * 4, y + 4);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        acc = mfma_f32_k4(x[r], y[r], acc);
        acc2 = mfma_f32_k4(x[4 + r], y[4 + r], acc2);
      }
    }
    acc += acc2;
    float* o = wave == 0 ? ls : wave == 1 ? ms
               : rec + (wave == 2 ? W::QB : W::QK);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = gs * 4 + r;                     // row; column gl
      const bool keep = wave < 2 ? gl < t : gl <= t;
      const float x = keep ? acc[r] : 0.f;
      o[t * SP + gl] = wave == 2 ? -x : x;
    }
  }
  __syncthreads();

  // ---- wave 0: T = (I + L)^-1, a lane per column; the others write out ----
  if (wave == 0) {
    if (lane < C) {
      float tc[C];
#pragma unroll
      for (int t = 0; t < C; ++t) {
        float x = t == lane ? 1.f : 0.f;
#pragma unroll
        for (int s = 0; s < t; ++s) x -= ls[t * SP + s] * tc[s];
        tc[t] = x;
        ts[t * SP + lane] = x;
      }
    }
  } else {
    for (int i = (tid - 64) * 4; i < C * DP; i += 192 * 4) {
      const int at = (i / DP) * PP + i % DP;
      *reinterpret_cast<f32x4*>(rec + W::R + at) =
          *reinterpret_cast<const f32x4*>(rs + at);
    }
    for (int i = tid - 64; i < DP * 4; i += 192) {
      const int d = i >> 2, t = (i & 3) * 4;        // 4 tokens of a channel
      float dc = 0.f;
#pragma unroll
      for (int g = 0; g < GR; ++g) dc += csum[g][d];
      dc = __expf(dc);
      f32x4 kx, bx;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        kx[r] = ksh[(t + r) * PP + d] * dc;
        bx[r] = -bs[(t + r) * PP + d] * dc;
      }
      *reinterpret_cast<f32x4*>(rec + W::KT + d * SP + t) = kx;
      *reinterpret_cast<f32x4*>(rec + W::BT + d * SP + t) = bx;
    }
  }
  __syncthreads();

  // ---- T U, 16 columns per wave and step; T tril_(U K^T) -----------------
  float tf[4];
  load_vec<4>(ts + gl * SP + gs * 4, tf);
  for (int d = wave * 16; d < DP; d += 64) {
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int r = 0; r < 4; ++r)
      acc = mfma_f32_k4(tf[r], us[(gs * 4 + r) * PP + d + gl], acc);
#pragma unroll
    for (int r = 0; r < 4; ++r)
      rec[W::TU + (gs * 4 + r) * PP + d + gl] = acc[r];
  }
  if (wave == 3) {
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int r = 0; r < 4; ++r)
      acc = mfma_f32_k4(tf[r], ms[(gs * 4 + r) * SP + gl], acc);
#pragma unroll
    for (int r = 0; r < 4; ++r)
      rec[W::TM + (gs * 4 + r) * SP + gl] = acc[r];
  }
}

// grid (heads, seqs, column groups).  A workgroup is NC column groups of 16
// value columns by KS parts of the key rows: wave (kp, cg) keeps its rows of
// its columns of S.  With KS = 2 the parts' shares of P and O meet in LDS.
// A record's loads fly under two chunks' MFMAs and land in the other half of
// LDS.
template <typename T, int DP, int KS, int NC>
__global__ __launch_bounds__(KS * NC * 64) void delta_scan_kernel(
    const DeltaArgs p, const int* __restrict__ chunk_cu,
    const float* __restrict__ ws, float* __restrict__ o) {
  typedef Rec<DP> W;
  constexpr int PP = W::PP, NT = KS * NC * 64, TT = DP / 16 / KS;
  constexpr int V4 = W::SIZE / 4, PER = (V4 + NT - 1) / NT;
  extern __shared__ __attribute__((aligned(16))) float smem[];
  f32x4* xch = reinterpret_cast<f32x4*>(smem + 2 * W::SIZE);  // [2][KS*NC*64]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int cg = wave % NC, kp = wave / NC;
  const int head = blockIdx.x, seq = blockIdx.y;
  const int D = p.dim, HD = p.heads * D;
  const int vcol = (blockIdx.z * NC + cg) * 16 + gl;
  const bool vlive = vcol < D;
  const int vc = min(vcol, D - 1);
  const int row0 = p.cu[seq], len = p.cu[seq + 1] - row0;
  const int ch0 = chunk_cu[seq], nch = chunk_cu[seq + 1] - ch0;
  const bool fresh = p.starts[seq] == 0;
  float* S = p.state + ((size_t)p.slots[seq] * p.heads + head) * D * D;
  const int k0 = kp * TT * 16;                  // this wave's key rows

  f32x4 s[TT];
#pragma unroll
  for (int t = 0; t < TT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int kr = k0 + t * 16 + gs * 4 + r;
      s[t][r] = !fresh && vlive && kr < D ? S[(size_t)kr * D + vcol] : 0.f;
    }

  f32x4 stage[2][PER];
  float v[4], vn[2][4];
#define DC_FETCH(c, h)                                                        \
  do {                                                                        \
    const f32x4* src = reinterpret_cast<const f32x4*>(                        \
        ws + ((size_t)(ch0 + (c)) * p.heads + head) * W::SIZE);               \
    _Pragma("unroll") for (int i = 0; i < PER; ++i)                           \
      stage[h][i] = src[min(tid + i * NT, V4 - 1)];                           \
    _Pragma("unroll") for (int r = 0; r < 4; ++r) {                           \
      const int t = (c) * C + gs * 4 + r;                                     \
      vn[h][r] = to_f(((const T*)p.proj)[                                     \
          (size_t)(row0 + min(t, len - 1)) * p.proj_stride + p.off_v +        \
          head * D + vc]);                                                    \
      if (t >= len || !vlive) vn[h][r] = 0.f;                                 \
    }                                                                         \
  } while (0)
#define DC_LAND(half)                                                         \
  do {                                                                        \
    f32x4* dst = reinterpret_cast<f32x4*>(smem + (half) * W::SIZE);           \
    _Pragma("unroll") for (int i = 0; i < PER; ++i)                           \
      if (tid + i * NT < V4) dst[tid + i * NT] = stage[half][i];              \
    _Pragma("unroll") for (int r = 0; r < 4; ++r) v[r] = vn[half][r];         \
  } while (0)
  DC_FETCH(0, 0);
  DC_LAND(0);
  DC_FETCH(min(1, nch - 1), 1);
  __syncthreads();
  for (int cc = 0; cc < nch; cc += 2)
#pragma unroll
  for (int h = 0; h < 2; ++h) {
    const int c = cc + h;
    if (c >= nch) break;
    const float* rec = smem + h * W::SIZE;
    // always: a skipped load would make the waits below drain every load
    DC_FETCH(min(c + 2, nch - 1), h);

    // P and O over the old state, two products side by side
    f32x4 pa = {0.f, 0.f, 0.f, 0.f}, oa = pa;
    if (kp == 0) {
      float x[4], y[4];
      load_vec<4>(rec + W::TM + gl * SP + gs * 4, x);
      load_vec<4>(rec + W::QK + gl * SP + gs * 4, y);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        pa = mfma_f32_k4(x[r], v[r], pa);
        oa = mfma_f32_k4(y[r], v[r], oa);
      }
    }
#pragma unroll
    for (int t = 0; t < TT; ++t) {
      float x[4], y[4];
      load_vec<4>(rec + W::TU + gl * PP + k0 + t * 16 + gs * 4, x);
      load_vec<4>(rec + W::R + gl * PP + k0 + t * 16 + gs * 4, y);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        pa = mfma_f32_k4(x[r], s[t][r], pa);
        oa = mfma_f32_k4(y[r], s[t][r], oa);
      }
    }
    if constexpr (KS == 2) {
      xch[wave * 64 + lane] = pa;
      if (kp == 1) xch[(KS * NC + cg) * 64 + lane] = oa;
    }
    // the decay and k v^T parts do not wait for P
#pragma unroll
    for (int t = 0; t < TT; ++t) {
      float x[4], d[4];
      load_vec<4>(rec + W::DC + k0 + t * 16 + gs * 4, d);
      load_vec<4>(rec + W::KT + (k0 + t * 16 + gl) * SP + gs * 4, x);
#pragma unroll
      for (int r = 0; r < 4; ++r) s[t][r] *= d[r];
#pragma unroll
      for (int r = 0; r < 4; ++r) s[t] = mfma_f32_k4(x[r], v[r], s[t]);
    }
    if constexpr (KS == 2) {
      __syncthreads();
      const f32x4 p0 = xch[cg * 64 + lane], p1 = xch[(NC + cg) * 64 + lane];
      pa = p0 + p1;
      if (kp == 0) oa += xch[(KS * NC + cg) * 64 + lane];
    }
#pragma unroll
    for (int t = 0; t < TT; ++t) {
      float y[4];
      load_vec<4>(rec + W::BT + (k0 + t * 16 + gl) * SP + gs * 4, y);
#pragma unroll
      for (int r = 0; r < 4; ++r) s[t] = mfma_f32_k4(y[r], pa[r], s[t]);
    }
    if (kp == 0) {
      float y[4];
      load_vec<4>(rec + W::QB + gl * SP + gs * 4, y);
#pragma unroll
      for (int r = 0; r < 4; ++r) oa = mfma_f32_k4(y[r], pa[r], oa);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = c * C + gs * 4 + r;
        if (t < len && vlive)
          o[(size_t)(row0 + t) * HD + head * D + vcol] = oa[r];
      }
    }
    DC_LAND(1 - h);
    __syncthreads();
  }
#undef DC_FETCH
#undef DC_LAND
#pragma unroll
  for (int t = 0; t < TT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int kr = k0 + t * 16 + gs * 4 + r;
      if (vlive && kr < D) S[(size_t)kr * D + vcol] = s[t][r];
    }
}

// out = o / rms(o) * norm_w * sigmoid(g).  VEC: dim is 4 * LPI for a power of
// two LPI, and LPI lanes take a row of a head; else one wave does.
template <typename T, int LPI>
__global__ __launch_bounds__(256) void delta_out_vec_kernel(
    const DeltaArgs p, const float* __restrict__ o, const long items) {
  const int lane = threadIdx.x & 63;
  const long item = (blockIdx.x * 4L + (threadIdx.x >> 6)) * (64 / LPI) +
                    lane / LPI;
  const int d = (lane % LPI) * 4;
  const long it = item < items ? item : items - 1;
  const int head = (int)(it % p.heads);
  const long row = it / p.heads;
  float x[4], w[4];
  load_vec<4>(o + it * (LPI * 4) + d, x);
  float ss = 0.f;
#pragma unroll
  for (int r = 0; r < 4; ++r) ss += x[r] * x[r];
#pragma unroll
  for (int off = LPI / 2; off >= 1; off >>= 1) ss += __shfl_xor(ss, off, 64);
  const float inv = 1.f / sqrtf(ss / (LPI * 4) + p.norm_eps);
  const int col = head * LPI * 4 + d;
  load_vec<4>(p.norm_w + col, w);
  if (item >= items) return;
  const T* g = (const T*)p.proj + row * p.proj_stride + p.off_g + col;
  T* out = (T*)p.out + row * p.out_stride + col;
  if constexpr (sizeof(T) == 2) {
    union { uint2 u; __hip_bfloat16 e[4]; } gv, ov;
    gv.u = *reinterpret_cast<const uint2*>(g);
#pragma unroll
    for (int r = 0; r < 4; ++r)
      ov.e[r] = f2bf(x[r] * inv * w[r] * sigmoid_f(bf2f(gv.e[r])));
    *reinterpret_cast<uint2*>(out) = ov.u;
  } else {
    float gv[4];
    load_vec<4>((const float*)g, gv);
#pragma unroll
    for (int r = 0; r < 4; ++r) gv[r] = x[r] * inv * w[r] * sigmoid_f(gv[r]);
    store_vec<4>((float*)out, gv);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void delta_out_kernel(
    const DeltaArgs p, const float* __restrict__ o, const long items) {
  const long item = blockIdx.x * 4L + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (item >= items) return;
  const int head = (int)(item % p.heads);
  const long row = item / p.heads;
  const int D = p.dim;
  const float* src = o + item * D;
  float ss = 0.f;
  for (int d = lane; d < D; d += 64) ss += src[d] * src[d];
  const float inv = 1.f / sqrtf(wave_sum(ss) / D + p.norm_eps);
  const T* g = (const T*)p.proj + row * p.proj_stride + p.off_g + head * D;
  T* out = (T*)p.out + row * p.out_stride + head * D;
  for (int d = lane; d < D; d += 64)
    out[d] = from_f<T>(src[d] * inv * p.norm_w[head * D + d] *
                       sigmoid_f(to_f(g[d])));
}

template <typename T, int DP, int KS, int NC>
void delta_chunk_t(const DeltaArgs& p, const int* tiles, const int* chunk_cu,
                   float* ws, float* o, int n_tiles, int seqs, long rows,
                   hipStream_t s) {
  constexpr int NT = KS * NC * 64;
  const int zs = (p.dim + NC * 16 - 1) / (NC * 16);
  const size_t lds = 2 * Rec<DP>::SIZE * sizeof(float) +
                     (KS == 2 ? (size_t)(KS + 1) * NC * 64 * 16 : 0);
  static bool once = false;
  if (!once) {
    (void)hipFuncSetAttribute((const void*)delta_scan_kernel<T, DP, KS, NC>,
                              hipFuncAttributeMaxDynamicSharedMemorySize,
                              (int)lds);
    once = true;
  }
  delta_prep_kernel<T, DP><<<dim3(n_tiles, p.heads), 256, 0, s>>>(p, tiles,
                                                                  ws);
  delta_scan_kernel<T, DP, KS, NC><<<dim3(p.heads, seqs, zs), NT, lds, s>>>(
      p, chunk_cu, ws, o);
  const long items = rows * p.heads;
  const bool vec = p.dim == DP && p.proj_stride % 4 == 0 &&
                   p.out_stride % 4 == 0 && p.off_g % 4 == 0 &&
                   ((uintptr_t)p.proj & 15) == 0 &&
                   ((uintptr_t)p.out & 15) == 0;
  if (vec) {
    const long per = 4L * (64 / (DP / 4));
    delta_out_vec_kernel<T, DP / 4>
        <<<(int)((items + per - 1) / per), 256, 0, s>>>(p, o, items);
  } else {
    delta_out_kernel<T><<<(int)((items + 3) / 4), 256, 0, s>>>(p, o, items);
  }
}

template <typename T>
void delta_chunk_d(const DeltaArgs& p, const int* tiles, const int* chunk_cu,
                   float* ws, float* o, int n_tiles, int seqs, long rows,
                   hipStream_t s) {
  if (p.dim <= 32) {
    delta_chunk_t<T, 32, 1, 2>(p, tiles, chunk_cu, ws, o, n_tiles, seqs, rows, s);
  } else if (p.dim <= 64) {
    delta_chunk_t<T, 64, 2, 2>(p, tiles, chunk_cu, ws, o, n_tiles, seqs, rows, s);
  } else {
    delta_chunk_t<T, 128, 2, 4>(p, tiles, chunk_cu, ws, o, n_tiles, seqs, rows, s);
  }
}

}  // namespace

extern "C" {

int delta_chunk_tokens() { return C; }

// floats of workspace per chunk and head
long delta_chunk_record(int dim) {
  return dim <= 32 ? Rec<32>::SIZE : dim <= 64 ? Rec<64>::SIZE
                                               : Rec<128>::SIZE;
}

void launch_delta_chunk(const DeltaArgs* p, const int* tiles,
                        const int* chunk_cu, float* ws, float* o, int n_tiles,
                        int seqs, long rows, int f32, hipStream_t s) {
  if (f32) {
    delta_chunk_d<float>(*p, tiles, chunk_cu, ws, o, n_tiles, seqs, rows, s);
  } else {
    delta_chunk_d<__hip_bfloat16>(*p, tiles, chunk_cu, ws, o, n_tiles, seqs,
                                  rows, s);
  }
}

}  // extern "C"
