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
// and head; delta_scan.h walks the chunks and applies the head norm and gate.
// Missing tokens of a last chunk have u = k = r = 0 and no decay.
#include "delta_scan.h"
#include "mix_args.h"

namespace {

template <typename T, int DP>
__global__ __launch_bounds__(256) void delta_prep_kernel(
    const DeltaArgs p, const int* __restrict__ tiles, float* __restrict__ ws) {
  typedef Rec<DP, true> W;
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

template <typename T, int DP, int KS, int NC>
void delta_chunk_t(const DeltaArgs& p, const int* tiles, const int* chunk_cu,
                   float* ws, float* o, int n_tiles, int seqs, long rows,
                   hipStream_t s) {
  delta_prep_kernel<T, DP><<<dim3(n_tiles, p.heads), 256, 0, s>>>(p, tiles,
                                                                  ws);
  DeltaScanArgs sa{};
  sa.v = (const T*)p.proj + p.off_v;
  sa.state = p.state; sa.slots = p.slots; sa.cu = p.cu; sa.starts = p.starts;
  sa.chunk_cu = chunk_cu; sa.ws = ws; sa.o = o;
  sa.v_row = p.proj_stride;
  sa.heads = p.heads; sa.dk = sa.dv = p.dim;
  delta_scan<T, DP, KS, NC, true>(sa, seqs, s);
  DeltaOutArgs oa{};
  oa.o = o; oa.gate = (const T*)p.proj + p.off_g; oa.norm_w = p.norm_w;
  oa.out = p.out;
  oa.g_row = p.proj_stride; oa.o_row = p.out_stride;
  oa.heads = p.heads; oa.dv = oa.w_head = p.dim;
  oa.eps = p.norm_eps;
  delta_out<T>(oa, rows, s);
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
  return dim <= 32 ? Rec<32, true>::SIZE
       : dim <= 64 ? Rec<64, true>::SIZE : Rec<128, true>::SIZE;
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
