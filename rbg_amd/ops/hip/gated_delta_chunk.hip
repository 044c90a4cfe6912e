// Gated delta rule over prompts, 16 tokens at a time (gfx950), in f32 on the
// matrix cores; q, k and v come convolved.
//
// Write c_t for the chunk's cumulative log decay (per key channel, or one for
// the head), S for the state before the chunk, and
//   A_ts = sum_d k_t k_s e^{c_t - c_s}     Q_ts = sum_d q_t k_s e^{c_t - c_s}
//   T = (I + diag(beta) tril_(A))^-1 diag(beta)          (tril_: strictly lower)
// Then U = T (V - (k e^c) S) holds the tokens' updates, and with P = -U
//   P  = (T k e^c) S - T V
//   O  = (q e^c) S - tril(Q) P
//   S' = e^{c_15} S - (k e^{c_15 - c})^T P
// which is what delta_scan.h walks.  Every exponent there is at most zero; only
// A and Q have factors of both signs when the matrix cores form them, e^{c_t -
// c_7} and e^{c_7 - c_s}.  A chunk whose decays span more than RANGE forms A and
// Q from running products instead, so that any decay keeps its precision.  One
// decay per head factors out of A and Q altogether.  Sums of log decays are taken
// over the tokens they span, never as differences of longer ones.
// Missing tokens of a last chunk have q = k = beta = 0 and no decay.
#include "delta_scan.h"
#include "gated_delta.h"

namespace {

constexpr float RANGE = 30.f;

template <typename T, int DP, bool CHANNEL>
__global__ __launch_bounds__(256) void gated_prep_kernel(
    const GatedDeltaArgs p, const int* __restrict__ tiles,
    float* __restrict__ ws) {
  typedef Rec<DP, false> W;
  constexpr int PP = W::PP;
  constexpr int GR = 256 / DP;          // token groups in the staging step
  constexpr int TPG = C / GR;           // tokens per group
  constexpr int NWV = (DP + 63) / 64;   // waves that share a token's channels
  // CHANNEL: kx = k e^{c_t - c_7}, qx = q e^{c_t - c_7}, ky = k e^{c_7 - c_t};
  // in a wide chunk k, q and the decay factors.  Else kx = k, qx = q.
  __shared__ __attribute__((aligned(16))) float kx[C * PP], qx[C * PP],
      ky[CHANNEL ? C * PP : 4];
  __shared__ __attribute__((aligned(16))) float ls[C * SP], ts[C * SP];
  __shared__ float fs[CHANNEL ? 1 : C * SP];    // e^{c_t - c_s} of the head
  __shared__ f32x4 half[2][64];
  __shared__ float csum[GR][DP], nk[C][NWV], nq[C][NWV], bs[C], lws[C];
  __shared__ float mid[DP];                     // e^{c_7}
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int tile = blockIdx.x, head = blockIdx.y;
  const int kvh = head / (p.heads / p.kv_heads);
  const int seq = tiles[tile * 2], t0 = tiles[tile * 2 + 1];
  const int row0 = p.cu[seq] + t0;
  const int n = min(C, p.cu[seq + 1] - row0);
  const int D = p.dim;
  float* rec = ws + ((size_t)tile * p.heads + head) * W::SIZE;

  // ---- channels x tokens: unit vectors and decays -------------------------
  const int ch = tid % DP, grp = tid / DP;
  const bool live = ch < D;
  const int cc = min(ch, D - 1);
  const float rate = expf(p.a_log[head]);
  const float bias = p.dt_bias[CHANNEL ? head * D + cc : head];
  float lw[TPG], kv[TPG], qv[TPG], sum = 0.f;
#pragma unroll
  for (int i = 0; i < TPG; ++i) {
    const int t = grp * TPG + i;
    const size_t row = row0 + min(t, n - 1);
    const T* y = (const T*)p.qkv + row * p.qkv_row + kvh * D + cc;
    const float z = to_f(((const T*)p.decay)[
        row * p.decay_row + (CHANNEL ? head * D + cc : head)]);
    const float a = to_f(y[p.off_k]), b = to_f(y[p.off_q]);
    lw[i] = t < n && (live || !CHANNEL) ? log_decay(z, bias, rate) : 0.f;
    kv[i] = live && t < n ? a : 0.f;
    qv[i] = live && t < n ? b : 0.f;
    // squared norms over channels: lanes of the same token
    float sk = kv[i] * kv[i], sq = qv[i] * qv[i];
#pragma unroll
    for (int off = (DP < 64 ? DP : 64) / 2; off >= 1; off >>= 1) {
      sk += __shfl_xor(sk, off, 64);
      sq += __shfl_xor(sq, off, 64);
    }
    if ((ch & 63) == 0) {
      nk[t][ch >> 6] = sk;
      nq[t][ch >> 6] = sq;
    }
    if (ch == 0) lws[t] = lw[i];
    sum += lw[i];
  }
  csum[grp][ch] = sum;
  if (tid < C)
    bs[tid] = tid < n ? sigmoid_f(to_f(((const T*)p.beta)[
        (size_t)(row0 + tid) * p.beta_row + head])) : 0.f;
  __syncthreads();
  float before = 0.f, after = 0.f, c7 = 0.f, tot = 0.f;
#pragma unroll
  for (int g = 0; g < GR; ++g) {
    if (g < grp) before += csum[g][ch];
    if (g > grp) after += csum[g][ch];
    if (g < GR / 2) c7 += csum[g][ch];
    tot += csum[g][ch];
  }
  bool wide = false;
  if (CHANNEL) wide = __syncthreads_or(tot < -RANGE);
  float bt[TPG];
#pragma unroll
  for (int i = TPG - 1; i >= 0; --i) {          // sums of what comes after
    bt[i] = __expf(after);
    after += lw[i];
  }
#pragma unroll
  for (int i = 0; i < TPG; ++i) {
    const int t = grp * TPG + i, at = t * PP + ch;
    float sk = 0.f, sq = 0.f;
#pragma unroll
    for (int w = 0; w < NWV; ++w) {
      sk += nk[t][w];
      sq += nq[t][w];
    }
    const float k = kv[i] / sqrtf(sk + p.unit_eps);
    const float q = qv[i] * (p.q_scale / sqrtf(sq + p.unit_eps));
    before += lw[i];                            // now c_t
    rec[W::R + at] = q * __expf(before);
    bt[i] *= -k;
    if (CHANNEL) {
      const float e = wide ? 1.f : __expf(before - c7);
      kx[at] = k * e;
      qx[at] = q * e;
      ky[at] = wide ? __expf(lw[i]) : k * __expf(c7 - before);
    } else {
      kx[at] = k;
      qx[at] = q;
    }
  }
  store_vec<TPG>(rec + W::BT + ch * SP + grp * TPG, bt);
  if (grp == 0) {
    rec[W::DC + ch] = __expf(tot);
    mid[ch] = wide ? 1.f : __expf(c7);
  }
  if (!CHANNEL) {
    const int t = tid >> 4, s = tid & 15;
    float x = 0.f;
    for (int j = s + 1; j <= t; ++j) x += lws[j];
    fs[t * SP + s] = s <= t ? __expf(x) : 0.f;
  }
  __syncthreads();

  // ---- A and Q: beta_t A_ts into ls, -Q_ts into the record ------------------
  auto put_a = [&](int t, int s, float x) {
    ls[t * SP + s] = s < t ? bs[t] * x : 0.f;
  };
  auto put_q = [&](int t, int s, float x) {
    rec[W::QB + t * SP + s] = s <= t ? -x : 0.f;
  };
  if (CHANNEL && wide) {
    // a thread follows one s through its share of the channels
    const int s = tid >> 4, part = tid & 15;
    float a[C], q[C];
#pragma unroll
    for (int t = 0; t < C; ++t) a[t] = q[t] = 0.f;
    for (int d = part; d < DP; d += 16) {
      float f = kx[s * PP + d];
#pragma unroll
      for (int t = 0; t < C; ++t) {
        if (t < s) continue;
        if (t > s) f *= ky[t * PP + d];
        a[t] += f * kx[t * PP + d];
        q[t] += f * qx[t * PP + d];
      }
    }
#pragma unroll
    for (int t = 0; t < C; ++t) {
      const float x = group16_sum(a[t]), y = group16_sum(q[t]);
      if (part == t) {
        put_a(t, s, x);
        put_q(t, s, y);
      }
    }
    __syncthreads();
    if (tid < DP) {                             // kx = k e^{c_t}
      float f = 1.f;
      for (int t = 0; t < C; ++t) {
        f *= ky[t * PP + tid];
        kx[t * PP + tid] *= f;
      }
    }
  } else {
    // waves 0, 1: A and Q over the first half of the channels; 2, 3: the other
    const bool is_q = wave & 1;
    const int d0 = (wave >> 1) * (DP / 2);
    const float* a = is_q ? qx : kx;
    const float* b = CHANNEL ? ky : kx;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int d = d0; d < d0 + DP / 2; d += 16) {
      float x[4], y[4];
      load_vec<4>(a + gl * PP + d + gs * 4, x);
      load_vec<4>(b + gl * PP + d + gs * 4, y);
#pragma unroll
      for (int r = 0; r < 4; ++r) acc = mfma_f32_k4(x[r], y[r], acc);
    }
    if (wave >= 2) half[wave - 2][lane] = acc;
    __syncthreads();
    if (wave < 2) {
      acc += half[wave][lane];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = gs * 4 + r;
        const float x = CHANNEL ? acc[r] : acc[r] * fs[t * SP + gl];
        if (is_q) put_q(t, gl, x);
        else put_a(t, gl, x);
      }
    }
  }
  __syncthreads();

  // ---- T, a lane per column -------------------------------------------------
  if (wave == 0 && lane < C) {
    float tc[C], c = 0.f;
    const float b = bs[lane];
    if (!CHANNEL)
      for (int j = 0; j <= lane; ++j) c += lws[j];
    const float e = CHANNEL ? 1.f : __expf(c);
#pragma unroll
    for (int t = 0; t < C; ++t) {
      float x = t == lane ? 1.f : 0.f;
#pragma unroll
      for (int s = 0; s < t; ++s) x -= ls[t * SP + s] * tc[s];
      tc[t] = x;
      ts[t * SP + lane] = x * b * e;            // times k e^c below
      rec[W::TM + t * SP + lane] = -x * b;
    }
  }
  __syncthreads();

  // ---- T (k e^c), 16 columns per wave and step -----------------------------
  float tf[4];
  load_vec<4>(ts + gl * SP + gs * 4, tf);
  for (int d = wave * 16; d < DP; d += 64) {
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int r = 0; r < 4; ++r)
      acc = mfma_f32_k4(tf[r], kx[(gs * 4 + r) * PP + d + gl], acc);
    const float m = CHANNEL ? mid[d + gl] : 1.f;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      rec[W::TU + (gs * 4 + r) * PP + d + gl] = acc[r] * m;
  }
}

template <typename T, int DP, int KS, int NC>
void gated_chunk_t(const GatedDeltaArgs& p, const int* tiles,
                   const int* chunk_cu, float* ws, float* o, int n_tiles,
                   int seqs, long rows, hipStream_t s) {
  const dim3 grid(n_tiles, p.heads);
  if (p.per_channel) {
    gated_prep_kernel<T, DP, true><<<grid, 256, 0, s>>>(p, tiles, ws);
  } else {
    gated_prep_kernel<T, DP, false><<<grid, 256, 0, s>>>(p, tiles, ws);
  }
  DeltaScanArgs sa{};
  sa.v = (const T*)p.qkv + p.off_v;
  sa.state = p.state; sa.slots = p.slots; sa.cu = p.cu; sa.starts = p.starts;
  sa.chunk_cu = chunk_cu; sa.ws = ws; sa.o = o;
  sa.v_row = p.qkv_row;
  sa.heads = p.heads; sa.dk = p.dim; sa.dv = p.vdim;
  delta_scan<T, DP, KS, NC, false>(sa, seqs, s);
  DeltaOutArgs oa{};
  oa.o = o; oa.gate = p.gate; oa.norm_w = p.norm_w; oa.out = p.out;
  oa.g_row = p.gate_row; oa.o_row = p.out_row;
  oa.heads = p.heads; oa.dv = p.vdim; oa.w_head = 0;
  oa.silu = p.silu; oa.eps = p.norm_eps;
  delta_out<T>(oa, rows, s);
}

template <typename T>
void gated_chunk_d(const GatedDeltaArgs& p, const int* tiles,
                   const int* chunk_cu, float* ws, float* o, int n_tiles,
                   int seqs, long rows, hipStream_t s) {
#define GC_GO(DP, KS, NC)                                                     \
  gated_chunk_t<T, DP, KS, NC>(p, tiles, chunk_cu, ws, o, n_tiles, seqs,      \
                               rows, s)
  if (p.dim <= 32) GC_GO(32, 1, 2);
  else if (p.dim <= 64) GC_GO(64, 2, 2);
  else GC_GO(128, 2, 4);
#undef GC_GO
}

}  // namespace

extern "C" {

int gated_chunk_tokens() { return C; }
int gated_chunk_max_dim() { return 128; }

// floats of workspace per chunk and head
long gated_chunk_record(int dim) {
  return dim <= 32 ? Rec<32, false>::SIZE
       : dim <= 64 ? Rec<64, false>::SIZE : Rec<128, false>::SIZE;
}

void launch_gated_chunk(const GatedDeltaArgs* p, const int* tiles,
                        const int* chunk_cu, float* ws, float* o, int n_tiles,
                        int seqs, long rows, int f32, hipStream_t s) {
  if (f32) {
    gated_chunk_d<float>(*p, tiles, chunk_cu, ws, o, n_tiles, seqs, rows, s);
  } else {
    gated_chunk_d<__hip_bfloat16>(*p, tiles, chunk_cu, ws, o, n_tiles, seqs,
                                  rows, s);
  }
}

}  // extern "C"
