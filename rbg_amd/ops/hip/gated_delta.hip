// Gated delta rule (gfx950), token by token: decode steps and head sizes that
// the chunked form does not take.
//
// Per head and token, q and k unit vectors (q also times q_scale):
//   S <- g S            g per head, or per key channel (rows of S)
//   u = beta (v - S^T k)      S <- S + k u^T      o = S^T q
//   out = o / rms(o) * norm_w * gate
// with S [dim, vdim] in f32 in the sequence's state slot; several value heads may
// share a query/key head.  In a decode step the short convolution of q, k and v,
// with its ring of past inputs, is part of the kernel.
//
// One workgroup holds a head's whole state in registers: a thread owns four
// value columns of every RP-th key row.  Both products with the state are taken
// before the update, as S_new^T q = (g S)^T q + (k.q) u, so the key rows are
// reduced once.
#include "gated_delta.h"

namespace {

template <typename T, int DK, int DV, int NT>
__global__ __launch_bounds__(NT) void gated_step_kernel(
    const GatedDeltaArgs p) {
  constexpr int CG = DV / 4;              // column groups of 4
  constexpr int RP = NT / CG;             // key rows per pass
  constexpr int IT = DK / RP;             // passes = rows per thread
  constexpr int NWV = NT / 64;
  static_assert(IT * RP == DK && RP * CG == NT, "shape");
  __shared__ float q_s[DK], k_s[DK], g_s[DK], v_s[DV];
  __shared__ float red[NWV][2][DV];

  const int head = blockIdx.x, seq = blockIdx.y;
  const int ratio = p.heads / p.kv_heads, kvh = head / ratio;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int cg = tid % CG, rg = tid / CG;
  const int D = p.dim, E = p.vdim;
  const int row0 = p.cu ? p.cu[seq] : seq;
  const int len = p.cu ? p.cu[seq + 1] - row0 : 1;
  const int start = p.starts[seq], slot = p.slots[seq];
  float* S = p.state + ((size_t)slot * p.heads + head) * D * E;
  const bool vec = (E & 3) == 0;
  const float rate = expf(p.a_log[head]);

  float s[IT][4];
#pragma unroll
  for (int it = 0; it < IT; ++it) {
    const int kr = it * RP + rg, c = cg * 4;
#pragma unroll
    for (int j = 0; j < 4; ++j) s[it][j] = 0.f;
    if (start > 0 && kr < D) {
      if (vec) {
        if (c < E) load_vec<4>(S + (size_t)kr * E + c, s[it]);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c + j < E) s[it][j] = S[(size_t)kr * E + c + j];
      }
    }
  }

  for (int t = 0; t < len; ++t) {
    const size_t row = row0 + t;
    const T* y = (const T*)p.qkv + row * p.qkv_row;
    // q, k, v side by side: DK, DK and DV places
    for (int i = tid; i < 2 * DK + DV; i += NT) {
      const int part = i < DK ? 0 : i < 2 * DK ? 1 : 2;
      const int c = i - part * DK;
      const bool live = part < 2 ? c < D : c < E;
      const int col = part == 0 ? p.off_q + kvh * D + c
                    : part == 1 ? p.off_k + kvh * D + c
                                : p.off_v + head * E + c;
      float x = 0.f;
      if (live) {
        x = to_f(y[col]);
        if (p.conv_w != nullptr) {
          const int ch = col - p.off_q, pos = start;
          T* ring = (T*)p.ring + (size_t)slot * p.taps * p.channels + ch;
          const float* w = p.conv_w + ch;
          float a = w[(size_t)(p.taps - 1) * p.channels] * x;
          for (int j = 1; j < p.taps; ++j)
            if (pos >= j)
              a += w[(size_t)(p.taps - 1 - j) * p.channels] *
                   to_f(ring[(size_t)((pos - j) % p.taps) * p.channels]);
          if (p.taps > 1 && (part == 2 || head % ratio == 0))
            ring[(size_t)(pos % p.taps) * p.channels] = y[col];
          x = a * sigmoid_f(a);
        }
      }
      if (part == 0) q_s[c] = x;
      else if (part == 1) k_s[c] = x;
      else v_s[c] = x;
    }
    if (p.per_channel) {
      const T* z = (const T*)p.decay + row * p.decay_row + head * D;
      for (int i = tid; i < DK; i += NT)
        g_s[i] = i < D ? __expf(log_decay(to_f(z[i]), p.dt_bias[head * D + i],
                                          rate)) : 0.f;
    } else {
      const float g = __expf(log_decay(
          to_f(((const T*)p.decay)[row * p.decay_row + head]),
          p.dt_bias[head], rate));
      for (int i = tid; i < DK; i += NT) g_s[i] = g;
    }
    const float beta =
        sigmoid_f(to_f(((const T*)p.beta)[row * p.beta_row + head]));
    __syncthreads();
    float kk = 0.f, qq = 0.f, kq = 0.f;
#pragma unroll
    for (int i = 0; i < DK / 64; ++i) {
      const float a = k_s[i * 64 + lane], b = q_s[i * 64 + lane];
      kk += a * a;
      qq += b * b;
      kq += a * b;
    }
    const float ki = 1.f / sqrtf(wave_sum(kk) + p.unit_eps);
    const float qi = p.q_scale / sqrtf(wave_sum(qq) + p.unit_eps);
    kq = wave_sum(kq) * ki * qi;

    float pk[4] = {0.f, 0.f, 0.f, 0.f}, pq[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int kr = it * RP + rg;
      const float g = g_s[kr], a = k_s[kr], b = q_s[kr];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        s[it][j] *= g;
        pk[j] += a * s[it][j];
        pq[j] += b * s[it][j];
      }
    }
#pragma unroll
    for (int off = CG; off < 64; off <<= 1)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        pk[j] += __shfl_xor(pk[j], off, 64);
        pq[j] += __shfl_xor(pq[j], off, 64);
      }
    if (lane < CG || CG >= 64) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        red[wave][0][cg * 4 + j] = pk[j];
        red[wave][1][cg * 4 + j] = pq[j];
      }
    }
    __syncthreads();
    float u[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      float a = 0.f;
#pragma unroll
      for (int w = 0; w < NWV; ++w) a += red[w][0][cg * 4 + j];
      u[j] = beta * (v_s[cg * 4 + j] - a * ki) * ki;
    }
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const float a = k_s[it * RP + rg];
#pragma unroll
      for (int j = 0; j < 4; ++j) s[it][j] += a * u[j];
    }
    if (wave == NWV - 1) {
      constexpr int OC = (DV + 63) / 64;
      float o[OC], ss = 0.f;
#pragma unroll
      for (int i = 0; i < OC; ++i) {
        const int c = i * 64 + lane;
        o[i] = 0.f;
        if (c >= E) continue;
        float a = 0.f, b = 0.f;
#pragma unroll
        for (int w = 0; w < NWV; ++w) {
          a += red[w][0][c];
          b += red[w][1][c];
        }
        o[i] = b * qi + kq * beta * (v_s[c] - a * ki);
        ss += o[i] * o[i];
      }
      const float inv = 1.f / sqrtf(wave_sum(ss) / E + p.norm_eps);
      const T* gate = (const T*)p.gate + row * p.gate_row + head * E;
      T* out = (T*)p.out + row * p.out_row + head * E;
#pragma unroll
      for (int i = 0; i < OC; ++i) {
        const int c = i * 64 + lane;
        if (c >= E) continue;
        const float z = to_f(gate[c]), sg = sigmoid_f(z);
        out[c] = from_f<T>(o[i] * inv * p.norm_w[c] * (p.silu ? z * sg : sg));
      }
    }
    if (t + 1 < len) __syncthreads();     // the vectors are read
  }

#pragma unroll
  for (int it = 0; it < IT; ++it) {
    const int kr = it * RP + rg, c = cg * 4;
    if (kr < D) {
      if (vec) {
        if (c < E) store_vec<4>(S + (size_t)kr * E + c, s[it]);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c + j < E) S[(size_t)kr * E + c + j] = s[it][j];
      }
    }
  }
}

template <typename T>
void gated_step_t(const GatedDeltaArgs& p, int seqs, hipStream_t s) {
  const dim3 grid(p.heads, seqs);
#define GS_GO(DK, DV, NT)                                                     \
  gated_step_kernel<T, DK, DV, NT><<<grid, NT, 0, s>>>(p)
  if (p.dim <= 64) {
    if (p.vdim <= 32) GS_GO(64, 32, 64);
    else if (p.vdim <= 64) GS_GO(64, 64, 256);
    else if (p.vdim <= 128) GS_GO(64, 128, 256);
    else GS_GO(64, 256, 256);
  } else if (p.dim <= 128) {
    if (p.vdim <= 32) GS_GO(128, 32, 128);
    else if (p.vdim <= 64) GS_GO(128, 64, 256);
    // few heads: more threads shorten each one's walk
    else if (p.vdim <= 128 && p.heads * seqs <= 512) GS_GO(128, 128, 512);
    else if (p.vdim <= 128) GS_GO(128, 128, 256);
    else GS_GO(128, 256, 512);
  } else {
    if (p.vdim <= 32) GS_GO(256, 32, 256);
    else if (p.vdim <= 64) GS_GO(256, 64, 256);
    else if (p.vdim <= 128) GS_GO(256, 128, 512);
    else GS_GO(256, 256, 1024);
  }
#undef GS_GO
}

}  // namespace

extern "C" void launch_gated_step(const GatedDeltaArgs* p, int seqs, int f32,
                                  hipStream_t s) {
  if (f32) gated_step_t<float>(*p, seqs, s);
  else gated_step_t<__hip_bfloat16>(*p, seqs, s);
}
