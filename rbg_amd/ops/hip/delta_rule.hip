// Generalized delta rule with per-channel decay (gfx950), token by token.
//
// Per head and token, with the unit key u = k / sqrt(sum k^2 + unit_eps):
//   w = exp(-decay_scale * sigmoid(z + w0))      a = sigmoid(a_in + a_bias)
//   S <- diag(w) S - (a*u)(u^T S) + k v^T        o = S^T r
//   out = o / rms(o) * norm_w * sigmoid(g)
// with S [dim, dim] (key rows, value columns) in f32 in the sequence's state
// slot.  z is either read, or formed here as W2 tanh(low) so that a decode
// step needs no further launch.
//
// One workgroup holds a head's whole state in registers: a thread owns four
// value columns of every RP-th key row.  The two products with S reduce over
// key rows by wave shuffles, then over waves through LDS.  A decode step is one
// read and one write of the state, which is its traffic; the same kernel walks
// several tokens for short portions.
#include "mix_args.h"
#include "vec_io.h"

namespace {

// MINW: waves per SIMD the registers must allow (the loads of one workgroup
// hide behind the others' work)
template <typename T, int DP, int NT, int MINW>
__global__ __launch_bounds__(NT, MINW) void delta_step_kernel(const DeltaArgs p) {
  constexpr int CG = DP / 4;              // column groups of 4
  constexpr int RP = NT / CG;             // key rows per pass
  constexpr int IT = DP / RP;             // passes = rows per thread
  constexpr int NWV = NT / 64;
  constexpr int DW = (DP + 63) / 64;      // waves that stage channels
  extern __shared__ float low_s[];        // [rank]
  __shared__ float w_s[DP], b_s[DP], u_s[DP], k_s[DP], r_s[DP], v_s[DP];
  __shared__ float red[NWV][DP], red2[NWV][DP], part[2][DW];

  const int head = blockIdx.x, seq = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int cg = tid % CG, rg = tid / CG;
  const int D = p.dim, HD = p.heads * D;
  const int row0 = p.cu ? p.cu[seq] : seq;
  const int len = p.cu ? p.cu[seq + 1] - row0 : 1;
  const bool fresh = p.starts[seq] == 0;
  float* S = p.state + ((size_t)p.slots[seq] * p.heads + head) * D * D;
  const bool vec = (D & 3) == 0;

  float s[IT][4];
#pragma unroll
  for (int it = 0; it < IT; ++it) {
    const int kr = it * RP + rg, c = cg * 4;
#pragma unroll
    for (int j = 0; j < 4; ++j) s[it][j] = 0.f;
    if (!fresh && kr < D) {
      if (vec) {
        if (c < D) load_vec<4>(S + (size_t)kr * D + c, s[it]);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c + j < D) s[it][j] = S[(size_t)kr * D + c + j];
      }
    }
  }

  const bool staging = wave < DW;         // whole waves: they reduce
  const bool live = tid < D;
  const int ch = head * D + tid;
  float w0 = 0.f, ab = 0.f, nw = 0.f;
  if (live) { w0 = p.w0[ch]; ab = p.a_bias[ch]; nw = p.norm_w[ch]; }

  for (int t = 0; t < len; ++t) {
    const T* pr = (const T*)p.proj + (size_t)(row0 + t) * p.proj_stride;
    float kk = 0.f, av = 0.f, zz = 0.f, gate = 0.f;
    if (p.z == nullptr) {
      for (int j = tid; j < p.rank; j += NT)
        low_s[j] = round_to<T>(tanhf(to_f(pr[p.off_low + j])));
      __syncthreads();
    }
    if (staging) {
      if (live) {
        kk = to_f(pr[p.off_k + ch]);
        r_s[tid] = to_f(pr[p.off_r + ch]);
        v_s[tid] = to_f(pr[p.off_v + ch]);
        gate = sigmoid_f(to_f(pr[p.off_g + ch]));
        av = sigmoid_f(to_f(pr[p.off_a + ch]) + ab);
        if (p.z != nullptr) {
          zz = to_f(((const T*)p.z)[(size_t)(row0 + t) * HD + ch]);
        } else {
          const T* w2 = (const T*)p.w2 + (size_t)ch * p.rank;
          if ((p.rank & 7) == 0) {
#pragma unroll 2
            for (int j = 0; j < p.rank; j += 8) {
              float wv[8];
              load_vec<8>(w2 + j, wv);
#pragma unroll
              for (int e = 0; e < 8; ++e) zz += wv[e] * low_s[j + e];
            }
          } else {
#pragma unroll 2
            for (int j = 0; j < p.rank; ++j) zz += to_f(w2[j]) * low_s[j];
          }
        }
        w_s[tid] = expf(-p.decay_scale * sigmoid_f(zz + w0));
      } else if (tid < DP) {
        r_s[tid] = v_s[tid] = w_s[tid] = 0.f;
      }
      if (tid < DP) k_s[tid] = kk;
      const float ss = wave_sum(kk * kk);
      if (lane == 0) part[0][wave] = ss;
    }
    __syncthreads();
    if (staging) {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < DW; ++i) ss += part[0][i];
      const float u = kk / sqrtf(ss + p.unit_eps);
      if (tid < DP) {
        u_s[tid] = u;
        b_s[tid] = av * u;
      }
    }
    __syncthreads();

    // q = u^T S over the old state
    float q[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const float u = u_s[it * RP + rg];
#pragma unroll
      for (int j = 0; j < 4; ++j) q[j] += u * s[it][j];
    }
#pragma unroll
    for (int off = CG; off < 64; off <<= 1)
#pragma unroll
      for (int j = 0; j < 4; ++j) q[j] += __shfl_xor(q[j], off, 64);
    if (lane < CG || CG >= 64) {
#pragma unroll
      for (int j = 0; j < 4; ++j) red[wave][cg * 4 + j] = q[j];
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      q[j] = 0.f;
#pragma unroll
      for (int i = 0; i < NWV; ++i) q[j] += red[i][cg * 4 + j];
    }
    float o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int it = 0; it < IT; ++it) {
      const int kr = it * RP + rg;
      const float wv = w_s[kr], b = b_s[kr], kv = k_s[kr], r = r_s[kr];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        s[it][j] = wv * s[it][j] - b * q[j] + kv * v_s[cg * 4 + j];
        o[j] += r * s[it][j];
      }
    }
#pragma unroll
    for (int off = CG; off < 64; off <<= 1)
#pragma unroll
      for (int j = 0; j < 4; ++j) o[j] += __shfl_xor(o[j], off, 64);
    if (lane < CG || CG >= 64) {
#pragma unroll
      for (int j = 0; j < 4; ++j) red2[wave][cg * 4 + j] = o[j];
    }
    __syncthreads();
    float ov = 0.f;
    if (staging) {
      if (tid < DP) {
#pragma unroll
        for (int i = 0; i < NWV; ++i) ov += red2[i][tid];
      }
      const float ss = wave_sum(ov * ov);
      if (lane == 0) part[1][wave] = ss;
    }
    __syncthreads();
    if (live) {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < DW; ++i) ss += part[1][i];
      ov = ov / sqrtf(ss / D + p.norm_eps) * nw * gate;
      ((T*)p.out)[(size_t)(row0 + t) * p.out_stride + ch] = from_f<T>(ov);
    }
  }

#pragma unroll
  for (int it = 0; it < IT; ++it) {
    const int kr = it * RP + rg, c = cg * 4;
    if (kr < D) {
      if (vec) {
        if (c < D) store_vec<4>(S + (size_t)kr * D + c, s[it]);
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (c + j < D) S[(size_t)kr * D + c + j] = s[it][j];
      }
    }
  }
}

template <typename T>
void delta_step_t(const DeltaArgs& p, int seqs, hipStream_t s) {
  const dim3 grid(p.heads, seqs);
  const size_t lds = sizeof(float) * (p.z ? 0 : p.rank);
#define DS_GO(DP, NT, MW)                                                     \
  delta_step_kernel<T, DP, NT, MW><<<grid, NT, lds, s>>>(p)
  if (p.dim <= 32) {
    DS_GO(32, 64, 4);
  } else if (p.dim <= 64) {
    DS_GO(64, 256, 5);
  } else if (p.dim <= 128) {
    // few heads: more threads shorten each one's walk
    if (p.heads * seqs <= 512) { DS_GO(128, 512, 2); }
    else { DS_GO(128, 256, 3); }
  } else {
    DS_GO(256, 1024, 4);
  }
#undef DS_GO
}

}  // namespace

extern "C" void launch_delta_step(const DeltaArgs* p, int seqs, int f32,
                                  hipStream_t s) {
  if (f32) delta_step_t<float>(*p, seqs, s);
  else delta_step_t<__hip_bfloat16>(*p, seqs, s);
}
