// Routing of tokens to experts (gfx950).
//
//   logits   x W^T with f32 sums: a workgroup takes 16 experts and 16 * MT
//            tokens, its waves split K and meet in LDS.  W rows are MFMA A
//            fragments, so lanes are tokens and registers experts.
//   choose   one wave per token: sigmoid, correction, the two best of each group
//            of neighbours, the best groups, the best experts of those.  Ranks
//            are counted, not sorted: an expert's rank is the number of experts
//            ahead of it in the order (score, index), which is total, so every
//            place is filled exactly once whatever the scores are.
//   lay out  one workgroup: pairs (token, choice) counted per expert, offsets
//            by a scan, tiles of one expert each, and the permutation.
#include "mfma_util.h"
#include "moe_args.h"
#include "vec_io.h"

namespace {

constexpr int UN = 4;                           // 32-k steps in flight

template <int MT, int NW>
__global__ __launch_bounds__(NW * 64) void router_logits_kernel(
    float* __restrict__ out, const __hip_bfloat16* __restrict__ x,
    const __hip_bfloat16* __restrict__ w, const int tokens, const int experts,
    const int k_len) {
  __shared__ f32x4 red[NW][MT][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int e0 = blockIdx.x * 16, t0 = blockIdx.y * 16 * MT;
  const __hip_bfloat16* wr = w + (size_t)min(e0 + gl, experts - 1) * k_len;
  const __hip_bfloat16* xr[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t)
    xr[t] = x + (size_t)min(t0 + t * 16 + gl, tokens - 1) * k_len;
  f32x4 acc[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) acc[t] = {0.f, 0.f, 0.f, 0.f};
  const int per = ((k_len + NW * 32 - 1) / (NW * 32)) * 32;
  const int kb = wave * per, ke = min(kb + per, k_len);
  for (int k0 = kb; k0 < ke; k0 += 32 * UN) {
    // unconditional clamped loads, all before the first product
    mf_bf8 wf[UN], xf[UN][MT];
    const mf_bf8 z = {};
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const int kc = min(k0 + u * 32 + gs * 8, k_len - 8);
      wf[u] = frag8(wr + kc);
#pragma unroll
      for (int t = 0; t < MT; ++t) xf[u][t] = frag8(xr[t] + kc);
    }
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const mf_bf8 w1 = k0 + u * 32 + gs * 8 < ke ? wf[u] : z;
#pragma unroll
      for (int t = 0; t < MT; ++t)
        acc[t] = mfma_bf16_k32(w1, xf[u][t], acc[t]);
    }
  }
#pragma unroll
  for (int t = 0; t < MT; ++t) red[wave][t][lane] = acc[t];
  __syncthreads();
  for (int i = threadIdx.x; i < MT * 64; i += NW * 64) {
    const int t = i >> 6, ln = i & 63;
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int wv = 0; wv < NW; ++wv) s += red[wv][t][ln];
    const int tok = t0 + t * 16 + (ln & 15), e = e0 + (ln >> 4) * 4;
    if (tok >= tokens) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (e + r < experts) out[(size_t)tok * experts + e + r] = s[r];
  }
}

// any sizes, bf16 or f32: one wave per (token, expert)
template <typename T>
__global__ __launch_bounds__(256) void router_rows_kernel(
    float* __restrict__ out, const T* __restrict__ x, const T* __restrict__ w,
    const long items, const int experts, const int k_len) {
  const long item = blockIdx.x * 4L + (threadIdx.x >> 6);
  if (item >= items) return;
  const T* xr = x + (size_t)(item / experts) * k_len;
  const T* wr = w + (size_t)(item % experts) * k_len;
  float s = 0.f;
  for (int k = threadIdx.x & 63; k < k_len; k += 64)
    s += to_f(xr[k]) * to_f(wr[k]);
  s = wave_sum(s);
  if ((threadIdx.x & 63) == 0) out[item] = s;
}

DEV_INLINE void wave_fence() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  __builtin_amdgcn_wave_barrier();
}

DEV_INLINE float sigmoid_exact(float z) { return 1.f / (1.f + expf(-z)); }

// One wave, one token.  choice [experts], group [groups]: its own LDS.
DEV_INLINE void choose(const MoeRouteArgs& p, const int token, float* choice,
                       float* group, const int lane) {
  const float* z = p.logits + (size_t)token * p.experts;
  for (int e = lane; e < p.experts; e += 64)    // NaN becomes the least score
    choice[e] = fmaxf(sigmoid_exact(z[e]) + p.correction[e], -3e38f);
  wave_fence();
  const int size = p.experts / p.groups;
  if (p.keep < p.groups) {
    for (int g = lane; g < p.groups; g += 64) {
      float a = -INFINITY, b = -INFINITY;
      for (int i = 0; i < size; ++i) {
        const float c = choice[g * size + i];
        b = fmaxf(b, fminf(a, c));
        a = fmaxf(a, c);
      }
      group[g] = size > 1 ? a + b : a;
    }
    wave_fence();
    // groups beyond 64 keep their scores in LDS until every rank is known
    for (int g0 = 0; g0 < p.groups; g0 += 64) {
      const int g = g0 + lane;
      if (g < p.groups) {
        int rank = 0;
        const float mine = group[g];
        for (int o = 0; o < p.groups; ++o)
          rank += group[o] > mine || (group[o] == mine && o < g);
        if (rank >= p.keep)
          for (int i = 0; i < size; ++i) choice[g * size + i] = -INFINITY;
      }
    }
    wave_fence();
  }
  for (int e = lane; e < p.experts; e += 64) {
    const float mine = choice[e];
    if (mine == -INFINITY) continue;
    int rank = 0;
    for (int o = 0; o < p.experts; ++o) {
      const float c = choice[o];
      rank += c > mine || (c == mine && o < e);
    }
    if (rank < p.top) {
      p.ids[(size_t)token * p.top + rank] = e;
      p.weights[(size_t)token * p.top + rank] = sigmoid_exact(z[e]);
    }
  }
  wave_fence();
}

// One workgroup of NT threads.  count [experts], cursor [experts], scan
// [2 * waves]: LDS.
template <int NT>
DEV_INLINE void lay_out(const MoeRouteArgs& p, int* count, int* cursor,
                        int* scan) {
  const int tid = threadIdx.x, pairs = p.tokens * p.top;
  for (int e = tid; e < p.experts; e += NT) count[e] = 0;
  __syncthreads();
#pragma unroll 4
  for (int i = tid; i < pairs; i += NT) atomicAdd(&count[p.ids[i]], 1);
  __syncthreads();
  // exclusive sums of rows (low half) and tiles (high half), NT experts a round
  int rows0 = 0, tiles0 = 0;
  for (int e0 = 0; e0 < p.experts; e0 += NT) {
    const int e = e0 + tid, n = e < p.experts ? count[e] : 0;
    const int nt = (n + p.tile - 1) / p.tile;
    int r = n, t = nt;
    // inclusive scan within the wave, then over the waves
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const int a = __shfl_up(r, off, 64), b = __shfl_up(t, off, 64);
      if ((tid & 63) >= off) {
        r += a;
        t += b;
      }
    }
    if ((tid & 63) == 63) {
      scan[(tid >> 6) * 2] = r;
      scan[(tid >> 6) * 2 + 1] = t;
    }
    __syncthreads();
    int ra = rows0, ta = tiles0;
    for (int wv = 0; wv < NT / 64; ++wv) {
      if (wv < (tid >> 6)) {
        ra += scan[wv * 2];
        ta += scan[wv * 2 + 1];
      }
      rows0 += scan[wv * 2];
      tiles0 += scan[wv * 2 + 1];
    }
    if (e < p.experts) {
      const int first = ra + r - n;
      cursor[e] = first;
      for (int i = 0; i < nt; ++i) {
        int* o = p.tiles + (size_t)(ta + t - nt + i) * 3;
        o[0] = e;
        o[1] = first + i * p.tile;
        o[2] = min(p.tile, n - i * p.tile);
      }
    }
    __syncthreads();
  }
  if (tid == 0) *p.count = tiles0;
#pragma unroll 4
  for (int i = tid; i < pairs; i += NT) {
    const int at = atomicAdd(&cursor[p.ids[i]], 1);
    p.inv[i] = at;
    p.rows[at] = i / p.top;
  }
}

__global__ __launch_bounds__(256) void choose_kernel(const MoeRouteArgs p) {
  extern __shared__ float route_smem[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int token = blockIdx.x * 4 + wave;
  if (token >= p.tokens) return;                // whole wave leaves
  float* mine = route_smem + wave * (p.experts + p.groups);
  choose(p, token, mine, mine + p.experts, lane);
}

constexpr int LN = 1024;

__global__ __launch_bounds__(LN) void lay_out_kernel(const MoeRouteArgs p) {
  extern __shared__ int lay_smem[];
  lay_out<LN>(p, lay_smem, lay_smem + p.experts, lay_smem + 2 * p.experts);
}

// decode batches: both in one workgroup
__global__ __launch_bounds__(LN) void route_small_kernel(const MoeRouteArgs p) {
  extern __shared__ float route_smem[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float* mine = route_smem + wave * (p.experts + p.groups);
  for (int t = wave; t < p.tokens; t += LN / 64)
    choose(p, t, mine, mine + p.experts, lane);
  __threadfence_block();
  __syncthreads();
  int* lay = (int*)route_smem;
  lay_out<LN>(p, lay, lay + p.experts, lay + 2 * p.experts);
}

}  // namespace

extern "C" {

void launch_router_logits(float* out, const void* x, const void* w, int tokens,
                          int experts, int k, int f32, int vec,
                          hipStream_t s) {
  if (vec) {
    const __hip_bfloat16 *xb = (const __hip_bfloat16*)x,
                         *wb = (const __hip_bfloat16*)w;
    const int eb = (experts + 15) / 16;
    if (tokens <= 512) {
      router_logits_kernel<1, 8><<<dim3(eb, (tokens + 15) / 16), 512, 0, s>>>(
          out, xb, wb, tokens, experts, k);
    } else {
      router_logits_kernel<4, 4><<<dim3(eb, (tokens + 63) / 64), 256, 0, s>>>(
          out, xb, wb, tokens, experts, k);
    }
    return;
  }
  const long items = (long)tokens * experts;
  const int grid = (int)((items + 3) / 4);
  if (f32) {
    router_rows_kernel<float><<<grid, 256, 0, s>>>(
        out, (const float*)x, (const float*)w, items, experts, k);
  } else {
    router_rows_kernel<__hip_bfloat16><<<grid, 256, 0, s>>>(
        out, (const __hip_bfloat16*)x, (const __hip_bfloat16*)w, items,
        experts, k);
  }
}

int moe_max_experts() { return 1024; }

void launch_moe_route(const MoeRouteArgs* p, hipStream_t s) {
  const size_t lay = sizeof(int) * (2 * p->experts + 2 * LN / 64);
  if (p->tokens <= 64 && p->experts <= 512) {
    const size_t own = sizeof(float) * 16 * (p->experts + p->groups);
    route_small_kernel<<<1, LN, own > lay ? own : lay, s>>>(*p);
    return;
  }
  choose_kernel<<<(p->tokens + 3) / 4, 256,
                  sizeof(float) * 4 * (p->experts + p->groups), s>>>(*p);
  lay_out_kernel<<<1, LN, lay, s>>>(*p);
}

}  // extern "C"
