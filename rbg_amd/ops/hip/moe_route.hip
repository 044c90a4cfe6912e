// Routing of tokens to experts (gfx950).
//
//   logits   x W^T with f32 sums.  W rows are MFMA A fragments: lanes are tokens,
//            registers experts.
//   choose   one wave per token: sigmoid, logit or softmax, correction, the
//            two best of each group of neighbours, the best groups, the best
//            experts of those; weights by the rule's mode.  Ranks are counted, not sorted: an expert's rank is the number of experts
//            ahead of it in the order (score, index), which is total, so every
//            place is filled exactly once whatever the scores are.
//   lay out  pairs (token, choice) counted per expert, offsets by a scan, tiles
//            of one expert each, and the permutation: one workgroup, together
//            with the choice for small batches; for prompts the counting and the
//            permutation are spread over blocks of tokens.  Experts from `real`
//            on have no weights: their pairs are weighed, but get no row.
#include "lds_stream.h"
#include "expert_args.h"
#include "vec_io.h"

namespace {

constexpr int UN = 4;                           // 32-k steps in flight

// decode batches: 8 waves split K
__global__ __launch_bounds__(512) void router_skinny_kernel(
    float* __restrict__ out, const __hip_bfloat16* __restrict__ x,
    const __hip_bfloat16* __restrict__ w, const int tokens, const int experts,
    const int k_len) {
  constexpr int KW = 8;
  __shared__ f32x4 red[KW][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int gl = lane & 15, gs = lane >> 4;
  const int e0 = blockIdx.x * 16, t0 = blockIdx.y * 16;
  const __hip_bfloat16* wr = w + (size_t)min(e0 + gl, experts - 1) * k_len;
  const __hip_bfloat16* xr = x + (size_t)min(t0 + gl, tokens - 1) * k_len;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  const int per = ((k_len + KW * 32 - 1) / (KW * 32)) * 32;
  const int kb = wave * per, ke = min(kb + per, k_len);
  for (int k0 = kb; k0 < ke; k0 += 32 * UN) {
    // unconditional clamped loads, all before the first product
    mf_bf8 wf[UN], xf[UN];
    const mf_bf8 z = {};
#pragma unroll
    for (int u = 0; u < UN; ++u) {
      const int kc = min(k0 + u * 32 + gs * 8, k_len - 8);
      wf[u] = frag8(wr + kc);
      xf[u] = frag8(xr + kc);
    }
#pragma unroll
    for (int u = 0; u < UN; ++u)
      acc = mfma_bf16_k32(k0 + u * 32 + gs * 8 < ke ? wf[u] : z, xf[u], acc);
  }
  red[wave][lane] = acc;
  __syncthreads();
  if (wave > 0) return;
#pragma unroll
  for (int kk = 1; kk < KW; ++kk) acc += red[kk][lane];
  const int e = e0 + gs * 4;
  if (t0 + gl >= tokens) return;
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (e + r < experts) out[(size_t)(t0 + gl) * experts + e + r] = acc[r];
}

// prompts: 32 tokens x 64 experts through LDS
using RouterStream = LdsStream<32, 4>;

__global__ __launch_bounds__(256) void router_stream_kernel(
    float* __restrict__ out, const __hip_bfloat16* __restrict__ x,
    const __hip_bfloat16* __restrict__ w, const int tokens, const int experts,
    const int k_len) {
  __shared__ __attribute__((aligned(16))) char smem[RouterStream::BYTES];
  const int e0 = blockIdx.x * 64, t0 = blockIdx.y * 32;
  const int piece = stage_piece(), row = RouterStream::row();
  const uint32_t xo[1] = {
      ((uint32_t)min(row, tokens - 1 - t0) * k_len + piece * 8) * 2};
  const uint32_t wo[2] = {
      ((uint32_t)min(e0 + row, experts - 1) * k_len + piece * 8) * 2,
      ((uint32_t)min(e0 + 32 + row, experts - 1) * k_len + piece * 8) * 2};
  f32x4 acc[2];
  RouterStream::run(x + (size_t)t0 * k_len, xo, w, wo, k_len,
                    blockIdx.y % ((k_len + BK - 1) / BK), 2, smem, acc);
  const int e = e0 + (threadIdx.x >> 6) * 16 + ((threadIdx.x & 63) >> 4) * 4;
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int tok = t0 + j * 16 + (threadIdx.x & 15);
    if (tok >= tokens) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (e + r < experts) out[(size_t)tok * experts + e + r] = acc[j][r];
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

// LDS floats of one wave's choice: experts (twice) and groups, padded to whole
// quads, and the chosen's numbers and weights
__host__ __device__ inline int choice_floats(const MoeRouteArgs& p) {
  return 2 * ((p.experts + 3) & ~3) + ((p.groups + 3) & ~3) +
         2 * ((p.top + 3) & ~3);
}

// how many of the n values (padded with -inf) are ahead of value `mine` at `at`
DEV_INLINE int rank_of(const float* v, const int n, const float mine,
                       const int at) {
  int rank = 0;
#pragma unroll 4
  for (int o = 0; o < n; o += 4) {
    const float4 c = *reinterpret_cast<const float4*>(v + o);
    rank += c.x > mine || (c.x == mine && o < at);
    rank += c.y > mine || (c.y == mine && o + 1 < at);
    rank += c.z > mine || (c.z == mine && o + 2 < at);
    rank += c.w > mine || (c.w == mine && o + 3 < at);
  }
  return rank;
}

// One wave, one token; `choice` is its own LDS.
DEV_INLINE void choose(const MoeRouteArgs& p, const int token, float* choice,
                       const int lane) {
  const float* z = p.logits + (size_t)token * p.experts;
  const int ep = (p.experts + 3) & ~3, gp = (p.groups + 3) & ~3;
  float* score = choice + ep;
  float* group = score + ep;
  float* won = group + gp;                      // by rank
  int* who = (int*)(won + ((p.top + 3) & ~3));
  float most = -INFINITY;
  for (int e = lane; e < p.experts; e += 64) {
    score[e] = z[e];
    choice[e] = p.correction[e];
    most = fmaxf(most, score[e]);
  }
  if (p.mode == ROUTE_SHARE) {                  // softmax over all
    most = wave_max(most);
    float sum = 0.f;
    for (int e = lane; e < p.experts; e += 64) {
      score[e] = expf(score[e] - most);
      sum += score[e];
    }
    const float part = 1.f / wave_sum(sum);
    for (int e = lane; e < p.experts; e += 64) score[e] *= part;
  } else if (p.mode == ROUTE_SIGMOID) {
    for (int e = lane; e < p.experts; e += 64)
      score[e] = sigmoid_exact(score[e]);
  }
  for (int e = lane; e < ep; e += 64)           // NaN becomes the least score
    choice[e] = e < p.experts ? fmaxf(score[e] + choice[e], -3e38f)
                              : -INFINITY;
  wave_fence();
  const int size = p.experts / p.groups;
  if (p.keep < p.groups) {
    for (int g = lane; g < gp; g += 64) {
      float a = -INFINITY, b = -INFINITY;
      if (g < p.groups) {
#pragma unroll 4
        for (int i = 0; i < size; ++i) {
          const float c = choice[g * size + i];
          b = fmaxf(b, fminf(a, c));
          a = fmaxf(a, c);
        }
        if (size > 1) a += b;
      }
      group[g] = a;
    }
    wave_fence();
    for (int g = lane; g < p.groups; g += 64)
      if (rank_of(group, gp, group[g], g) >= p.keep)
        for (int i = 0; i < size; ++i) choice[g * size + i] = -INFINITY;
    wave_fence();
  }
  if (p.mode == ROUTE_CHOSEN) {
    most = -INFINITY;
    for (int e = lane; e < p.experts; e += 64) most = fmaxf(most, choice[e]);
    most = wave_max(most);
  }
  for (int e = lane; e < p.experts; e += 64) {
    const float mine = choice[e];
    if (mine == -INFINITY) continue;
    const int rank = rank_of(choice, ep, mine, e);
    if (rank < p.top) {
      won[rank] = p.mode == ROUTE_CHOSEN ? expf(mine - most) : score[e];
      who[rank] = e;
    }
  }
  wave_fence();
  float scale = 1.f;
  if (p.mode != ROUTE_SIGMOID) {
    float total = 0.f;
    for (int r = lane; r < p.top; r += 64) total += won[r];
    total = wave_sum(total);
    scale = p.mode == ROUTE_SHARE ? p.scale / (total + 1e-20f) : 1.f / total;
  }
  for (int r = lane; r < p.top; r += 64) {
    p.ids[(size_t)token * p.top + r] = who[r];
    p.weights[(size_t)token * p.top + r] = won[r] * scale;
  }
  wave_fence();
}

// From each expert's count (LDS) its first row (LDS, cursor) and its tiles.  One
// workgroup of NT threads; scan [2 * waves]: LDS.
template <int NT>
DEV_INLINE void offsets(const MoeRouteArgs& p, const int* count, int* cursor,
                        int* scan) {
  const int tid = threadIdx.x;
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
#pragma unroll
    for (int wv = 0; wv < NT / 64; ++wv) {
      const int a = scan[wv * 2], b = scan[wv * 2 + 1];
      if (wv < (tid >> 6)) {
        ra += a;
        ta += b;
      }
      rows0 += a;
      tiles0 += b;
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
}

// Pairs [lo, hi) counted into, or placed by, an LDS array over the experts.
template <int NT>
DEV_INLINE void count_pairs(const MoeRouteArgs& p, int* count, int lo, int hi) {
  for (int e = threadIdx.x; e < p.experts; e += NT) count[e] = 0;
  __syncthreads();
#pragma unroll 4
  for (int i = lo + threadIdx.x; i < hi; i += NT)
    if (p.ids[i] < p.real) atomicAdd(&count[p.ids[i]], 1);
  __syncthreads();
}

template <int NT>
DEV_INLINE void place_pairs(const MoeRouteArgs& p, int* cursor, int lo,
                            int hi) {
#pragma unroll 4
  for (int i = lo + threadIdx.x; i < hi; i += NT) {
    const int e = p.ids[i];
    const int at = e < p.real ? atomicAdd(&cursor[e], 1) : -1;
    p.inv[i] = at;
    if (at >= 0) p.rows[at] = i / p.top;
  }
}

// decode batches: choice and layout in one workgroup
template <int NT>
__global__ __launch_bounds__(NT) void route_small_kernel(const MoeRouteArgs p) {
  extern __shared__ float route_smem[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float* mine = route_smem + wave * choice_floats(p);
  for (int t = wave; t < p.tokens; t += NT / 64) choose(p, t, mine, lane);
  __threadfence_block();
  __syncthreads();
  int* count = (int*)route_smem;
  int* cursor = count + p.experts;
  count_pairs<NT>(p, count, 0, p.tokens * p.top);
  offsets<NT>(p, count, cursor, cursor + p.experts);
  place_pairs<NT>(p, cursor, 0, p.tokens * p.top);
}

// middling batches: the choice, 4 tokens a workgroup, then the layout in one
__global__ __launch_bounds__(256) void choose_kernel(const MoeRouteArgs p) {
  extern __shared__ float route_smem[];
  const int wave = threadIdx.x >> 6, t = blockIdx.x * 4 + wave;
  if (t < p.tokens)                             // whole waves
    choose(p, t, route_smem + wave * choice_floats(p),
           threadIdx.x & 63);
}

constexpr int CN = 1024;

__global__ __launch_bounds__(CN) void lay_out_kernel(const MoeRouteArgs p) {
  extern __shared__ int lay_smem[];
  int* cursor = lay_smem + p.experts;
  count_pairs<CN>(p, lay_smem, 0, p.tokens * p.top);
  offsets<CN>(p, lay_smem, cursor, cursor + p.experts);
  place_pairs<CN>(p, cursor, 0, p.tokens * p.top);
}

// prompts: BT tokens' choice, and how often it took each expert: part [blocks,
// experts]
constexpr int BT = 32;

template <int NT>
__global__ __launch_bounds__(NT) void choose_count_kernel(
    const MoeRouteArgs p) {
  extern __shared__ float route_smem[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float* mine = route_smem + wave * choice_floats(p);
  const int lo = blockIdx.x * BT, hi = min(lo + BT, p.tokens);
  for (int t = lo + wave; t < hi; t += NT / 64) choose(p, t, mine, lane);
  __threadfence_block();
  __syncthreads();
  int* count = (int*)route_smem;
  count_pairs<NT>(p, count, lo * p.top, hi * p.top);
  for (int e = threadIdx.x; e < p.experts; e += NT)
    p.part[(size_t)blockIdx.x * p.experts + e] = count[e];
}

// part becomes the first row of each block's pairs of each expert.  A thread
// takes a run of blocks of one expert.
__global__ __launch_bounds__(CN) void offsets_kernel(const MoeRouteArgs p,
                                                     const int blocks) {
  extern __shared__ int lay_smem[];
  int* count = lay_smem;                        // [experts]
  int* cursor = count + p.experts;              // [experts]
  int* scan = cursor + p.experts;               // [2 * waves]
  int* run = scan + 2 * CN / 64;                // [CN]
  const int lanes = min(max(CN / p.experts, 1), 32);    // runs per expert
  const int len = (blocks + lanes - 1) / lanes;
  const int e = threadIdx.x % p.experts, r = threadIdx.x / p.experts;
  const bool on = p.experts <= CN && r < lanes;
  const int b0 = min(r * len, blocks), b1 = min(b0 + len, blocks);
  int n = 0;
  if (on) {
#pragma unroll 8
    for (int b = b0; b < b1; ++b) n += p.part[(size_t)b * p.experts + e];
    run[r * p.experts + e] = n;
  }
  __syncthreads();
  if (threadIdx.x < p.experts) {
    int total = 0;
    for (int i = 0; i < lanes; ++i) {
      const int v = run[i * p.experts + threadIdx.x];
      run[i * p.experts + threadIdx.x] = total;
      total += v;
    }
    count[threadIdx.x] = total;
  }
  __syncthreads();
  offsets<CN>(p, count, cursor, scan);
  if (on) {
    int at = cursor[e] + run[r * p.experts + e];
#pragma unroll 8
    for (int b = b0; b < b1; ++b) {
      const int v = p.part[(size_t)b * p.experts + e];
      p.part[(size_t)b * p.experts + e] = at;
      at += v;
    }
  }
}

__global__ __launch_bounds__(256) void place_kernel(const MoeRouteArgs p) {
  extern __shared__ int lay_smem[];
  for (int e = threadIdx.x; e < p.experts; e += 256)
    lay_smem[e] = p.part[(size_t)blockIdx.x * p.experts + e];
  __syncthreads();
  const int lo = blockIdx.x * BT, hi = min(lo + BT, p.tokens);
  place_pairs<256>(p, lay_smem, lo * p.top, hi * p.top);
}

}  // namespace

extern "C" {

void launch_router_logits(float* out, const void* x, const void* w, int tokens,
                          int experts, int k, int f32, int vec,
                          hipStream_t s) {
  if (vec) {
    const __hip_bfloat16 *xb = (const __hip_bfloat16*)x,
                         *wb = (const __hip_bfloat16*)w;
    if (tokens <= 512) {
      router_skinny_kernel
          <<<dim3((experts + 15) / 16, (tokens + 15) / 16), 512, 0, s>>>(
              out, xb, wb, tokens, experts, k);
    } else {
      router_stream_kernel
          <<<dim3((experts + 63) / 64, (tokens + 31) / 32), 256, 0, s>>>(
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

// blocks of tokens that count on their own
int moe_route_blocks(int tokens) {
  return tokens <= 512 ? 0 : (tokens + BT - 1) / BT;
}

void launch_moe_route(const MoeRouteArgs* p, hipStream_t s) {
  const int blocks = moe_route_blocks(p->tokens);
  const size_t own = sizeof(float) * choice_floats(*p);
  const size_t lay = sizeof(int) * (2 * p->experts + 32);
  if (blocks > 0) {
    if (own * 16 <= 65536) {
      choose_count_kernel<1024><<<blocks, 1024, own * 16, s>>>(*p);
    } else {
      choose_count_kernel<256><<<blocks, 256, own * 4, s>>>(*p);
    }
    offsets_kernel<<<1, CN, lay + sizeof(int) * CN, s>>>(*p, blocks);
    place_kernel<<<blocks, 256, sizeof(int) * p->experts, s>>>(*p);
  } else if (p->tokens <= 4) {
    route_small_kernel<256><<<1, 256, own * 4 > lay ? own * 4 : lay, s>>>(*p);
  } else if (p->tokens <= 16 && own * 16 <= 65536) {
    route_small_kernel<1024><<<1, 1024, own * 16 > lay ? own * 16 : lay,
                               s>>>(*p);
  } else {
    choose_kernel<<<(p->tokens + 3) / 4, 256, own * 4, s>>>(*p);
    lay_out_kernel<<<1, CN, lay, s>>>(*p);
  }
}

}  // extern "C"
