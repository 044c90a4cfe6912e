// Latent attention (gfx950): the normed latent is the only cached row, and a
// query sees the last `window` positions (window 0: all of them).
//
//   latent_store  c = rms_norm(down-projection) * w, and behind it a rotated key
//                 part that all heads share, written to the paged pool and to a
//                 contiguous buffer for this step's expansion; a second latent
//                 (of queries) may be normed in the same launch
//   rotate        the rotated part of a step's queries, in place
//   attn_rows     one wave per (query row, head), any head sizes, bf16 or f32:
//                 keys 64 at a time, a lane scores a key, then the lanes hold
//                 the value dimensions.  Contiguous keys/values (expanded per
//                 head, prefill) or the paged latents themselves as both key
//                 and value (query absorbed into the latent space, decode).
#include "latent_args.h"
#include "rotary.h"
#include "vec_io.h"

namespace {

// blockIdx.y 0: the latent and its key part; 1: the second latent
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_store_kernel(
    const LatentStoreArgs p) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (row >= p.rows) return;
  const bool second = blockIdx.y == 1;
  const int rank = second ? p.rank2 : p.rank;
  const T* src = second ? (const T*)p.x2 + (size_t)row * p.x2_row
                        : (const T*)p.x + (size_t)row * p.x_row;
  const float* w = second ? p.w2 : p.w;
  const int wide = second ? rank : rank + p.rot.dims;
  T* c = (second ? (T*)p.c2 : (T*)p.c) + (size_t)row * wide;
  const int slot = second ? -1 : p.slots[row];
  T* kept = slot >= 0 ? (T*)p.cache + (size_t)slot * wide : nullptr;
  float ss = 0.f;
  for (int i = lane * V; i < rank; i += 64 * V) {
    float v[V];
    load_vec<V>(src + i, v);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += v[j] * v[j];
  }
  const float inv = 1.f / sqrtf(wave_sum(ss) / rank + p.eps);
  for (int i = lane * V; i < rank; i += 64 * V) {
    float v[V], wv[V];
    load_vec<V>(src + i, v);
    load_vec<V>(w + i, wv);
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = v[j] * inv * wv[j];
    if (kept != nullptr) store_vec<V>(kept + i, v);
    store_vec<V>(c + i, v);
  }
  if (second || p.rot.dims == 0) return;
  const float* cs = rotary_row(p.rot, row);
  for (int i = lane; i < p.rot.dims / 2; i += 64) {
    rotate_pair(p.rot, cs, i, src + rank, c + rank);
    if (kept != nullptr) rotate_pair(p.rot, cs, i, src + rank, kept + rank);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void rotate_kernel(const RotateArgs p,
                                                     const long total) {
  const long item = blockIdx.x * 256l + threadIdx.x;
  if (item >= total) return;
  const int half = p.rot.dims / 2, i = (int)(item % half);
  const int head = (int)(item / half % p.heads);
  const int row = (int)(item / ((long)half * p.heads));
  T* x = (T*)p.x + row * p.x_row + head * p.x_head;
  rotate_pair(p.rot, rotary_row(p.rot, row), i, x, x);
}

__global__ __launch_bounds__(256) void rotate_vec_kernel(const RotateArgs p,
                                                         const long total) {
  const long item = blockIdx.x * 256l + threadIdx.x;
  if (item >= total) return;
  const int per = rotary_vecs(p.rot);
  const int head = (int)(item / per % p.heads);
  const int row = (int)(item / ((long)per * p.heads));
  __hip_bfloat16* x = (__hip_bfloat16*)p.x + row * p.x_row + head * p.x_head;
  rotate_vec(p.rot, rotary_row(p.rot, row), (int)(item % per), x, x);
}

// NACC: value dimensions per lane (dv <= 64 * NACC)
template <typename T, int NACC, bool PAGED>
__global__ __launch_bounds__(256) void attn_rows_kernel(const AttnRowsArgs p) {
  extern __shared__ float smem[];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const long item = (long)blockIdx.x * 4 + wave;
  if (item >= (long)p.rows * p.heads) return;       // whole wave leaves
  const int row = (int)(item / p.heads), head = (int)(item % p.heads);
  float* q = smem + wave * (p.d + 64);
  float* pr = q + p.d;
  const T* qp = (const T*)p.q + row * p.q_row + head * p.q_head;
  for (int i = lane; i < p.d; i += 64) q[i] = to_f(qp[i]);

  int pos, base = 0;
  const int* table = nullptr;
  if (PAGED) {
    pos = p.ctx[row] - 1;
    table = p.tables + (size_t)row * p.max_pages;
  } else {
    base = p.row_info[row * 2];
    pos = p.row_info[row * 2 + 1];
  }
  auto key_row = [&](int j) -> long {
    return PAGED ? (long)table[j / p.page_size] * p.page_size +
                       j % p.page_size
                 : (long)base + j;
  };
  const int lo = p.window > 0 ? max(0, pos - p.window + 1) : 0;
  const T* kp = (const T*)p.k + head * p.k_head;
  const T* k2 = (const T*)p.k2;
  const T* vp = (const T*)p.v + head * p.v_head;
  float m = -INFINITY, l = 0.f, acc[NACC];
  if (p.sink != nullptr) {
    m = p.sink[head];
    l = 1.f;
  }
#pragma unroll
  for (int i = 0; i < NACC; ++i) acc[i] = 0.f;

  for (int j0 = lo; j0 <= pos; j0 += 64) {
    const int j = j0 + lane;
    float s = -INFINITY;
    if (j <= pos) {
      const long at = key_row(j);
      const T* kr = kp + at * p.k_row;
      float dot = 0.f;
      for (int i = 0; i < p.d1; ++i) dot += q[i] * to_f(kr[i]);
      if (k2 != nullptr) {
        kr = k2 + at * p.k2_row - p.d1;
        for (int i = p.d1; i < p.d; ++i) dot += q[i] * to_f(kr[i]);
      }
      s = dot * p.scale;
    }
    const float mn = fmaxf(m, wave_max(s));
    const float e = expf(s - mn);
    const float corr = expf(m - mn);
    l = l * corr + wave_sum(e);
    m = mn;
    pr[lane] = e;                 // wave-private LDS: lockstep, no barrier
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < NACC; ++i) acc[i] *= corr;
    const int n = min(64, pos - j0 + 1);
    for (int t = 0; t < n; ++t) {
      const T* vr = vp + key_row(j0 + t) * p.v_row;
      const float w = pr[t];
#pragma unroll
      for (int i = 0; i < NACC; ++i) {
        const int d = i * 64 + lane;
        if (d < p.dv) acc[i] += w * to_f(vr[d]);
      }
    }
    __builtin_amdgcn_wave_barrier();
  }
  T* op = (T*)p.out + row * p.o_row + head * p.o_head;
#pragma unroll
  for (int i = 0; i < NACC; ++i) {
    const int d = i * 64 + lane;
    if (d < p.dv) {
      float o = acc[i] / l;
      if (p.gate != nullptr)
        o *= sigmoid_f(to_f(((const T*)p.gate)[row * p.g_row +
                                               (long)head * p.dv + d]));
      op[d] = from_f<T>(o);
    }
  }
}

template <typename T, bool PAGED>
void attn_rows_t(const AttnRowsArgs& p, hipStream_t s) {
  const long items = (long)p.rows * p.heads;
  const int grid = (int)((items + 3) / 4);
  const size_t lds = sizeof(float) * 4 * (p.d + 64);
#define AR_GO(N) attn_rows_kernel<T, N, PAGED><<<grid, 256, lds, s>>>(p)
  if (p.dv <= 64) AR_GO(1);
  else if (p.dv <= 128) AR_GO(2);
  else if (p.dv <= 256) AR_GO(4);
  else if (p.dv <= 512) AR_GO(8);
  else AR_GO(16);
#undef AR_GO
}

}  // namespace

extern "C" {

void launch_latent_store(const LatentStoreArgs* p, int f32, int vec,
                         hipStream_t s) {
  const dim3 grid((p->rows + 3) / 4, p->x2 != nullptr ? 2 : 1);
#define LS_GO(T, V) latent_store_kernel<T, V><<<grid, 256, 0, s>>>(*p)
  if (f32) { if (vec) LS_GO(float, 8); else LS_GO(float, 1); }
  else { if (vec) LS_GO(__hip_bfloat16, 8); else LS_GO(__hip_bfloat16, 1); }
#undef LS_GO
}

void launch_rotate(const RotateArgs* p, int f32, int vec, hipStream_t s) {
  const long per = vec ? rotary_vecs(p->rot) : p->rot.dims / 2;
  const long total = (long)p->rows * p->heads * per;
  const int grid = (int)((total + 255) / 256);
  if (vec) {
    rotate_vec_kernel<<<grid, 256, 0, s>>>(*p, total);
  } else if (f32) {
    rotate_kernel<float><<<grid, 256, 0, s>>>(*p, total);
  } else {
    rotate_kernel<__hip_bfloat16><<<grid, 256, 0, s>>>(*p, total);
  }
}

void launch_attn_rows(const AttnRowsArgs* p, int f32, hipStream_t s) {
  const bool paged = p->tables != nullptr;
  if (f32) {
    if (paged) attn_rows_t<float, true>(*p, s);
    else attn_rows_t<float, false>(*p, s);
  } else {
    if (paged) attn_rows_t<__hip_bfloat16, true>(*p, s);
    else attn_rows_t<__hip_bfloat16, false>(*p, s);
  }
}

}  // extern "C"
