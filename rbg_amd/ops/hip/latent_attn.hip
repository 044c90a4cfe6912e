// Latent attention (gfx950): the normed latent is the only cached row, and a
// query sees the last `window` positions (window 0: all of them).
//
//   latent_store  c = rms_norm(down-projection) * w, written to the paged pool
//                 and to a contiguous buffer for this step's expansion
//   attn_rows     one wave per (query row, head), any head sizes, bf16 or f32:
//                 keys 64 at a time, a lane scores a key, then the lanes hold
//                 the value dimensions.  Contiguous keys/values (expanded per
//                 head, prefill) or the paged latents themselves as both key
//                 and value (query absorbed into the latent space, decode).
#include "latent_args.h"
#include "vec_io.h"

namespace {

template <typename T, int V>
__global__ __launch_bounds__(256) void latent_store_kernel(
    T* __restrict__ c, T* __restrict__ cache, const T* __restrict__ x,
    const long x_stride, const float* __restrict__ w,
    const int* __restrict__ slots, const int rows, const int rank,
    const float eps) {
  const int row = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (row >= rows) return;
  const T* src = x + (size_t)row * x_stride;
  float ss = 0.f;
  for (int i = lane * V; i < rank; i += 64 * V) {
    float v[V];
    load_vec<V>(src + i, v);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += v[j] * v[j];
  }
  const float inv = 1.f / sqrtf(wave_sum(ss) / rank + eps);
  const int slot = slots[row];
  for (int i = lane * V; i < rank; i += 64 * V) {
    float v[V], wv[V];
    load_vec<V>(src + i, v);
    load_vec<V>(w + i, wv);
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] = v[j] * inv * wv[j];
    if (slot >= 0) store_vec<V>(cache + (size_t)slot * rank + i, v);
    if (c != nullptr) store_vec<V>(c + (size_t)row * rank + i, v);
  }
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
  const T* vp = (const T*)p.v + head * p.v_head;
  float m = -INFINITY, l = 0.f, acc[NACC];
#pragma unroll
  for (int i = 0; i < NACC; ++i) acc[i] = 0.f;

  for (int j0 = lo; j0 <= pos; j0 += 64) {
    const int j = j0 + lane;
    float s = -INFINITY;
    if (j <= pos) {
      const T* kr = kp + key_row(j) * p.k_row;
      float dot = 0.f;
      for (int i = 0; i < p.d; ++i) dot += q[i] * to_f(kr[i]);
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

void launch_latent_store(void* c, void* cache, const void* x, long x_stride,
                         const float* w, const int* slots, int rows, int rank,
                         float eps, int f32, hipStream_t s) {
  const int grid = (rows + 3) / 4;
  const bool vec = rank % 8 == 0 && x_stride % 8 == 0 &&
                   ((uintptr_t)x & 15) == 0;
#define LS_GO(T, V) latent_store_kernel<T, V><<<grid, 256, 0, s>>>(           \
      (T*)c, (T*)cache, (const T*)x, x_stride, w, slots, rows, rank, eps)
  if (f32) { if (vec) LS_GO(float, 8); else LS_GO(float, 1); }
  else { if (vec) LS_GO(__hip_bfloat16, 8); else LS_GO(__hip_bfloat16, 1); }
#undef LS_GO
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
