// Dtype-generic vector access for the kernels that run in bf16 or f32: values
// travel as floats in registers, V elements per access.
#pragma once
#include "common.h"

DEV_INLINE float to_f(float v) { return v; }
DEV_INLINE float to_f(__hip_bfloat16 v) { return __bfloat162float(v); }
template <typename T> DEV_INLINE T from_f(float v);
template <> DEV_INLINE float from_f<float>(float v) { return v; }
template <> DEV_INLINE __hip_bfloat16 from_f<__hip_bfloat16>(float v) {
  return __float2bfloat16(v);
}
// v rounded to T and back: what a reader of the stored value will see
template <typename T> DEV_INLINE float round_to(float v) {
  return to_f(from_f<T>(v));
}

template <int V>
DEV_INLINE void load_vec(const __hip_bfloat16* p, float* o) {
  if constexpr (V == 8) {
    Bf16x8U t;
    t.u = *reinterpret_cast<const uint4*>(p);
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = bf2f(t.e[j]);
  } else if constexpr (V == 4) {
    union { uint2 u; __hip_bfloat16 e[4]; } t;
    t.u = *reinterpret_cast<const uint2*>(p);
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = bf2f(t.e[j]);
  } else {
#pragma unroll
    for (int j = 0; j < V; ++j) o[j] = bf2f(p[j]);
  }
}

template <int V>
DEV_INLINE void load_vec(const float* p, float* o) {
  if constexpr (V % 4 == 0) {
#pragma unroll
    for (int j = 0; j < V; j += 4) {
      const float4 t = *reinterpret_cast<const float4*>(p + j);
      o[j] = t.x; o[j + 1] = t.y; o[j + 2] = t.z; o[j + 3] = t.w;
    }
  } else {
#pragma unroll
    for (int j = 0; j < V; ++j) o[j] = p[j];
  }
}

template <int V>
DEV_INLINE void store_vec(__hip_bfloat16* p, const float* o) {
  if constexpr (V == 8) {
    Bf16x8U t;
#pragma unroll
    for (int j = 0; j < 8; ++j) t.e[j] = f2bf(o[j]);
    *reinterpret_cast<uint4*>(p) = t.u;
  } else if constexpr (V == 4) {
    union { uint2 u; __hip_bfloat16 e[4]; } t;
#pragma unroll
    for (int j = 0; j < 4; ++j) t.e[j] = f2bf(o[j]);
    *reinterpret_cast<uint2*>(p) = t.u;
  } else {
#pragma unroll
    for (int j = 0; j < V; ++j) p[j] = f2bf(o[j]);
  }
}

template <int V>
DEV_INLINE void store_vec(float* p, const float* o) {
  if constexpr (V % 4 == 0) {
#pragma unroll
    for (int j = 0; j < V; j += 4)
      *reinterpret_cast<float4*>(p + j) =
          make_float4(o[j], o[j + 1], o[j + 2], o[j + 3]);
  } else {
#pragma unroll
    for (int j = 0; j < V; ++j) p[j] = o[j];
  }
}

// f32 to about two units in the last place: hardware exp2 and reciprocal
DEV_INLINE float rcp_f(float x) { return __builtin_amdgcn_rcpf(x); }
DEV_INLINE float sigmoid_f(float z) { return rcp_f(1.f + __expf(-z)); }
