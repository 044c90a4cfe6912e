// MFMA operands used by the token-mixer kernels.
//
// All of them keep products in "C layout" (column = lane & 15, row =
// 4 * (lane >> 4) + r) and feed one product's registers to the next as a B
// operand without moving them: the contraction index of an MFMA may be
// permuted freely if A and B agree, so the A side is read with
//   index 4 * (lane >> 4) + r   where the B side is register r.
#pragma once
#include "common.h"

typedef __attribute__((ext_vector_type(4))) __bf16 mf_bf4;
typedef __attribute__((ext_vector_type(8))) __bf16 mf_bf8;
// staging registers: HIP's own uint4 is a class that ends up in scratch memory
// when kept in arrays
typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;

DEV_INLINE mf_bf8 frag8(const __hip_bfloat16* p) {
  union { uint4 u; mf_bf8 v; } c;
  c.u = *reinterpret_cast<const uint4*>(p);
  return c.v;
}

// Transposing LDS read.  Within 16 lanes, lane i passes the address of row
// i >> 2, columns 4 * (i & 3) .. +3; it receives rows 0..3 of column i.
DEV_INLINE mf_bf4 tr_read4(const __hip_bfloat16* p) {
  typedef __attribute__((address_space(3))) mf_bf4 lds_bf4;
  return __builtin_amdgcn_ds_read_tr16_b64_v4bf16(
      (lds_bf4*)(uint32_t)(uintptr_t)p);
}

DEV_INLINE f32x4 mfma_bf16_k32(mf_bf8 a, mf_bf8 b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
}

DEV_INLINE f32x4 mfma_bf16_k16(mf_bf4 a, mf_bf4 b, f32x4 c) {
  union { mf_bf4 v; short4_t s; } x, y;
  x.v = a;
  y.v = b;
  return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(x.s, y.s, c, 0, 0, 0);
}

// true f32: A row = lane & 15, k = lane >> 4; B col = lane & 15, k = lane >> 4
DEV_INLINE f32x4 mfma_f32_k4(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// x = hi + lo with 16 bits of mantissa: two MFMAs keep an f32 operand's
// weight where one bf16 operand would round it to 8 bits
DEV_INLINE void split_bf16(float x, __bf16& hi, __bf16& lo) {
  hi = (__bf16)x;
  lo = (__bf16)(x - (float)hi);
}

DEV_INLINE float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }
constexpr float LOG2E = 1.4426950408889634f;
constexpr float MASKED = -1e30f;
