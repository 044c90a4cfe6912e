// Rotation of pairs by position, in f32.
#pragma once
#include "latent_args.h"
#include "vec_io.h"

// cosines (sines half a row further) of a row's position
DEV_INLINE const float* rotary_row(const RotaryArgs& r, const int row) {
  return r.cos_sin +
         (size_t)min(max(r.positions[row], 0), r.table_rows - 1) * r.dims;
}

// pair i of src into dst; the two may be the same
template <typename T>
DEV_INLINE void rotate_pair(const RotaryArgs& r, const float* cs, const int i,
                            const T* src, T* dst) {
  const int half = r.dims / 2;
  const int a = r.interleaved ? 2 * i : i, b = r.interleaved ? a + 1 : i + half;
  const float c = cs[i], s = cs[half + i];
  const float u = to_f(src[a]), v = to_f(src[b]);
  dst[a] = from_f<T>(u * c - v * s);
  dst[b] = from_f<T>(v * c + u * s);
}

// 8 neighbouring elements at a time (twice 8 when the halves are paired): how many
// such pieces there are, and piece i of src into dst, which may be the same.  The
// dims are a multiple of 8 (16), the rows aligned.
__host__ DEV_INLINE int rotary_vecs(const RotaryArgs& r) {
  return r.interleaved ? r.dims / 8 : r.dims / 16;
}

DEV_INLINE void rotate_vec(const RotaryArgs& r, const float* cs, const int i,
                           const __hip_bfloat16* src, __hip_bfloat16* dst) {
  const int half = r.dims / 2, at = i * 8;
  float a[8], o[8];
  load_vec<8>(src + at, a);
  if (r.interleaved) {
    float c[4], s[4];
    load_vec<4>(cs + at / 2, c);
    load_vec<4>(cs + half + at / 2, s);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      o[2 * j] = a[2 * j] * c[j] - a[2 * j + 1] * s[j];
      o[2 * j + 1] = a[2 * j + 1] * c[j] + a[2 * j] * s[j];
    }
    store_vec<8>(dst + at, o);
    return;
  }
  float b[8], c[8], s[8];
  load_vec<8>(src + half + at, b);
  load_vec<8>(cs + at, c);
  load_vec<8>(cs + half + at, s);
#pragma unroll
  for (int j = 0; j < 8; ++j) o[j] = a[j] * c[j] - b[j] * s[j];
  store_vec<8>(dst + at, o);
#pragma unroll
  for (int j = 0; j < 8; ++j) o[j] = b[j] * c[j] + a[j] * s[j];
  store_vec<8>(dst + half + at, o);
}
