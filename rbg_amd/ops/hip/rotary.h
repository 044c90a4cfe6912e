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
