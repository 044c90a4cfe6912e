// Gated activations shared by the elementwise and the expert kernels.
#pragma once
#include "act_kinds.h"
#include "vec_io.h"

DEV_INLINE float silu_glu_f(float g, float u) { return g * sigmoid_f(g) * u; }

// a gate bounded above and a linear part bounded on both sides and moved by one:
// min(g, limit) sigmoid(1.702 min(g, limit)) (clamp(u, -limit, limit) + 1)
DEV_INLINE float clamped_glu_f(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * sigmoid_f(1.702f * g) * (u + 1.f);
}
