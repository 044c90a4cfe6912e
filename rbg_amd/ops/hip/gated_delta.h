// Scalar parts of the gated delta rule, for its decode and prompt kernels.
#pragma once
#include "gated_args.h"
#include "vec_io.h"

// log(1 + e^x) to a few units in the last place, also where it is tiny
DEV_INLINE float softplus_f(float x) {
  const float e = __expf(-fabsf(x)), u = 1.f + e;
  // log(1 + e) = e * log(u) / (u - 1): the rounding of u cancels
  const float l = u == 1.f ? e : e * __logf(u) * rcp_f(u - 1.f);
  return fmaxf(x, 0.f) + l;
}

// log of the factor that a token puts on the state
DEV_INLINE float log_decay(float logit, float bias, float rate) {
  return -rate * softplus_f(logit + bias);
}
