// f32 residual stream of designs that gate and scale each branch by the layer's
// input:
//     x += sum over branches of (y + bias) * scale * sigmoid(logits + gate_bias)
//     out = rms(x) * w              w per coordinate, or one number
// in one pass, where y is a row of the branch's output or the weighed sum of a
// token's expert rows.  One workgroup per token; the row stays in registers.
#include "expert_rows.h"
#include "gated_args.h"

namespace {

constexpr int NT = 256, NW = NT / 64;

// IT * NT * V >= width
template <typename T, int V, int IT>
__global__ __launch_bounds__(NT) void gate_norm_kernel(const GateNormArgs p) {
  __shared__ float red[NW];
  const size_t token = blockIdx.x, base = token * p.width;
  float xr[IT][V], ss = 0.f;
#pragma unroll
  for (int k = 0; k < IT; ++k) {
    const int i = (k * NT + threadIdx.x) * V;
    if (i >= p.width) continue;
    load_vec<V>(p.x + base + i, xr[k]);
    bool any = false;
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const GateBranch& br = p.branch[b];
      if (br.rows == nullptr) continue;
      any = true;
      float y[V], z[V], c[V];
      branch_row<T, V>((const T*)br.rows, br.inv, br.weights, br.top, token,
                       p.width, i, y);
      load_vec<V>((const T*)br.logits + token * br.logit_row + i, z);
      load_vec<V>(br.gate_bias + i, c);
#pragma unroll
      for (int j = 0; j < V; ++j) z[j] = sigmoid_f(z[j] + c[j]);
      if (br.bias != nullptr) {
        load_vec<V>(br.bias + i, c);
#pragma unroll
        for (int j = 0; j < V; ++j) y[j] += c[j];
      }
      load_vec<V>(br.scale + i, c);
#pragma unroll
      for (int j = 0; j < V; ++j) xr[k][j] += y[j] * c[j] * z[j];
    }
    if (any) store_vec<V>(p.x + base + i, xr[k]);
#pragma unroll
    for (int j = 0; j < V; ++j) ss += xr[k][j] * xr[k][j];
  }
  if (p.w == nullptr) return;
  const float sc = 1.f / sqrtf(block_sum<NW>(ss, red) / p.width + p.eps);
#pragma unroll
  for (int k = 0; k < IT; ++k) {
    const int i = (k * NT + threadIdx.x) * V;
    if (i >= p.width) continue;
    float g[V];
    if (p.w_step) {
      load_vec<V>(p.w + i, g);
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) g[j] = p.w[0];
    }
#pragma unroll
    for (int j = 0; j < V; ++j) g[j] *= xr[k][j] * sc;
    store_vec<V>((T*)p.out + base + i, g);
  }
}

template <typename T, int V>
void gate_norm_v(const GateNormArgs& p, hipStream_t s) {
#define GN_GO(IT) gate_norm_kernel<T, V, IT><<<p.tokens, NT, 0, s>>>(p)
  const int it = (p.width + NT * V - 1) / (NT * V);
  if (it <= 1) GN_GO(1);
  else if (it <= 2) GN_GO(2);
  else if (it <= 4) GN_GO(4);
  else GN_GO(8);
#undef GN_GO
}

}  // namespace

extern "C" {

// widest row: 8 steps of a workgroup
int gate_norm_max_width(int vec) { return vec ? NT * 64 : NT * 8; }

void launch_gate_norm(const GateNormArgs* p, int f32, int vec, hipStream_t s) {
  if (f32) {
    if (vec) gate_norm_v<float, 8>(*p, s);
    else gate_norm_v<float, 1>(*p, s);
  } else {
    if (vec) gate_norm_v<__hip_bfloat16, 8>(*p, s);
    else gate_norm_v<__hip_bfloat16, 1>(*p, s);
  }
}

}  // extern "C"
