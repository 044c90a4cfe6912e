// Argument blocks shared by the token-mixer kernels and their bindings.
#pragma once

struct DeltaArgs {
  const void* proj;       // [rows, proj_stride]; column offsets below
  const void* z;          // [rows, heads*dim] or null: from low/w2
  const void* w2;         // [heads*dim, rank]
  const float* w0;        // [heads*dim]
  const float* a_bias;    // [heads*dim]
  const float* norm_w;    // [heads*dim]
  float* state;           // [slots, heads, dim, dim]
  const int* slots;       // [seqs]
  const int* cu;          // [seqs+1] rows, or null: one row per sequence
  const int* starts;      // [seqs] position of the first row
  void* out;              // [rows, out_stride]
  long proj_stride, out_stride;
  int off_r, off_k, off_v, off_a, off_g, off_low;
  int heads, dim, rank;
  float decay_scale, unit_eps, norm_eps;
};
