// Argument block shared by the hyper-connection kernel and its binding.
#pragma once

struct HyperArgs {
  float* x;               // [tokens, streams, width]
  const void* rows;       // [tokens, width] of what is pending, or null
  const void* experts;    // [tokens * top, width] in expert order, or null
  const int* inv;         // [tokens, top] pair -> expert row, negative: `self`;
                          //   null: no experts
  const float* weights;   // [tokens, top]
  const void* self;       // [tokens, width], or null
  const float* conn;      // [streams * streams | streams] = mix[from, to], out
                          //   of the pending sublayer; null: nothing pending
  const float* read;      // [streams] what the next sublayer reads
  const float* w;         // [width] norm weight, or null: no norm
  const float* b;         // [width]
  const float* alpha;     // [1]
  void* out;              // [tokens, width]
  int tokens, streams, width, top;
  float mult;             // of what is pending, beside out
};
