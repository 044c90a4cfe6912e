// Argument blocks shared by the expert kernels and their bindings.
#pragma once

struct MoeRouteArgs {
  const float* logits;    // [tokens, experts]
  const float* correction;
  float* weights;         // [tokens, top]
  int* ids;               // [tokens, top]
  int* inv;               // [tokens * top] pair -> row
  int* rows;              // [tokens * top] row -> token
  int* tiles;             // [.., 3] = expert, first row, rows
  int* count;             // [1] tiles used
  int* part;              // [blocks, experts] of moe_route_blocks
  int tokens, experts, groups, keep, top, tile;
  int softmax;            // choice by logit + correction, weights by softmax
                          //   over the chosen; else sigmoids
};

struct MoeGemmArgs {
  const void* x;          // [.., k] rows
  const void* w;          // [experts, n, k]
  void* out;              // [pairs, n], swiglu: [pairs, n / 2]
  const int* rows;        // gather: row -> row of x; null: the same
  const int* tiles;
  const int* count;
  int max_tiles, tile, n, k, relu2;
  int swiglu;             // silu(gate) * up; w's rows go gate, gate, up, up
};
