// Argument blocks shared by the expert kernels and their bindings.
#pragma once

// ROUTE_SIGMOID  choice by sigmoid + correction, weights the sigmoids
// ROUTE_CHOSEN   choice by logit + correction, weights the softmax of the chosen
// ROUTE_SHARE    choice by softmax + correction, weights the chosen ones' shares
//                of their own softmax values, times a constant
enum RouteMode { ROUTE_SIGMOID = 0, ROUTE_CHOSEN = 1, ROUTE_SHARE = 2 };

// of a grouped product, on its way out; the gated ones read w's rows as gate,
// gate, up, up
enum ExpertAct { EXPERT_NONE = 0, EXPERT_RELU2 = 1, EXPERT_SILU_GLU = 2,
                 EXPERT_CLAMPED_GLU = 3 };

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
  int real;               // experts with weights; the others return their
                          //   input, and their pairs get no row (inv -1)
  int mode;               // RouteMode
  float scale;            // ROUTE_SHARE: of the weights
};

struct MoeGemmArgs {
  const void* x;          // [.., k] rows
  const void* w;          // [experts, n, k]
  void* out;              // [pairs, n], gated: [pairs, n / 2]
  const int* rows;        // gather: row -> row of x; null: the same
  const int* tiles;
  const int* count;
  int max_tiles, tile, n, k;
  int act;                // ExpertAct
  float limit;            // EXPERT_CLAMPED_GLU
};
