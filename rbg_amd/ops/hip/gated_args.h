// Argument blocks of the gated-delta, short-convolution and gated-norm kernels
// and their bindings.
#pragma once

struct ShortConvArgs {
  const void* x;          // [rows, x_row]
  const float* w;         // [taps, width]; the last one is the current token's
  void* ring;             // [slots, taps, width]: input of position p at p % taps
  void* out;              // [rows, width]
  const int* tiles;       // [n_tiles, 2] = sequence, first token
  const int* cu;          // [seqs+1] rows
  const int* starts;      // [seqs] position of the first row
  const int* slots;       // [seqs]
  long x_row;
  int n_tiles, tile, width, taps;
};

struct GatedDeltaArgs {
  const void* qkv;        // + row*qkv_row; q, k [kv_heads, dim], v [heads, vdim]
  const void* beta;       // + row*beta_row, one logit per head
  const void* decay;      // + row*decay_row, logits per head (and key channel)
  const void* gate;       // + row*gate_row, heads x vdim
  const float* a_log;     // [heads]
  const float* dt_bias;   // [heads] or [heads*dim]
  const float* norm_w;    // [vdim]
  float* state;           // [slots, heads, dim, vdim]
  const int* slots;       // [seqs]
  const int* cu;          // [seqs+1] rows, or null: one row per sequence
  const int* starts;      // [seqs] position of the first row
  void* out;              // + row*out_row, heads x vdim
  // not null: qkv holds the inputs of a short convolution with silu, whose
  // channels are counted from off_q on
  const float* conv_w;    // [taps, channels]
  void* ring;             // [slots, taps, channels]
  long qkv_row, beta_row, decay_row, gate_row, out_row;
  int off_q, off_k, off_v;
  int heads, kv_heads, dim, vdim, taps, channels;
  int per_channel;        // decay per key channel
  int silu;               // output gate: silu, else sigmoid
  float q_scale, unit_eps, norm_eps;
};

// one branch that a layer left to be added to the stream
struct GateBranch {
  const void* rows;       // [tokens, width], or expert rows; null: no branch
  const int* inv;         // expert rows: [tokens, top] pair -> row
  const float* weights;   //              [tokens, top]
  const void* logits;     // + token*logit_row: the gate's logits
  const float* gate_bias; // [width]
  const float* scale;     // [width]
  const float* bias;      // [width] added to the rows, or null
  long logit_row;
  int top;
};

struct GateNormArgs {
  float* x;               // [tokens, width]
  GateBranch branch[2];
  const float* w;         // norm weight, w_step apart; null: no norm
  void* out;              // [tokens, width]
  int tokens, width, w_step;
  float eps;
};
