// Argument blocks shared by the latent-attention kernels and their bindings.
#pragma once

// Rotary positions: pair i of the rotated dims is (2i, 2i + 1) when interleaved,
// else (i, i + dims / 2).
struct RotaryArgs {
  const float* cos_sin;   // [table_rows, dims] = [cos | sin]
  const int* positions;   // [rows]
  int dims;               // 0: nothing rotates
  int interleaved, table_rows;
};

struct LatentStoreArgs {
  const void* x;          // + row*x_row: rank latent columns, then rot.dims
  const float* w;         // [rank]
  void* c;                // [rows, rank + rot.dims]
  void* cache;            // [.., rank + rot.dims]
  const int* slots;       // [rows]
  const void* x2;         // null, or + row*x2_row: normed under w2 into c2
  const float* w2;        // [rank2]
  void* c2;               // [rows, rank2]
  RotaryArgs rot;
  long x_row, x2_row;
  int rows, rank, rank2;
  float eps;
};

// in place
struct RotateArgs {
  void* x;                // + row*x_row + head*x_head, rot.dims elements
  RotaryArgs rot;
  long x_row, x_head;
  int rows, heads;
};

struct AttnRowsArgs {
  const void* q;          // + row*q_row + head*q_head
  const void* k;          // + key_row*k_row + head*k_head
  const void* k2;         // null, or + key_row*k2_row: dims d1.. of every head
  const void* v;          // + key_row*v_row + head*v_head
  const float* sink;      // null, or [heads]: a logit without key or value
  const void* gate;       // null, or + row*g_row + head*dv: times sigmoid
  void* out;              // + row*o_row + head*o_head
  const int* row_info;    // contiguous: [rows, 2] = key row of position
                          //   offset 0, offset of the query
  const int* tables;      // paged: [rows, max_pages]
  const int* ctx;         // paged: [rows] tokens visible incl. this one
  long q_row, q_head, k_row, k_head, k2_row, v_row, v_head, g_row, o_row,
      o_head;
  int rows, heads, d, d1, dv, window, page_size, max_pages;
  float scale;
};

// bf16 only; d, d1, dv and every stride but dv's are multiples of 8
struct WindowAttnArgs {
  const void* q;          // + row*q_row + head*q_head
  const void* k;
  const void* k2;         // null, or + key_row*k2_row: dims d1.. of every head
  const void* v;
  const float* sink;      // null, or [heads]: a logit without key or value
  const void* gate;       // null, or + row*g_row + head*dv
  void* out;              // + row*o_row + head*dv
  const int* blocks;      // [n_blocks, 2] = sequence, first query (of 128)
  const int* seq_info;    // [seqs, 4] = first query row, queries, first key
                          //   row, offset of the first query among the keys
  long q_row, q_head, k_row, k_head, k2_row, v_row, v_head, g_row, o_row;
  int n_blocks, heads, d, d1, dv, window;
  float scale;
};

// bf16 only; d, rank and the q strides are multiples of 8, page_size of 16
struct LatentDecodeArgs {
  const void* q;          // + seq*q_row + head*q_head, d elements
  const void* cache;      // [pages, page_size, d]; the first rank are the value
  const float* sink;      // null, or [heads]: a logit without key or value
  const int* tables;      // [seqs, max_pages]
  const int* ctx;         // [seqs] tokens visible incl. this one
  void* out;              // [seqs, heads, rank]
  float* part_o;          // [splits, seqs, heads, rank]   (splits > 1)
  float* part_ml;         // [splits, seqs, heads, 2]
  long q_row, q_head;
  int seqs, heads, d, rank, window, page_size, max_pages, splits;
  float scale;
};

// out[s, h, j] = sum_k x[s, h, k] w[h, j, k], times sigmoid(gate); behind a
// head's n columns follow the rotated dims of tail
struct HeadLinearArgs {
  const void* x;          // + s*x_row + h*x_head
  const void* w;          // [heads, n, k]
  const void* gate;       // null, or + s*g_row + h*n
  const void* tail;       // + s*t_row + h*t_head, rot.dims elements
  void* out;              // + s*o_row + h*o_head
  RotaryArgs rot;
  long x_row, x_head, g_row, t_row, t_head, o_row, o_head;
  int rows, heads, n, k;
  int pack;               // out (and gate) allow 8-byte accesses
  int tail_vec;           // tail and its place in out allow 16-byte accesses
};
