// Argument blocks shared by the latent-attention kernels and their bindings.
#pragma once

struct AttnRowsArgs {
  const void* q;          // + row*q_row + head*q_head
  const void* k;          // + key_row*k_row + head*k_head
  const void* v;          // + key_row*v_row + head*v_head
  const void* gate;       // null, or + row*g_row + head*dv: times sigmoid
  void* out;              // + row*o_row + head*o_head
  const int* row_info;    // contiguous: [rows, 2] = key row of position
                          //   offset 0, offset of the query
  const int* tables;      // paged: [rows, max_pages]
  const int* ctx;         // paged: [rows] tokens visible incl. this one
  long q_row, q_head, k_row, k_head, v_row, v_head, g_row, o_row, o_head;
  int rows, heads, d, dv, window, page_size, max_pages;
  float scale;
};

// bf16 only; d, dv and every stride but dv's are multiples of 8
struct WindowAttnArgs {
  const void* q;          // + row*q_row + head*q_head
  const void* k;
  const void* v;
  const void* gate;       // null, or + row*g_row + head*dv
  void* out;              // + row*o_row + head*dv
  const int* blocks;      // [n_blocks, 2] = sequence, first query (of 128)
  const int* seq_info;    // [seqs, 4] = first query row, queries, first key
                          //   row, offset of the first query among the keys
  long q_row, q_head, k_row, k_head, v_row, v_head, g_row, o_row;
  int n_blocks, heads, d, dv, window;
  float scale;
};

// bf16 only; rank and the q strides are multiples of 8, page_size of 16
struct LatentDecodeArgs {
  const void* q;          // + seq*q_row + head*q_head, rank elements
  const void* cache;      // [pages, page_size, rank]
  const int* tables;      // [seqs, max_pages]
  const int* ctx;         // [seqs] tokens visible incl. this one
  void* out;              // [seqs, heads, rank]
  float* part_o;          // [splits, seqs, heads, rank]   (splits > 1)
  float* part_ml;         // [splits, seqs, heads, 2]
  long q_row, q_head;
  int seqs, heads, rank, window, page_size, max_pages, splits;
  float scale;
};

// out[s, h*n + j] = sum_k x[s, h, k] w[h, j, k], times sigmoid(gate)
struct HeadLinearArgs {
  const void* x;          // + s*x_row + h*x_head
  const void* w;          // [heads, n, k]
  const void* gate;       // null, or + s*g_row + h*n
  void* out;              // + s*o_row + h*n
  long x_row, x_head, g_row, o_row;
  int rows, heads, n, k;
  int pack;               // out (and gate) allow 8-byte accesses
};
