// Argument blocks shared by the paged-attention kernels and their bindings.
#pragma once

struct PagedAttnArgs {
  const void* q;          // + row*q_row + head*q_head
  const void* k;          // [pages, kv_heads, page_size, maps*d]
  const void* v;          // [pages, kv_heads, page_size, dv]
  void* out;              // + row*o_row + head*dv
  const int* tables;      // [seqs, max_pages]
  const int* ctx;         // decode: [seqs] tokens visible incl. this one
  const int* seq_info;    // prompts: [seqs, 3] = first row, rows, position of
                          //   the first
  const int* row_info;    // prompts: [rows, 2] = sequence, position
  const int* blocks;      // prompts: [n_blocks, 2] = sequence, first query
  float* part_o;          // decode: [splits, seqs, heads*maps, dv] when
  float* part_ml;         //         splits > 1 or maps == 2; [.., 2]
  const float* lam;       // maps == 2: [1] what the second map counts
  long q_row, q_head, o_row;
  int rows, heads, kv_heads, d, dv, page_size, max_pages, n_blocks, splits;
  int page_shift;         // log2(page_size); prompt and decode forms only
  float scale, softcap;   // softcap 0: none
  int sink;               // one key of score 0 without a value
  int window;             // keys seen, this one included; 0: all before
  int maps;               // 2: a head's q and k are two of size d, and its
                          //   output (o1 - lam o2) / rms * out_scale
  float out_scale, out_eps;
};

struct RopePagedArgs {
  void* proj;             // [rows, stride]
  const float* bias;      // [width], or null
  const float* cos_sin;   // [positions, rot] = [cos | sin]; null: rot is 0
  const int* positions;   // [rows]
  const int* slots;       // [rows]
  void* k;                // [pages, kv_heads, page_size, d], or null
  void* v;                // [pages, kv_heads, page_size, dv]
  long stride;
  int off_q, off_k, off_v;
  int rows, heads, kv_heads, d, dv, rot, page_size, table_rows;
};
