// Launch arguments of the latent attention kernels (latent_attn.hip).
#pragma once
#include <hip/hip_runtime.h>

struct LatentArgs {
  void* out;              // [rows, rank] when n_split == 1
  float* part;            // [n_split, rows, rank]
  float2* part_ml;        // [n_split, rows]
  const void* q;          // [rows, row]
  const void* cache;      // [slots, row]
  const int* tables;      // [seqs, max_blocks]
  const int* seq_lens;    // [seqs] cached tokens, this step's included
  const int* ctx_lens;    // [seqs] before this step; null: seq_len - 1 (decode)
  const int* row_starts;  // [seqs] first token row; null: seq
  const int* tile_seq;    // [tiles]; null: decode, tile -> (seq, part of heads)
  const int* tile_r0;     // [tiles] first flattened row within the sequence
  int H, max_blocks, kv_block, window, n_split, rows;
  float scale;
};
