// Launch arguments of the latent attention kernels: absorbed (latent_attn.hip)
// and expanded (latent_prefill.hip).
#pragma once
#include <hip/hip_runtime.h>

struct LatentArgs {
  void* out;              // [rows, rank] when n_split == 1
  float* part;            // [n_split, rows, rank]
  float2* part_ml;        // [n_split, rows]
  const void* q;          // [rows, rank] absorbed queries
  const void* q_rot;      // [tokens, H, rot] not yet rotated, strides below
  const float* cos_sin;   // [2, positions, rot_dim / 2]
  const void* cache;      // [slots, row]
  const float* sink;      // [H] or null
  const int* tables;      // [seqs, max_blocks]
  const int* seq_lens;    // [seqs] cached tokens, this step's included
  const int* ctx_lens;    // [seqs] before this step; null: seq_len - 1 (decode)
  const int* row_starts;  // [seqs] first token row; null: seq
  const int* tile_seq;    // [tiles]; null: decode, tile -> (seq, part of heads)
  const int* tile_r0;     // [tiles] first flattened row within the sequence
  int64_t rot_token, rot_head, positions;
  int rot_dim;
  int H, max_blocks, kv_block, window, n_split, rows;
  float scale;
};

struct LatentPrefillArgs {
  void* out;              // [tokens, H * v], rows out_stride apart
  const void* q;          // [tokens, H, d + rot], rows q_stride apart, not rotated
  const void* kv;         // [keys, H * d | H * v], rows kv_stride apart
  const void* k_rot;      // [keys, rot], rows rot_stride apart
  const void* gate;       // [tokens, H], rows gate_stride apart, or null
  const float* sink;      // [H] or null
  const float* cos_sin;   // [2, positions, rot_dim / 2]
  const int *seq_lens, *ctx_lens, *row_starts, *tile_seq, *tile_q0;
  const int* key_first;   // [seqs] position of a sequence's first key row
  const int* key_starts;  // [seqs] that row
  int64_t out_stride, q_stride, kv_stride, rot_stride, gate_stride, positions;
  int H, n_tiles, rot_dim, window;
  float scale;
};

// Where merged rows go: row r is head r % H of token r / H.
struct SplitOut {
  void* out;              // bf16, tokens out_stride apart
  const void* gate;       // [tokens, H] bf16 before its sigmoid, or null
  int64_t out_stride, gate_stride;
  int H;
  bool sum;               // partial results are summed as they are, no softmax
};

// bf16 rows of ``width`` from n_split (at most 64) partial sums [n_split, rows, width]
// with their (maximum in the exp2 domain, sum) [n_split, rows]; an empty split has sum
// -1 and is one of a row's last
extern "C" void launch_split_combine(const SplitOut* out, const float* part,
                                     const float2* part_ml, int rows, int width, int n_split,
                                     hipStream_t stream);
