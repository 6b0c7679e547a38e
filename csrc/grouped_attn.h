// Launch arguments of grouped attention (grouped_attn.hip, grouped_prefill.hip).
#pragma once
#include <hip/hip_runtime.h>

struct GroupedArgs {
  void* out;              // [tokens, H, v], tokens out_stride apart
  float* part;            // [n_split, rows, v]
  float2* part_ml;        // [n_split, rows]
  const void* q;          // [tokens, H, d], tokens q_stride apart
  const void* k_cache;    // [slots, G, d]
  const void* v_cache;    // [slots, G, v]
  const float* sink;      // [H] or null
  const float* bias;      // [H, n_bias] by distance, the last for all larger ones; or null
  const float* talk;      // [H, H] or null: head h's scores are sum_g talk[h, g] * head g's
  const void* gate;       // [tokens, H] before its sigmoid, gate_stride apart; or null
  const int* tables;      // [seqs, max_blocks]
  const int* seq_lens;    // [seqs] cached tokens, this step's included
  const int* ctx_lens;    // [seqs] before this step; null: seq_len - 1 (decode)
  const int* row_starts;  // [seqs] first token row; null: seq
  const int* tile_seq;    // [tiles]; null: decode, one token per sequence
  const int* tile_q0;     // [tiles] first token of the tile within the chunk
  int64_t q_stride, out_stride, gate_stride;
  int H, G, n_tiles, max_blocks, kv_block, window, keep, n_split, rows, n_bias;
  int chunk;              // only keys of the query's own chunk; 2^30: all
  float scale, cap;       // cap 0: none
  bool sigmoid;           // weights sigmoid(score), not a softmax
};

#ifdef __HIPCC__
// first key that position pos sees beyond the kept ones
static inline __device__ int first_key(const GroupedArgs& a, int pos) {
  return max(max(0, pos - a.window + 1), pos - pos % a.chunk);
}
#endif
