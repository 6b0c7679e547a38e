// Launch arguments of the gated delta rule (gated_delta.hip).
#pragma once
#include <hip/hip_runtime.h>

struct DeltaArgs {
  // inputs by token row, in the model's dtype; q | k | v channels, C = 2 G D + H V
  const void* qkv;        // [N, C] before the convolution
  const void* conv;       // [C, taps]
  const void* b;          // [N, H]
  const void* z;          // [N, H * D], or [N, H] with head_decay
  const void* gate;       // [N, H * V]
  const float* A_log;     // [H]
  const float* dt_bias;   // like a row of z
  const float* norm;      // [V]
  float* state;           // [slots, H, D, V]
  void* ring;             // [slots, taps, C]: input of position p at p % taps
  void* out;              // [N, H * V]
  // workspace of the prompt kernels
  void* y;                // [N, C] convolved
  float* unit;            // [N, G, 3] factors that make q and k unit vectors, then q . k
  float* g;               // [N, H * D] decays; null with head_decay
  float* o;               // [N, H, V] before the norm
  const int* seq_lens;    // [seqs] tokens including this step's
  const int* ctx_lens;    // [seqs] before this step; null: decode
  const int* row_starts;  // [seqs]
  const int* slots;       // [seqs]
  const int* tile_seq;    // [tiles]
  const int* tile_q0;     // [tiles]
  int64_t qkv_stride, b_stride, z_stride, gate_stride;
  int H, G, D, V, C, taps, N, seqs, n_tiles;
  float eps, unit_eps, q_scale;
  bool head_decay;        // one decay per head
  bool gate_silu;         // gate silu(x), else sigmoid(x)
};
