// Launch arguments of attention_inputs (attn_inputs.hip).
#pragma once
#include <hip/hip_runtime.h>

struct AttnInputsArgs {
  void* q;                // [N, H, d]
  void* k_cache;          // [slots, G, d]
  void* v_cache;          // [slots, G, v]
  const void* proj;       // [N, C] rows stride apart, C = (H + G) d + G v
  const void* conv;       // [taps, C] or null
  void* ring;             // [state slots, taps, C]: input of position p at p % taps
  const void* q_norm;     // [d] (row_norm: [H d]) or null: no norm of q and k
  const void* k_norm;     // [d] (row_norm: [G d])
  const float* head_mult; // [H] or null
  const float* cos_sin;   // [2, P, pairs] or null
  const int64_t* positions;
  const int64_t* slots;
  const int* back;        // [N] rows of the same sequence right before a row; null: 0
  const int* states;      // [N] state slot of a row
  const int* ring_rows;   // rows whose inputs join the ring in a launch of their own
  int64_t stride, P;
  int N, H, G, d, v, dim, vdim, C, taps, pairs, n_ring_rows;
  float eps, q_coef, q_every;  // q_every 0: no temperature
  bool v_norm, write_ring;     // write_ring: every row is its sequence's only one
  bool row_norm;               // q and k are normed over all their heads at once
};
