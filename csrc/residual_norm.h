// How residual_norm (residual_norm.hip) treats the residual.
#pragma once
#include <stdint.h>

// partial sums a depth block prepares for its later layers
#define DEPTH_AHEAD 3

struct NormForm {
  bool center;              // layer norm of x, else RMS norm
  float offset;             // added to both norm weights
  float mult;               // on what is added to x
  // sum_j weights[n, j] * rows[n, j] joins y
  int top;                  // 0 = none
  const void* rows;         // [n, top, w]
  const float* weights;     // [n, top]
  // and then sigmoid(gate[n]) multiplies y
  const void* gate;         // [n, w] rows gate_stride apart, or null
  int64_t gate_stride;
  // the same norm of x under another weight
  const void* x_norm2;      // [w]
  void* out2;               // rows out2_stride apart, or null
  int64_t out2_stride;
  // depth average: x becomes state n_states - 1 and then sum_j coef[j] * state_j
  int n_states;             // 0 = none
  int first;                // states before it are in partial[ready]; 0: none are
  int ready;
  int ahead;                // sums over the n_states for the next layers, coefficients
                            // in the rows after coef's: partial[0 .. ahead - 1]
  float* states;            // [.., n, w]
  float* partial;           // [DEPTH_AHEAD, n, w]
  const float* coef;
  int64_t coef_stride, plane;  // plane = n * w
};
