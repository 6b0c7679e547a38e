// How residual_norm (residual_norm.hip) treats the residual.
#pragma once
#include <stdint.h>

struct NormForm {
  bool center;              // layer norm of x, else RMS norm
  float offset;             // added to both norm weights
  float mult;               // on what is added to x
  int n_depth;              // states averaged, the new one included; 0 = none
  float* depth;             // [states, n, w], states depth_stride apart
  const float* depth_coef;  // [n_depth]
  int64_t depth_stride;
};
