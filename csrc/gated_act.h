// The gated unit of gated_act.hip and experts.hip.
#pragma once
#include "common_t.h"

// g * sigmoid(alpha (g + cubic g^3)) * (u + offset), g capped at limit, u at +-limit
DEV float clamped_glu_f(float g, float u, float limit, float alpha, float offset, float cubic) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  float z = alpha * g;
  if (cubic != 0.f) z *= 1.f + cubic * g * g;
  return g * sigmoid_f(z) * (u + offset);
}
