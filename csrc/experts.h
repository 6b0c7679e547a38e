// Launch arguments of the mixture-of-experts kernels (experts.hip, experts_gemm.hip).
#pragma once
#include <hip/hip_runtime.h>

// One product of the routed experts.  An entry is a (token, choice) pair, number
// token * top + choice; entries are grouped by expert through perm.
struct ExpertsArgs {
  void* out;            // gate_up: [entries, O] in grouped order; down: [entries, O] by entry
  const void* x;        // gate_up: [tokens, K] rows x_stride apart; down: [entries, K] grouped
  const void* w;        // gate_up: [E, 2 O, K], gate rows then up rows; down: [E, O, K]
  const int* ids;       // [entries] expert
  const int* perm;      // [entries] entry of a grouped row
  const int* offsets;   // [E + 2] first grouped row of an expert; then the tiles in use
  const int* tile_expert;  // [tiles]
  const int* tile_row;     // [tiles] first grouped row of the tile
  int64_t x_stride;
  int entries, E, O, K, top, tiles;
  float limit, alpha, offset, cubic;  // gate_up: the gated unit
};

// rows of one tile of the large-batch product
#define EXPERT_TILE 256
