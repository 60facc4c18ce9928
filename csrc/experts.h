// Shared by the experts' kernels (csrc/experts.hip) and the tiled GEMM's grouped form (csrc/wide_gemm.hip).
#pragma once
#include <hip/hip_runtime.h>

// (token, choice) pairs in the order of their experts, in tiles of one expert each; everything is on the device
struct GroupedRows {
  int* order;  // pairs
  int* tile_expert; int* tile_first; int* tile_rows;  // tile i: rows order[tile_first[i]] .. of that expert
  int* n_tiles;
  int max_tiles;
  int row_div;  // row of x = pair / row_div
};

__device__ inline float clamped_glu(float gate, float up, float limit) {
  const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
  return g / (1.f + __builtin_amdgcn_exp2f(-1.702f * 1.4426950408889634f * g)) * (u + 1.f);
}
