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

// An expert's gate: g = min(gate, limit), u = clamp(up, -limit, limit), g sigmoid(slope g) (u + shift).  Clamped experts have slope 1.702
// and shift 1, silu-gated ones (silu(gate) up) no limit, slope 1 and shift 0.
struct ExpertGate { float limit, slope, shift; };

__device__ inline float expert_gate(float gate, float up, ExpertGate p) {
  const float g = fminf(gate, p.limit), u = fminf(fmaxf(up, -p.limit), p.limit);
  return g / (1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * p.slope * g)) * (u + p.shift);
}
