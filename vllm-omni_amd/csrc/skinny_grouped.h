// Grouped (per-expert) form of the decode-batch linear kernel, shared between skinny_gemm.hip (the kernel) and
// fused_moe.hip (its caller): every workgroup row (grid.y) is one tile of <= 64 token rows that all use ONE expert's
// weight matrix; rows are gathered through the MoE alignment's maps.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

namespace mi {

struct GroupedGemmArgs {
  void* out;                    // [max_rows, n_out]
  const void* a_rows;           // MI_MOE_PLAIN: rows [max_rows, k]; else x [T, k] (row = sorted_pairs[r] / top_k)
  const void* weights;          // [E, (MI_MOE_GATED ? 2 : 1) * n_out, k]
  const int32_t* sorted_pairs;  // [max_rows]: pair index or -1 (padding)
  const int32_t* tile_expert;   // [max_tiles]
  const int32_t* num_tiles;     // [1], device
  const float* pair_weights;    // MI_MOE_RELU_SQUARED: what a pair's row is multiplied by, or nullptr
  int32_t max_tiles, form, n_out, k, top_k, rows_per_tile;
  int64_t a_row_stride, out_row_stride, weight_expert_stride;
  int dtype;
};

// MI_OK, or MI_ERR_UNSUPPORTED when the shape is outside the ring kernel's envelope (the caller then runs its
// direct-from-global kernel).
int launch_grouped_skinny(const GroupedGemmArgs& a, hipStream_t s);

}  // namespace mi
