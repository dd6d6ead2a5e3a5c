// Parameters shared by the kernels of the gated delta rule.
#pragma once
#include "row_io.h"

namespace mi {
namespace {

struct DeltaParams {
  const void* proj;      // [rows][ld]: q (K D) | k (K D) | v (H V) | gate (H V) | b (H) | a (H)
  const void* convw;     // [CH][taps], CH = 2 K D + H V
  const void* norm_w;    // [V]
  void* ring;            // [slots][taps][CH]
  void* out;             // [rows][H V]
  const float* a_log;    // [H]
  const float* dt_bias;  // [H]
  float* state;          // [slots][H][D][V]
  const int32_t* slots;
  const int32_t* qsl;
  const int32_t* seq_lens;
  int64_t ld;
  int req0;
  int H, K, D, V, taps, CH, off_g, off_b, off_a;
  float eps;
};

}  // namespace
}  // namespace mi
