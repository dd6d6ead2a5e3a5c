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

// the last rows of every request's portion into its ring, after every reader of the rows they replace
template <typename T>
__global__ __launch_bounds__(256) void conv_ring_update_kernel(const DeltaParams p) {
  scalar_cache_acquire();
  const int r = p.req0 + blockIdx.y;
  const int s0 = p.qsl[r], L = p.qsl[r + 1] - s0;
  const int ch = blockIdx.x * 256 + threadIdx.x;
  // (a one-token portion through the step kernel has left its row there already: the same values again)
  if (L <= 0 || ch >= p.CH) return;
  const int start = p.seq_lens[r] - L;
  T* ring = reinterpret_cast<T*>(p.ring) + (int64_t)p.slots[r] * p.taps * p.CH;
  const T* proj = reinterpret_cast<const T*>(p.proj);
  for (int i = max(0, L - p.taps); i < L; ++i)
    if (start + i >= 0) ring[(int64_t)((start + i) % p.taps) * p.CH + ch] = proj[(s0 + i) * p.ld + ch];
}

}  // namespace
}  // namespace mi
