// Parameters shared by the kernels of the gated delta rule.
#pragma once
#include "row_io.h"

namespace mi {
namespace {

struct DeltaParams {
  const void* proj;      // [rows][ld]: q (K D) | k (K D) | v (H V)
  const void* gate;      // [rows][ld_gate]: H V
  const void* b;         // [rows][ld_b]: H
  const void* a;         // [rows][ld_a]: H, or H D with one decay per key channel
  const void* convw;     // [CH][taps], CH = 2 K D + H V
  const void* norm_w;    // [V]
  void* ring;            // [slots][taps][CH]
  void* out;             // [rows][ld_out], columns H V
  const float* a_log;    // [H]
  const float* dt_bias;  // [H], or [H D]
  float* state;          // [slots][H][D][V]
  const int32_t* slots;
  const int32_t* qsl;
  const int32_t* seq_lens;
  int64_t ld, ld_gate, ld_b, ld_a, ld_out;
  int req0;
  int H, K, D, V, taps, CH;
  int channel;           // one decay per head and key channel instead of one per head
  int sigmoid_gate;      // the output gate is sigmoid(gate) instead of silu(gate)
  float eps;
};

__device__ __forceinline__ float out_gate(const DeltaParams& p, float g) { return p.sigmoid_gate ? sigmoid_f(g) : silu_f(g); }

inline int delta_fill(DeltaParams& p, const mi_gated_delta_args* a) {
  if (!a || !a->qkv || !a->gate || !a->beta || !a->decay || !a->conv_w || !a->a_log || !a->dt_bias || !a->norm_w || !a->state ||
      !a->ring || !a->slots || !a->query_start_loc || !a->seq_lens || !a->out)
    return MI_ERR_INVALID_ARG;
  const int H = a->heads, K = a->kv_heads, D = a->dim, V = a->vdim;
  if (a->req0 < 0 || a->num_reqs < 0 || H <= 0 || K <= 0 || D <= 0 || V <= 0 || a->taps <= 0 || H % K) return MI_ERR_INVALID_ARG;
  const int CH = 2 * K * D + H * V;
  if (a->qkv_stride < CH || a->gate_stride < H * V || a->beta_stride < H || a->out_stride < H * V ||
      a->decay_stride < (a->channel_decay ? H * D : H))
    return MI_ERR_INVALID_ARG;
  p = DeltaParams{a->qkv, a->gate, a->beta, a->decay, a->conv_w, a->norm_w, a->ring, a->out, a->a_log, a->dt_bias, a->state,
                  a->slots, a->query_start_loc, a->seq_lens, a->qkv_stride, a->gate_stride, a->beta_stride, a->decay_stride,
                  a->out_stride, a->req0, H, K, D, V, a->taps, CH, a->channel_decay != 0, a->sigmoid_gate != 0, a->eps};
  return MI_OK;
}

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
