// The ring of a causal filter's inputs: a request's slot keeps the last `taps` input rows, the one of position p in place
// p % taps.  A row's filter reads the taps - 1 rows in front of it, so a step that brings one row may write its own place
// while others still read theirs; portions of several rows write in a launch behind every reader.
#pragma once
#include "row_io.h"

namespace mi {
namespace {

struct ConvInputs {
  const void* x;          // [rows][ld]: the step's inputs
  const void* w;          // [channels][taps], the last tap for the row itself
  void* ring;             // [slots][taps][channels]
  const int32_t* slots;   // per request
  const int32_t* qsl;
  const int32_t* seq_lens;
  int64_t ld;
  int req0, taps, channels;
};

// where the input b >= 1 rows in front of row i of a request's portion lies (position pos = start + i; the row itself where
// there is none: the caller drops the value)
template <typename T>
__device__ __forceinline__ const T* conv_input(const ConvInputs& p, const T* x_row, const T* ring, int i, int pos, int b) {
  const T* src = i >= b ? x_row - b * p.ld : ring + (int64_t)((pos - b) % p.taps) * p.channels;
  return pos >= b ? src : x_row;
}

// four taps of 8 neighbouring channels, the one for the row itself first
template <typename T>
__device__ __forceinline__ void conv_taps4(const T* w, float (&wt)[4][8]) {
#pragma unroll
  for (int m = 0; m < 4; ++m) {
    float v[8];
    Io<T>::template ldv<8>(w + 8 * m, v);
#pragma unroll
    for (int j = 0; j < 8; ++j) wt[3 - j % 4][2 * m + j / 4] = v[j];
  }
}

// the last rows of every request's portion into its ring (a one-row portion's is there already: the same values again)
template <typename T>
__global__ __launch_bounds__(256) void conv_inputs_update_kernel(const ConvInputs p) {
  scalar_cache_acquire();
  const int r = p.req0 + blockIdx.y;
  const int s0 = p.qsl[r], L = p.qsl[r + 1] - s0;
  const int ch = blockIdx.x * 256 + threadIdx.x;
  if (L <= 0 || ch >= p.channels) return;
  const int start = p.seq_lens[r] - L;
  T* ring = reinterpret_cast<T*>(p.ring) + (int64_t)p.slots[r] * p.taps * p.channels;
  const T* x = reinterpret_cast<const T*>(p.x);
  for (int i = max(0, L - p.taps); i < L; ++i)
    if (start + i >= 0) ring[(int64_t)((start + i) % p.taps) * p.channels + ch] = x[(s0 + i) * p.ld + ch];
}

template <typename T>
int launch_conv_update(const ConvInputs& p, int num_reqs, hipStream_t s) {
  hipLaunchKernelGGL((conv_inputs_update_kernel<T>), dim3((p.channels + 255) / 256, num_reqs), dim3(256), 0, s, p);
  return launch_status();
}

}  // namespace
}  // namespace mi
