// Typed row access of the kernels that exist for 16-bit AND 32-bit models: storage type T is uint16_t (bf16 bits) or
// float; arithmetic is fp32 either way.
#pragma once
#include "common.h"

namespace mi {
namespace {

template <typename T>
struct Io;

template <>
struct Io<uint16_t> {
  using E = Elem<bf16_tag>;
  static __device__ __forceinline__ float ld(const uint16_t* p) { return E::from_bits(*p); }
  static __device__ __forceinline__ void st(uint16_t* p, float v) { *p = E::to_bits(v); }
  template <int VEC>
  static __device__ __forceinline__ void ldv(const uint16_t* p, float (&v)[VEC]) {
    if constexpr (VEC == 8) {
      const uint4 w = *reinterpret_cast<const uint4*>(p);
      const uint32_t a[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
      for (int i = 0; i < 4; ++i) v[2 * i] = E::lo(a[i]), v[2 * i + 1] = E::hi(a[i]);
    } else {
#pragma unroll
      for (int i = 0; i < VEC; ++i) v[i] = E::from_bits(p[i]);
    }
  }
  template <int VEC>
  static __device__ __forceinline__ void stv(uint16_t* p, const float (&v)[VEC]) {
    if constexpr (VEC == 8) {
      *reinterpret_cast<uint4*>(p) =
          make_uint4(E::pack(v[0], v[1]), E::pack(v[2], v[3]), E::pack(v[4], v[5]), E::pack(v[6], v[7]));
    } else {
#pragma unroll
      for (int i = 0; i < VEC; ++i) p[i] = E::to_bits(v[i]);
    }
  }
};

template <>
struct Io<float> {
  static __device__ __forceinline__ float ld(const float* p) { return *p; }
  static __device__ __forceinline__ void st(float* p, float v) { *p = v; }
  template <int VEC>
  static __device__ __forceinline__ void ldv(const float* p, float (&v)[VEC]) {
    if constexpr (VEC == 8) {
      const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
      v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w, v[4] = b.x, v[5] = b.y, v[6] = b.z, v[7] = b.w;
    } else {
#pragma unroll
      for (int i = 0; i < VEC; ++i) v[i] = p[i];
    }
  }
  template <int VEC>
  static __device__ __forceinline__ void stv(float* p, const float (&v)[VEC]) {
    if constexpr (VEC == 8) {
      reinterpret_cast<float4*>(p)[0] = make_float4(v[0], v[1], v[2], v[3]);
      reinterpret_cast<float4*>(p)[1] = make_float4(v[4], v[5], v[6], v[7]);
    } else {
#pragma unroll
      for (int i = 0; i < VEC; ++i) p[i] = v[i];
    }
  }
};

// sum over a workgroup of at most 16 waves; every thread gets it
__device__ __forceinline__ float wg_sum(float v, float* smem) {
  v = wave_allreduce_sum(v);
  const int nw = blockDim.x >> 6;
  if (nw == 1) return v;
  if ((threadIdx.x & 63) == 0) smem[threadIdx.x >> 6] = v;
  __syncthreads();
  float r = 0.f;
  for (int i = 0; i < nw; ++i) r += smem[i];
  __syncthreads();
  return r;
}

__device__ __forceinline__ float inv_rms(float ss, int n, float eps) { return 1.0f / sqrtf(ss / (float)n + eps); }
__device__ __forceinline__ float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float silu_f(float x) { return x * sigmoid_f(x); }
__device__ __forceinline__ float softplus_f(float x) { return log1pf(expf(-fabsf(x))) + fmaxf(x, 0.f); }

// request of flat row t: the r with qsl[r] <= t < qsl[r + 1]
__device__ __forceinline__ int row_request(const int32_t* qsl, int n, int t) {
  int lo = 0, hi = n - 1;
  while (lo < hi) {
    const int mid = (lo + hi + 1) >> 1;
    if (qsl[mid] <= t) lo = mid;
    else hi = mid - 1;
  }
  return lo;
}

inline bool aligned16(const void* p) { return ((uintptr_t)p & 15) == 0; }

}  // namespace
}  // namespace mi
