// What attention whose values are its keys does in front of the scores, in one launch: the short causal filter over q and k,
// the value row (k as the filter leaves it), rotary positions on neighbouring pairs, the unweighted norm per head, and the K / V
// cache write.  q's heads and the cache's are `hd` apart, zeros behind a head's own values.
//
// A workgroup has kRows rows of a request (one in decode steps) and as many heads as its lanes hold (LPH lanes a head, VEC channels
// a lane).  The angles of its rows are formed once (positions, angles, sines and cosines in fp32) and shared through LDS.
#include "short_conv.h"

namespace mi {
namespace {

struct ConvRopeParams {
  ConvInputs in;
  void* q_out;
  void* kc;
  void* vc;
  const float* inv_freq;
  const int64_t* slot_mapping;
  int64_t q_stride, block_stride, token_stride, head_stride;
  int H, G, dim, hd, block_size, pairs;
  float eps;
};

constexpr int kRows = 8, kMaxPairs = 256;

template <typename T>
struct alignas(16) Oct {
  T v[8];
};

// what becomes of a row's filtered channels y (a lane has VEC of them, U times): value row, rotation, norm, stores
template <typename T, int LPH, int VEC, int U>
__device__ __forceinline__ void rope_norm_store(const ConvRopeParams& p, float (&y)[U][VEC], const float2* cs, int head, int sub, int64_t row) {
  float ss = 0.f;
#pragma unroll
  for (int u = 0; u < U; ++u)
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += y[u][j] * y[u][j];
#pragma unroll
  for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
  const float inv = inv_rms(ss, p.dim, p.eps);                  // a rotation leaves the mean square as it is
  T *dst, *vdst = nullptr;
  if (head < p.H) {
    dst = reinterpret_cast<T*>(p.q_out) + row * p.q_stride + (int64_t)head * p.hd;
  } else {
    const int64_t slot = p.slot_mapping[row];
    if (slot < 0) return;                                       // whole lane groups: the sums above are done
    const int64_t at = (slot / p.block_size) * p.block_stride + (slot % p.block_size) * p.token_stride + (head - p.H) * p.head_stride;
    dst = reinterpret_cast<T*>(p.kc) + at;
    vdst = reinterpret_cast<T*>(p.vc) + at;
  }
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int c = (sub + u * LPH) * VEC;
    if (c >= p.hd) continue;
    auto put = [&](T* to) {
      if constexpr (VEC == 8) {
        Io<T>::template stv<8>(to + c, y[u]);
      } else {
#pragma unroll
        for (int j = 0; j < VEC; ++j)
          if (c + j < p.hd) Io<T>::st(to + c + j, y[u][j]);
      }
    };
    if (vdst) put(vdst);
#pragma unroll
    for (int j = 0; j < VEC; j += 2) {
      const int k = (c + j) / 2;
      if (k < p.pairs) {
        const float2 a = cs[k];
        const float e = y[u][j], o = y[u][j + 1];
        y[u][j] = e * a.x - o * a.y;
        y[u][j + 1] = o * a.x + e * a.y;
      }
      y[u][j] *= inv;
      y[u][j + 1] *= inv;
    }
    put(dst);
  }
}

// cosines and sines of a workgroup's rows, [rows][pairs] (barrier by the caller)
__device__ __forceinline__ void rope_angles(const ConvRopeParams& p, float2* cs, int rows, int first) {
  for (int k = threadIdx.x; k < rows * p.pairs; k += 256) {
    const int i = k / p.pairs, j = k % p.pairs;
    float s, c;
    sincosf((float)max(first + i, 0) * p.inv_freq[j], &s, &c);
    cs[k] = make_float2(c, s);
  }
}

// four taps, 8 channels a lane, whole heads a multiple of 8: everything a thread's ROWS rows need is on its way before the angles
template <typename T, int LPH, int ROWS>
__global__ __launch_bounds__(256) void conv_rope_cache4_kernel(const ConvRopeParams p) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) float2 cs[];
  const int r = p.in.req0 + blockIdx.y, t0 = blockIdx.x * ROWS;
  const int s0 = p.in.qsl[r], n = p.in.qsl[r + 1] - s0, start = p.in.seq_lens[r] - n;   // start < 0: a padded row of a graph replay
  if (t0 >= n) return;
  const int rows = min(ROWS, n - t0);
  const int head = (blockIdx.z * 256 + threadIdx.x) / LPH, sub = threadIdx.x % LPH, units = p.H + p.G;
  const int c = sub * 8, hh = min(head, units - 1);
  const bool mine = c < p.dim;
  const int64_t at = (int64_t)hh * p.dim + (mine ? c : 0);
  const T* x = reinterpret_cast<const T*>(p.in.x) + (int64_t)(s0 + t0) * p.in.ld;
  T* ring = reinterpret_cast<T*>(p.in.ring) + (int64_t)p.in.slots[r] * 4 * p.in.channels;
  Oct<T> in[ROWS + 3];                     // in[b]: row b - 3 of the workgroup's
#pragma unroll
  for (int b = 1; b <= 3; ++b)
    in[3 - b] = *reinterpret_cast<const Oct<T>*>(conv_input(p.in, x, (const T*)ring, t0, start + t0, b) + at);
#pragma unroll
  for (int i = 0; i < ROWS; ++i) in[3 + i] = *reinterpret_cast<const Oct<T>*>(x + (int64_t)min(i, rows - 1) * p.in.ld + at);
  float wt[4][8];
  conv_taps4<T>(reinterpret_cast<const T*>(p.in.w) + at * 4, wt);
  rope_angles(p, cs, rows, start + t0);
  __syncthreads();
  if (head >= units) return;                                      // whole lane groups leave
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    if (i >= rows) break;
    float y[1][8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      float a = 0.f;
#pragma unroll
      for (int b = 0; b < 4; ++b) a += (i >= b || start + t0 + i >= b ? Io<T>::ld(&in[3 + i - b].v[j]) : 0.f) * wt[b][j];
      y[0][j] = mine ? a : 0.f;
    }
    // the request's only row: its place in the ring is nobody's to read
    if (n == 1 && start >= 0 && mine) *reinterpret_cast<Oct<T>*>(ring + (int64_t)(start % 4) * p.in.channels + at) = in[3];
    rope_norm_store<T, LPH, 8, 1>(p, y, cs + i * p.pairs, head, sub, s0 + t0 + i);
  }
}

// any sizes and taps: inputs read again for every row
template <typename T, int U>
__global__ __launch_bounds__(256) void conv_rope_cache_kernel(const ConvRopeParams p) {
  scalar_cache_acquire();
  constexpr int LPH = 64, VEC = 2;
  extern __shared__ __attribute__((aligned(16))) float2 cs[];
  const int r = p.in.req0 + blockIdx.y, t0 = blockIdx.x * kRows;
  const int s0 = p.in.qsl[r], n = p.in.qsl[r + 1] - s0, start = p.in.seq_lens[r] - n;
  if (t0 >= n) return;
  const int rows = min(kRows, n - t0);
  rope_angles(p, cs, rows, start + t0);
  __syncthreads();
  const int head = (blockIdx.z * 256 + threadIdx.x) / LPH, sub = threadIdx.x % LPH;
  if (head >= p.H + p.G) return;
  const int taps = p.in.taps;
  const T* x = reinterpret_cast<const T*>(p.in.x) + (int64_t)(s0 + t0) * p.in.ld + (int64_t)head * p.dim;
  T* ring = reinterpret_cast<T*>(p.in.ring) + (int64_t)p.in.slots[r] * taps * p.in.channels + (int64_t)head * p.dim;
  const T* w = reinterpret_cast<const T*>(p.in.w) + (int64_t)head * p.dim * taps;
  for (int i = 0; i < rows; ++i, x += p.in.ld) {
    const int pos = start + t0 + i;
    float y[U][VEC];
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        const int c = (sub + u * LPH) * VEC + j;
        y[u][j] = 0.f;
        if (c >= p.dim) continue;
        for (int b = 0; b < taps && b <= pos; ++b)
          y[u][j] += Io<T>::ld((b == 0 ? x : conv_input(p.in, x, (const T*)ring, t0 + i, pos, b)) + c) *
                     Io<T>::ld(w + (int64_t)c * taps + taps - 1 - b);
        if (n == 1 && start >= 0) ring[(int64_t)(pos % taps) * p.in.channels + c] = x[c];
      }
    rope_norm_store<T, LPH, VEC, U>(p, y, cs + i * p.pairs, head, sub, s0 + t0 + i);
  }
}

template <typename T>
int launch_conv_rope(const ConvRopeParams& p, int num_reqs, int max_query_len, bool vec, int update_ring, hipStream_t s) {
  const dim3 block(256);
  const int units = p.H + p.G;
  const size_t lds = (size_t)kRows * (p.pairs > 0 ? p.pairs : 1) * sizeof(float2);
#define MI_CR4(LPH, ROWS)                                                                                                     \
  hipLaunchKernelGGL((conv_rope_cache4_kernel<T, LPH, ROWS>),                                                                 \
                     dim3((max_query_len + ROWS - 1) / ROWS, num_reqs, (units * LPH + 255) / 256), block, lds, s, p)
#define MI_CR(U)                                                                                                              \
  hipLaunchKernelGGL((conv_rope_cache_kernel<T, U>), dim3((max_query_len + kRows - 1) / kRows, num_reqs, (units + 3) / 4), block, lds, s, p)
  if (vec && p.in.taps == 4 && p.hd <= 64) {
    if (max_query_len == 1) MI_CR4(8, 1);
    else MI_CR4(8, kRows);
  } else if (vec && p.in.taps == 4 && p.hd <= 128) {
    if (max_query_len == 1) MI_CR4(16, 1);
    else MI_CR4(16, kRows);
  } else if (p.hd <= 128) {
    MI_CR(1);
  } else if (p.hd <= 1024) {
    MI_CR(8);
  } else {
    return MI_ERR_UNSUPPORTED;
  }
#undef MI_CR4
#undef MI_CR
  const int rc = launch_status();
  return rc != MI_OK || !update_ring || max_query_len <= 1 ? rc : launch_conv_update<T>(p.in, num_reqs, s);
}

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int mi_conv_rope_cache(const mi_conv_rope_cache_args* a, int dtype, void* stream) {
  if (a && (a->num_reqs == 0 || a->max_query_len == 0)) return MI_OK;
  if (!a || !a->x || !a->conv_w || !a->ring || !a->q_out || !a->k_cache || !a->v_cache || !a->slots || !a->query_start_loc ||
      !a->seq_lens || !a->slot_mapping || (a->rot_dims && !a->inv_freq))
    return MI_ERR_INVALID_ARG;
  const int H = a->heads, G = a->kv_heads, D = a->dim, ch = (H + G) * D;
  if (a->req0 < 0 || a->num_reqs < 0 || a->max_query_len < 0 || H <= 0 || G <= 0 || D <= 0 || a->head_dim < D || a->block_size <= 0 ||
      a->taps <= 0 || a->rot_dims < 0 || a->rot_dims > D || a->rot_dims % 2)
    return MI_ERR_INVALID_ARG;
  if (a->x_stride < ch || a->q_stride < (int64_t)H * a->head_dim) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  if (a->num_reqs > 65535 || a->rot_dims / 2 > kMaxPairs) return MI_ERR_UNSUPPORTED;
  const ConvRopeParams p{{a->x, a->conv_w, a->ring, a->slots, a->query_start_loc, a->seq_lens, a->x_stride, a->req0, a->taps, ch},
                         a->q_out, a->k_cache, a->v_cache, a->inv_freq, a->slot_mapping, a->q_stride, a->cache_block_stride,
                         a->cache_token_stride, a->cache_head_stride, H, G, D, a->head_dim, a->block_size, a->rot_dims / 2, a->eps};
  const int al = dtype == MI_DTYPE_BF16 ? 8 : 4;
  const bool vec = D % 8 == 0 && a->head_dim % 8 == 0 && a->x_stride % al == 0 && a->q_stride % al == 0 &&
                   a->cache_block_stride % al == 0 && a->cache_token_stride % al == 0 && a->cache_head_stride % al == 0 &&
                   aligned16(a->x) && aligned16(a->conv_w) && aligned16(a->ring) && aligned16(a->q_out) && aligned16(a->k_cache) && aligned16(a->v_cache);
  hipStream_t s = (hipStream_t)stream;
  return dtype == MI_DTYPE_BF16 ? launch_conv_rope<uint16_t>(p, a->num_reqs, a->max_query_len, vec, a->update_ring, s)
                                : launch_conv_rope<float>(p, a->num_reqs, a->max_query_len, vec, a->update_ring, s);
}
