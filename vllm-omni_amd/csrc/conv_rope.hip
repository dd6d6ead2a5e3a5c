// What attention whose values are its keys does in front of the scores, in one launch: the short causal filter over q and k,
// the value row (k as the filter leaves it), rotary positions on neighbouring pairs, the unweighted norm per head, and the K / V
// cache write.  q's heads and the cache's are `hd` apart, zeros behind a head's own values.
//
// A workgroup has kRows rows of a request and as many heads as its lanes hold (LPH lanes a head, VEC channels a lane): a thread
// slides over its rows with the filter's inputs in registers.  The angles of a workgroup's rows are formed once (positions,
// angles, sines and cosines in fp32) and shared through LDS.
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

// TAPS: filter taps, 0 = any (inputs read again for every row)
template <typename T, int LPH, int VEC, int U, int TAPS>
__global__ __launch_bounds__(256) void conv_rope_cache_kernel(const ConvRopeParams p) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) float2 cs[];      // [kRows][pairs]: cosine, sine
  const int r = p.in.req0 + blockIdx.y, t0 = blockIdx.x * kRows;
  const int s0 = p.in.qsl[r], n = p.in.qsl[r + 1] - s0, start = p.in.seq_lens[r] - n;   // start < 0: a padded row of a graph replay
  if (t0 >= n) return;
  const int rows = min(kRows, n - t0);
  for (int k = threadIdx.x; k < rows * p.pairs; k += 256) {
    const int i = k / p.pairs, j = k % p.pairs;
    float s, c;
    sincosf((float)max(start + t0 + i, 0) * p.inv_freq[j], &s, &c);
    cs[k] = make_float2(c, s);
  }
  __syncthreads();
  const int head = (blockIdx.z * 256 + threadIdx.x) / LPH, sub = threadIdx.x % LPH;
  if (head >= p.H + p.G) return;                                  // whole lane groups leave
  const bool is_q = head < p.H;
  const int taps = TAPS ? TAPS : p.in.taps;
  const T* x = reinterpret_cast<const T*>(p.in.x) + (int64_t)(s0 + t0) * p.in.ld + (int64_t)head * p.dim;
  T* ring = reinterpret_cast<T*>(p.in.ring) + (int64_t)p.in.slots[r] * p.in.taps * p.in.channels + (int64_t)head * p.dim;
  const T* w = reinterpret_cast<const T*>(p.in.w) + (int64_t)head * p.dim * taps;
  auto load = [&](const T* src, int c, float (&v)[VEC]) {
    if constexpr (VEC == 8) {
      Io<T>::template ldv<8>(src + c, v);
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        const float a = Io<T>::ld(src + min(c + j, p.dim - 1));
        v[j] = c + j < p.dim ? a : 0.f;
      }
    }
  };
  constexpr int HELD = TAPS ? TAPS : 1;
  float wt[U][HELD][VEC], prev[U][HELD][VEC];                      // prev[b - 1]: the input b rows back
  if constexpr (TAPS > 0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = (sub + u * LPH) * VEC;
#pragma unroll
      for (int b = 0; b < TAPS; ++b)
#pragma unroll
        for (int j = 0; j < VEC; ++j) wt[u][b][j] = c + j < p.dim ? Io<T>::ld(w + (int64_t)(c + j) * TAPS + TAPS - 1 - b) : 0.f;
#pragma unroll
      for (int b = 1; b < TAPS; ++b) {
        const int pos = start + t0;
        load(conv_input(p.in, x, ring, t0, pos, b), c < p.dim ? c : 0, prev[u][b - 1]);
#pragma unroll
        for (int j = 0; j < VEC; ++j) prev[u][b - 1][j] = pos >= b && c + j < p.dim ? prev[u][b - 1][j] : 0.f;
      }
    }
  }
  for (int i = 0; i < rows; ++i, x += p.in.ld) {
    const int pos = start + t0 + i;
    float y[U][VEC];
    float ss = 0.f;
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int c = (sub + u * LPH) * VEC;
      const bool mine = c < p.dim;
      float cur[VEC];
      load(x, mine ? c : 0, cur);
      if constexpr (TAPS > 0) {
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          y[u][j] = cur[j] * wt[u][0][j];
#pragma unroll
          for (int b = 1; b < TAPS; ++b) y[u][j] += prev[u][b - 1][j] * wt[u][b][j];
        }
#pragma unroll
        for (int b = TAPS - 2; b > 0; --b)
#pragma unroll
          for (int j = 0; j < VEC; ++j) prev[u][b][j] = prev[u][b - 1][j];
#pragma unroll
        for (int j = 0; j < VEC; ++j) prev[u][0][j] = cur[j];
      } else {
#pragma unroll
        for (int j = 0; j < VEC; ++j) y[u][j] = 0.f;
        for (int b = 0; b < taps && b <= pos; ++b) {
          float v[VEC];
          load(b == 0 ? x : conv_input(p.in, x, (const T*)ring, t0 + i, pos, b), mine ? c : 0, v);
#pragma unroll
          for (int j = 0; j < VEC; ++j)
            if (c + j < p.dim) y[u][j] += v[j] * Io<T>::ld(w + (int64_t)(c + j) * taps + taps - 1 - b);
        }
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        y[u][j] = c + j < p.dim ? y[u][j] : 0.f;
        ss += y[u][j] * y[u][j];
      }
      if (n == 1 && start >= 0 && mine) {      // the request's only row: its place in the ring is nobody's to read
        T* dst = ring + (int64_t)(pos % p.in.taps) * p.in.channels;
        if constexpr (VEC == 8) {
          Io<T>::template stv<8>(dst + c, cur);
        } else {
#pragma unroll
          for (int j = 0; j < VEC; ++j)
            if (c + j < p.dim) Io<T>::st(dst + c + j, cur[j]);
        }
      }
    }
#pragma unroll
    for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    const float inv = inv_rms(ss, p.dim, p.eps);                  // a rotation leaves the mean square as it is
    const int64_t row = s0 + t0 + i;
    T *dst, *vdst = nullptr;
    if (is_q) {
      dst = reinterpret_cast<T*>(p.q_out) + row * p.q_stride + (int64_t)head * p.hd;
    } else {
      const int64_t slot = p.slot_mapping[row];
      if (slot < 0) continue;                                     // whole lane groups: the sums above are done
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
          const float2 a = cs[i * p.pairs + k];
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
}

template <typename T>
int launch_conv_rope(const ConvRopeParams& p, int num_reqs, int max_query_len, bool vec, int update_ring, hipStream_t s) {
  const dim3 block(256);
  const int units = p.H + p.G;
  const size_t lds = (size_t)kRows * (p.pairs > 0 ? p.pairs : 1) * sizeof(float2);
#define MI_CR(LPH, VEC, U, TAPS)                                                                                              \
  hipLaunchKernelGGL((conv_rope_cache_kernel<T, LPH, VEC, U, TAPS>),                                                          \
                     dim3((max_query_len + kRows - 1) / kRows, num_reqs, (units * LPH + 255) / 256), block, lds, s, p)
#define MI_CR_T(LPH, VEC, U)                                                                                                  \
  do {                                                                                                                        \
    if (p.in.taps == 4) MI_CR(LPH, VEC, U, 4);                                                                                \
    else MI_CR(LPH, VEC, U, 0);                                                                                               \
  } while (0)
  if (vec && p.hd <= 64) MI_CR_T(8, 8, 1);
  else if (vec && p.hd <= 128) MI_CR_T(16, 8, 1);
  else if (p.hd <= 128) MI_CR_T(64, 2, 1);
  else if (p.hd <= 1024) MI_CR(64, 2, 8, 0);
  else return MI_ERR_UNSUPPORTED;
#undef MI_CR_T
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
                   aligned16(a->x) && aligned16(a->ring) && aligned16(a->q_out) && aligned16(a->k_cache) && aligned16(a->v_cache);
  hipStream_t s = (hipStream_t)stream;
  return dtype == MI_DTYPE_BF16 ? launch_conv_rope<uint16_t>(p, a->num_reqs, a->max_query_len, vec, a->update_ring, s)
                                : launch_conv_rope<float>(p, a->num_reqs, a->max_query_len, vec, a->update_ring, s);
}
