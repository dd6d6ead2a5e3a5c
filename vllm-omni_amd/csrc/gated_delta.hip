// Gated delta rule with per-channel short convolutions in front of it: the recurrent mixer of a decoder layer.
//
// Per v-head h (its q/k head is h / (heads / kv_heads)) and token:
//   q, k, v   = silu(causal conv over time of the projections);  q, k made unit vectors, q times dim^-1/2
//   M_t = g M_(t-1) + k (x) e   with  e = b (v - g k M_(t-1)),   y = q M_t        ln g = -exp(A_log) softplus(a + dt_bias)
//   out       = y / rms(y) * norm * silu(gate), or sigmoid(gate)
// g is one number per head, or one per head and key channel (a diagonal in front of the rows of M).  A row's q, k, v
// projections arrive side by side, gate, b and a wherever the caller has them.  Per request slot the state is M [dim][vdim]
// fp32 per head and a ring of the last `taps` projection rows (row p % taps holds position p); a request whose first
// token is position 0 starts from zeros whatever the slot holds, so slots need no clearing.
//
// Kernels:
//   * gated_delta_step: one workgroup per (head, request), the state in registers, tokens one after the other: decode
//     (HBM bound: the state is read and written once), and any shape the chunked pair does not build.
//   * conv_ring_update: leaves a multi-token portion's last rows in the ring (after every reader of the old rows).
#include <type_traits>

#include "gated_delta.h"

namespace mi {
namespace {

typedef __attribute__((ext_vector_type(4))) float f32x4;

// LDS: q[D] k[D] v[V] red[2][groups * V] decay[D].  R: rows of the state a thread holds; TAPS: convolution taps, 0 = any (one load
// after the other); FULL: the threads' tiles cover the state exactly.  A decode step is one chain of memory latencies per
// workgroup, so everything a token needs is asked for before the first use, the state with it; loads are unconditional on
// clamped addresses and their values selected afterwards (a load behind a branch is waited for on its own).
template <typename T, int VEC, int NT, int R, int TAPS, bool FULL, bool CHN>
__global__ __launch_bounds__(NT, R <= 8 ? 4 : 1) void gated_delta_step_kernel(const DeltaParams p) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int h = blockIdx.x, r = p.req0 + blockIdx.y;
  const int s0 = p.qsl[r], s1 = p.qsl[r + 1], seq = p.seq_lens[r];
  const int64_t slot = p.slots[r];
  const int L = s1 - s0, start = seq - L;      // start < 0: a padded row of a graph replay (scratch slot)
  if (L <= 0) return;
  const int D = p.D, V = p.V, H = p.H, per = H / p.K, kh = h / per;
  float* sq = lds;
  float* sk = sq + D;
  float* sv = sk + D;
  const int lv = V / VEC, groups = NT / lv;
  float* red0 = sv + V;
  float* red1 = red0 + groups * V;
  float* sdec = red1 + groups * V;       // CHN: decays of the key channels
  const int tid = threadIdx.x, g = tid / lv, c = (tid % lv) * VEC;
  const bool on = FULL || g < groups;
  float* S = p.state + ((slot * H + h) * D) * (int64_t)V;
  const T* proj = reinterpret_cast<const T*>(p.proj);
  const T* convw = reinterpret_cast<const T*>(p.convw);
  T* ring = reinterpret_cast<T*>(p.ring) + slot * p.taps * (int64_t)p.CH;
  auto has = [&](int n) { return FULL || (on && g + n * groups < D); };      // row n of the thread's tile exists
  float st[R][VEC];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int d = FULL ? g + i * groups : min(g + i * groups, D - 1);
    if constexpr (VEC == 4) {
      const f32x4 a = __builtin_nontemporal_load(reinterpret_cast<const f32x4*>(S + (int64_t)d * V + c));
      st[i][0] = a[0], st[i][1] = a[1], st[i][2] = a[2], st[i][3] = a[3];
    } else {
      st[i][0] = S[(int64_t)d * V + c];
    }
  }
  const float neg_a = -expf(p.a_log[h]), dtb = CHN ? 0.f : p.dt_bias[h];
  const float qs = 1.0f / sqrtf((float)D);
  const int nch = 2 * D + V;
  for (int i = 0; i < L; ++i) {
    const int64_t row = s0 + i;
    const int pos = start + i;
    const T* pr = proj + row * p.ld;
    const T* ar = reinterpret_cast<const T*>(p.a) + row * p.ld_a + (int64_t)h * (CHN ? D : 1);
    const float raw_a = Io<T>::ld(ar + (CHN ? min(tid, D - 1) : 0));
    const float raw_b = Io<T>::ld(reinterpret_cast<const T*>(p.b) + row * p.ld_b + h);
    float gt[4], nw[4];                          // what the first wave ends the token with: gate and norm weights (vdim <= 256)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int v = min((tid & 63) + 64 * j, V - 1);
      gt[j] = Io<T>::ld(reinterpret_cast<const T*>(p.gate) + row * p.ld_gate + h * V + v);
      nw[j] = Io<T>::ld(reinterpret_cast<const T*>(p.norm_w) + v);
    }
    for (int n0 = 0; n0 < nch; n0 += NT) {
      const int n = min(n0 + tid, nch - 1);
      const int ch = n < D ? kh * D + n : n < 2 * D ? p.K * D + kh * D + (n - D) : 2 * p.K * D + h * V + (n - 2 * D);
      auto tap = [&](int b, int taps) -> float {     // the input b tokens back
        const T* src = i >= b ? pr - b * p.ld : ring + (int64_t)((pos - b) % taps) * p.CH;
        const float x = Io<T>::ld((pos >= b ? src : pr) + ch);
        return pos >= b ? x : 0.f;
      };
      const T cur = pr[ch];
      float acc;
      if constexpr (TAPS > 0) {
        float x[TAPS], w[TAPS];
        x[0] = Io<T>::ld(&cur);
#pragma unroll
        for (int b = 1; b < TAPS; ++b) x[b] = tap(b, TAPS);
#pragma unroll
        for (int b = 0; b < TAPS; ++b) w[b] = Io<T>::ld(convw + (int64_t)ch * TAPS + TAPS - 1 - b);
        acc = x[0] * w[0];
#pragma unroll
        for (int b = 1; b < TAPS; ++b) acc += x[b] * w[b];
      } else {
        acc = Io<T>::ld(&cur) * Io<T>::ld(convw + (int64_t)ch * p.taps + p.taps - 1);
        for (int b = 1; b < p.taps; ++b) acc += tap(b, p.taps) * Io<T>::ld(convw + (int64_t)ch * p.taps + p.taps - 1 - b);
      }
      if (n0 + tid < nch) lds[n] = silu_f(acc);
      // one token: its row of the ring is nobody's to read this step (readers take the taps - 1 rows before it)
      if (L == 1 && pos >= 0 && n0 + tid < nch && (n >= 2 * D || h % per == 0)) ring[(int64_t)(pos % p.taps) * p.CH + ch] = cur;
    }
    if constexpr (CHN) {
      for (int d = tid; d < D; d += NT)
        sdec[d] = expf(neg_a * softplus_f((d < NT ? raw_a : Io<T>::ld(ar + d)) + p.dt_bias[h * D + d]));
    }
    if (i == 0) {
#pragma unroll
      for (int n = 0; n < R; ++n)
#pragma unroll
        for (int j = 0; j < VEC; ++j) st[n][j] = start > 0 && has(n) ? st[n][j] : 0.f;
    }
    __syncthreads();
    float qq = 0.f, kk = 0.f;
    for (int d = tid & 63; d < D; d += 64) qq += sq[d] * sq[d], kk += sk[d] * sk[d];
    const float qn = qs / sqrtf(wave_allreduce_sum(qq) + 1e-6f), kn = 1.0f / sqrtf(wave_allreduce_sum(kk) + 1e-6f);
    const float decay = CHN ? 1.f : expf(neg_a * softplus_f(raw_a + dtb));
    const float beta = sigmoid_f(raw_b);
    float acc[VEC] = {};
#pragma unroll
    for (int n = 0; n < R; ++n) {
      const float k = has(n) ? sk[g + n * groups] * kn : 0.f;
      const float f = CHN ? (has(n) ? sdec[g + n * groups] : 0.f) : decay;
#pragma unroll
      for (int j = 0; j < VEC; ++j) st[n][j] *= f, acc[j] += st[n][j] * k;
    }
    if (on)
#pragma unroll
      for (int j = 0; j < VEC; ++j) red0[g * V + c + j] = acc[j];
    __syncthreads();
    float u[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      float t = 0.f;
      if (on)
        for (int n = 0; n < groups; ++n) t += red0[n * V + c + j];
      u[j] = on ? beta * (sv[c + j] - t) : 0.f;
      acc[j] = 0.f;
    }
#pragma unroll
    for (int n = 0; n < R; ++n) {
      const float k = has(n) ? sk[g + n * groups] * kn : 0.f, q = has(n) ? sq[g + n * groups] * qn : 0.f;
#pragma unroll
      for (int j = 0; j < VEC; ++j) st[n][j] += k * u[j], acc[j] += st[n][j] * q;
    }
    if (on)
#pragma unroll
      for (int j = 0; j < VEC; ++j) red1[g * V + c + j] = acc[j];
    __syncthreads();
    if (tid < 64) {   // the read-out: norm over vdim, gate, store
      float ss = 0.f;
      for (int v = tid; v < V; v += 64) {
        float t = 0.f;
        for (int n = 0; n < groups; ++n) t += red1[n * V + v];
        red1[v] = t;
        ss += t * t;
      }
      const float inv = inv_rms(wave_allreduce_sum(ss), V, p.eps);
      T* o = reinterpret_cast<T*>(p.out) + row * p.ld_out + (int64_t)h * V;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (tid + 64 * j < V) Io<T>::st(o + tid + 64 * j, red1[tid + 64 * j] * inv * nw[j] * out_gate(p, gt[j]));
    }
  }
#pragma unroll
  for (int i = 0; i < R; ++i) {
    if (!has(i)) continue;
    const int d = g + i * groups;
    if constexpr (VEC == 4) {
      const f32x4 a = {st[i][0], st[i][1], st[i][2], st[i][3]};
      __builtin_nontemporal_store(a, reinterpret_cast<f32x4*>(S + (int64_t)d * V + c));
    } else {
      S[(int64_t)d * V + c] = st[i][0];
    }
  }
}

template <typename T, int VEC, int NT, int R>
int launch_step(const DeltaParams& p, int nreq, hipStream_t s) {
  const int groups = NT / (p.V / VEC);
  const size_t lds = (size_t)(2 * p.D + p.V + 2 * groups * p.V + (p.channel ? p.D : 0)) * sizeof(float);
  const bool full = VEC == 4 && NT % (p.V / VEC) == 0 && p.D == R * groups;
  auto pick = [&](auto chn) {
    constexpr bool C = decltype(chn)::value;
    return p.taps != 4 ? gated_delta_step_kernel<T, VEC, NT, R, 0, false, C>
           : full      ? gated_delta_step_kernel<T, VEC, NT, R, 4, true, C>
                       : gated_delta_step_kernel<T, VEC, NT, R, 4, false, C>;
  };
  auto kern = p.channel ? pick(std::true_type{}) : pick(std::false_type{});
  if (lds > 65536) {
    if (hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)
      return MI_ERR_LAUNCH;
  }
  hipLaunchKernelGGL(kern, dim3(p.H, nreq), dim3(NT), lds, s, p);
  return launch_status();
}

template <typename T>
int step_dispatch(const DeltaParams& p, int nreq, hipStream_t s) {
  if (p.V > 256) return MI_ERR_UNSUPPORTED;
  const int vec = p.V % 4 == 0 ? 4 : 1;
  const int lv = p.V / vec;
  auto fits = [&](int nt, int r) { const int gr = nt / lv; return gr > 0 && (p.D + gr - 1) / gr <= r; };
  if (vec == 4) {
    if (fits(256, 8)) return launch_step<T, 4, 256, 8>(p, nreq, s);
    if (fits(512, 8)) return launch_step<T, 4, 512, 8>(p, nreq, s);
    if (fits(512, 16)) return launch_step<T, 4, 512, 16>(p, nreq, s);
    if (fits(1024, 16)) return launch_step<T, 4, 1024, 16>(p, nreq, s);
  } else {
    if (fits(256, 32)) return launch_step<T, 1, 256, 32>(p, nreq, s);
    if (fits(1024, 64)) return launch_step<T, 1, 1024, 64>(p, nreq, s);
  }
  return MI_ERR_UNSUPPORTED;
}

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int mi_gated_delta_step(const mi_gated_delta_args* args, int32_t update_ring, int dtype, void* stream) {
  if (args && args->num_reqs == 0) return MI_OK;
  DeltaParams p;
  const int rc = delta_fill(p, args);
  if (rc != MI_OK) return rc;
  const int num_reqs = args->num_reqs;
  hipStream_t s = (hipStream_t)stream;
  int st;
  if (dtype == MI_DTYPE_BF16) st = step_dispatch<uint16_t>(p, num_reqs, s);
  else if (dtype == MI_DTYPE_F32) st = step_dispatch<float>(p, num_reqs, s);
  else return MI_ERR_UNSUPPORTED;
  if (st != MI_OK || !update_ring) return st;
  const dim3 grid((p.CH + 255) / 256, num_reqs), block(256);
  if (dtype == MI_DTYPE_BF16) hipLaunchKernelGGL((conv_ring_update_kernel<uint16_t>), grid, block, 0, s, p);
  else hipLaunchKernelGGL((conv_ring_update_kernel<float>), grid, block, 0, s, p);
  return launch_status();
}
