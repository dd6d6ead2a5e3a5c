// Gated delta rule over prompt portions, in chunks of 64 tokens on the fp32 matrix cores.
//
// Within a chunk with entry state S0, G_i = sum of log decays up to i, u_i the corrected values:
//   (I + A) U = diag(b) (V - diag(e^G) K S0),   A_ij = b_i e^(G_i - G_j) k_i . k_j  (j < i)
//   O = diag(e^G) Q S0 + P U,                   P_ij = e^(G_i - G_j) q_i . k_j      (j <= i)
//   S1 = e^(G_C) S0 + sum_j e^(G_C - G_j) k_j u_j^T
// so everything but the S0 terms is independent between chunks:
//   * prep (one workgroup per chunk and head): convolutions, silu, unit q / k, gates; A, its unit-triangular inverse T,
//     P, and T diag(b) V, T diag(b e^G) K, diag(e^G) Q, (e^(G_C - G_j) k_j)^T to a workspace;
//   * scan (one workgroup per request, head and 16 value columns): chunk after chunk, U, O and S with S in registers;
//   * finish: o / rms(o) * norm * silu(gate).
// All products run on v_mfma_f32_16x16x4_f32: q, k, decays and state are 32-bit quantities of the recurrence.  The k order
// inside 16 consecutive k is permuted alike in both operands (step s takes k = 4 (lane / 16) + s), so an operand whose k is
// contiguous is one 16-byte read for four steps, and an accumulator tile IS the B operand of a following product.
#include "gated_delta.h"
#include "mfma_attn_common.h"

namespace mi {
namespace {

constexpr int kC = 64;             // tokens per chunk
constexpr int kPrepThreads = 512;

__device__ __forceinline__ f32x4_t mma4(const float (&a)[4], const float (&b)[4], f32x4_t c) {
#pragma unroll
  for (int s = 0; s < 4; ++s) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[s], b[s], c, 0, 0, 0);
  return c;
}
__device__ __forceinline__ void frag_rows(const float* p, int ld, int lane, float (&f)[4]) {   // [row][k], k contiguous
  const float4 v = *reinterpret_cast<const float4*>(p + (lane & 15) * ld + 4 * (lane >> 4));
  f[0] = v.x, f[1] = v.y, f[2] = v.z, f[3] = v.w;
}
__device__ __forceinline__ void frag_cols(const float* p, int ld, int lane, float (&f)[4]) {   // [k][col]
#pragma unroll
  for (int s = 0; s < 4; ++s) f[s] = p[(4 * (lane >> 4) + s) * ld + (lane & 15)];
}

// workspace of one (chunk, head): W [C][Dp], Q [C][Dp], Kt [Dp][C], P [C][C], U [C][Vp], then e^(G_C)
struct ChunkLayout {
  int Dp, Vp;
  __host__ __device__ int64_t w() const { return 0; }
  __host__ __device__ int64_t q() const { return (int64_t)kC * Dp; }
  __host__ __device__ int64_t kt() const { return 2 * (int64_t)kC * Dp; }
  __host__ __device__ int64_t pm() const { return 3 * (int64_t)kC * Dp; }
  __host__ __device__ int64_t u() const { return 3 * (int64_t)kC * Dp + kC * kC; }
  __host__ __device__ int64_t g() const { return u() + (int64_t)kC * Vp; }
  __host__ __device__ int64_t size() const { return g() + 16; }
};

__device__ __forceinline__ int64_t chunk_base(const DeltaParams& p, int r) {
  return (p.qsl[r] - p.qsl[p.req0]) / kC + (r - p.req0);
}

// conv + silu of channels [ch0, ch0 + n) of the chunk's rows into buf [C][ld]; zeros in rows past len and columns past n
template <typename T>
__device__ __forceinline__ void conv_rows(const DeltaParams& p, float* buf, int ld, int np, int ch0, int n, int64_t row0, int i0,
                                          int len, int start, const T* ring) {
  const T* proj = reinterpret_cast<const T*>(p.proj);
  const T* cw = reinterpret_cast<const T*>(p.convw);
  const int segs = kPrepThreads / np > 0 ? kPrepThreads / np : 1;      // row segments worked on side by side
  const int rows_per = (kC + segs - 1) / segs;
  for (int item = threadIdx.x; item < segs * np; item += kPrepThreads) {
    const int c = item % np, seg = item / np;
    const int a = seg * rows_per, b = min(kC, a + rows_per);
    if (c >= n) {
      for (int i = a; i < b; ++i) buf[i * ld + c] = 0.f;
      continue;
    }
    const int ch = ch0 + c;
    // input of chunk row i (may be negative: rows of this portion in front of the chunk, then the ring, then zeros)
    auto in = [&](int i) -> float {
      if (i >= len) return 0.f;
      if (i0 + i >= 0) return Io<T>::ld(proj + (row0 + i) * p.ld + ch);
      const int pos = start + i0 + i;
      return pos >= 0 ? Io<T>::ld(ring + (int64_t)(pos % p.taps) * p.CH + ch) : 0.f;
    };
    if (p.taps == 4) {
      const float w0 = Io<T>::ld(cw + ch * 4), w1 = Io<T>::ld(cw + ch * 4 + 1), w2 = Io<T>::ld(cw + ch * 4 + 2),
                  w3 = Io<T>::ld(cw + ch * 4 + 3);
      float x0 = in(a - 3), x1 = in(a - 2), x2 = in(a - 1);
      for (int i = a; i < b; ++i) {
        float v = 0.f;
        if (i < len) {
          const float x3 = Io<T>::ld(proj + (row0 + i) * p.ld + ch);
          v = silu_f(w0 * x0 + w1 * x1 + w2 * x2 + w3 * x3);
          x0 = x1, x1 = x2, x2 = x3;
        }
        buf[i * ld + c] = v;
      }
    } else {
      for (int i = a; i < b; ++i) {
        float v = 0.f;
        if (i < len) {
          for (int t = 0; t < p.taps; ++t) v += Io<T>::ld(cw + (int64_t)ch * p.taps + t) * in(i - (p.taps - 1) + t);
          v = silu_f(v);
        }
        buf[i * ld + c] = v;
      }
    }
  }
}

// the same, 8 channels a thread: every load of a thread is independent of the others.  Needs n, the channel offsets and the
// row strides to be multiples of 8.
template <typename T, int TAPS>
__device__ __forceinline__ void conv_rows8(const DeltaParams& p, float* buf, int ld, int np, int ch0, int n, int64_t row0, int i0,
                                           int len, int start, const T* ring) {
  const T* proj = reinterpret_cast<const T*>(p.proj);
  const T* cw = reinterpret_cast<const T*>(p.convw);
  const int per = np / 8;
  for (int item = threadIdx.x; item < kC * per; item += kPrepThreads) {
    const int c = (item % per) * 8, i = item / per;
    float acc[8] = {};
    if (c < n && i < len) {
      const int ch = ch0 + c;
      float w[TAPS][8], x[TAPS][8];
      float wf[8 * TAPS];
#pragma unroll
      for (int t = 0; t < TAPS; ++t) Io<T>::template ldv<8>(cw + (int64_t)ch * TAPS + 8 * t, *reinterpret_cast<float(*)[8]>(wf + 8 * t));
#pragma unroll
      for (int t = 0; t < TAPS; ++t)
#pragma unroll
        for (int j = 0; j < 8; ++j) w[t][j] = wf[j * TAPS + t];
#pragma unroll
      for (int t = 0; t < TAPS; ++t) {
        const int k = i - (TAPS - 1) + t;
        const int pos = start + i0 + k;
        if (i0 + k >= 0) {
          Io<T>::template ldv<8>(proj + (row0 + k) * p.ld + ch, x[t]);
        } else if (pos >= 0) {
          Io<T>::template ldv<8>(ring + (int64_t)(pos % TAPS) * p.CH + ch, x[t]);
        } else {
#pragma unroll
          for (int j = 0; j < 8; ++j) x[t][j] = 0.f;
        }
      }
#pragma unroll
      for (int t = 0; t < TAPS; ++t)
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[j] += w[t][j] * x[t][j];
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[j] = silu_f(acc[j]);
    }
    *reinterpret_cast<float4*>(buf + i * ld + c) = make_float4(acc[0], acc[1], acc[2], acc[3]);
    *reinterpret_cast<float4*>(buf + i * ld + c + 4) = make_float4(acc[4], acc[5], acc[6], acc[7]);
  }
}

template <typename T>
__device__ __forceinline__ void conv_tile(const DeltaParams& p, bool vec, float* buf, int ld, int np, int ch0, int n, int64_t row0,
                                          int i0, int len, int start, const T* ring) {
  if (vec && p.taps == 4) conv_rows8<T, 4>(p, buf, ld, np, ch0, n, row0, i0, len, start, ring);
  else if (vec && p.taps == 3) conv_rows8<T, 3>(p, buf, ld, np, ch0, n, row0, i0, len, start, ring);
  else if (vec && p.taps == 2) conv_rows8<T, 2>(p, buf, ld, np, ch0, n, row0, i0, len, start, ring);
  else conv_rows<T>(p, buf, ld, np, ch0, n, row0, i0, len, start, ring);
}

// rows of buf made unit vectors (16 lanes a row), then times mul
__device__ __forceinline__ void unit_rows(float* buf, int ld, int np, float mul) {
  const int sub = threadIdx.x & 15;
  for (int i = threadIdx.x >> 4; i < kC; i += kPrepThreads / 16) {
    float ss = 0.f;
    for (int c = sub; c < np; c += 16) ss += buf[i * ld + c] * buf[i * ld + c];
    ss = group_allreduce_sum<16>(ss);
    const float f = mul / sqrtf(ss + 1e-6f);
    for (int c = sub; c < np; c += 16) buf[i * ld + c] *= f;
  }
}

template <typename T>
__global__ __launch_bounds__(kPrepThreads, 4) void gated_delta_prep_kernel(const DeltaParams p, float* ws, const ChunkLayout lay, bool vec) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int r = p.req0 + blockIdx.z, h = blockIdx.y, ck = blockIdx.x;
  const int s0 = p.qsl[r], L = p.qsl[r + 1] - s0;
  const int i0 = ck * kC;
  if (i0 >= L) return;
  const int len = min(kC, L - i0);
  const int start = p.seq_lens[r] - L;
  const int64_t row0 = s0 + i0;
  const int Dp = lay.Dp, Vp = lay.Vp, ldk = Dp + 4, ldm = kC + 4;
  const int ldv = Vp + 4, big = kC * max(ldk, ldv);
  float* bufA = lds;                       // K, then V
  float* bufB = bufA + big;                // Q, then A and T
  float* mA = bufB;
  float* mT = bufB + kC * ldm;
  float* sG = bufB + max(kC * ldk, 2 * kC * ldm);   // G_i
  float* sB = sG + kC;                     // b_i
  float* sE = sB + kC;                     // b_i e^(G_i)
  float* sQ = sE + kC;                     // e^(G_i)
  float* sD = sQ + kC;                     // e^(G_C - G_i)
  float* out = ws + ((chunk_base(p, r) + ck) * p.H + h) * lay.size();
  const T* ring = reinterpret_cast<const T*>(p.ring) + (int64_t)p.slots[r] * p.taps * p.CH;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int kh = h / (p.H / p.K);
  conv_tile<T>(p, vec, bufA, ldk, Dp, p.K * p.D + kh * p.D, p.D, row0, i0, len, start, ring);
  conv_tile<T>(p, vec, bufB, ldk, Dp, kh * p.D, p.D, row0, i0, len, start, ring);
  if (wave == 0) {   // gates: cumulative log decay over the 64 tokens of the chunk
    const T* pr = reinterpret_cast<const T*>(p.proj) + (row0 + lane) * p.ld;
    float lg = 0.f, b = 0.f;
    if (lane < len) {
      lg = -expf(p.a_log[h]) * softplus_f(Io<T>::ld(pr + p.off_a + h) + p.dt_bias[h]);
      b = sigmoid_f(Io<T>::ld(pr + p.off_b + h));
    }
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float t = __shfl_up(lg, o, 64);
      if (lane >= o) lg += t;
    }
    sG[lane] = lg;
    sB[lane] = b;
    const float e = expf(lg);
    sE[lane] = b * e;
    sQ[lane] = e;
    sD[lane] = expf(__shfl(lg, 63, 64) - lg);
    if (lane == 63) out[lay.g()] = e;
  }
  __syncthreads();
  unit_rows(bufA, ldk, Dp, 1.0f);
  unit_rows(bufB, ldk, Dp, 1.0f / sqrtf((float)p.D));
  __syncthreads();
  // A and P, 16 tiles each, lower ones only: P goes out, A waits in registers until Q is dead
  f32x4_t keep[2];
#pragma unroll
  for (int n = 0; n < 4; ++n) {
    const int t = wave + n * (kPrepThreads / 64);
    const bool isP = n >= 2;
    const int ti = (t & 15) >> 2, tj = t & 3;
    if (!isP) keep[n] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (tj > ti) {
      if (isP)      // the scan multiplies whole rows of P
#pragma unroll
        for (int s = 0; s < 4; ++s) out[lay.pm() + (ti * 16 + 4 * (lane >> 4) + s) * kC + tj * 16 + (lane & 15)] = 0.f;
      continue;
    }
    const float* a = (isP ? bufB : bufA) + ti * 16 * ldk;
    const float* b = bufA + tj * 16 * ldk;
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
    for (int k = 0; k < Dp; k += 16) {
      float fa[4], fb[4];
      frag_rows(a + k, ldk, lane, fa);
      frag_rows(b + k, ldk, lane, fb);
      acc = mma4(fa, fb, acc);
    }
    const int j = tj * 16 + (lane & 15);
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int i = ti * 16 + 4 * (lane >> 4) + s;
      const float e = expf(fminf(sG[i] - sG[j], 0.f));
      if (isP) out[lay.pm() + i * kC + j] = j <= i ? acc[s] * e : 0.f;
      else keep[n & 1][s] = j < i ? acc[s] * e * sB[i] : 0.f;
    }
  }
  // diag(e^G) Q and the transposed, decayed keys
  for (int n = tid; n < kC * Dp / 4; n += kPrepThreads) {
    const int i = n / (Dp / 4), c = (n % (Dp / 4)) * 4;
    const float e = sQ[i];
    const float4 v = *reinterpret_cast<const float4*>(bufB + i * ldk + c);
    *reinterpret_cast<float4*>(out + lay.q() + (int64_t)i * Dp + c) = make_float4(v.x * e, v.y * e, v.z * e, v.w * e);
  }
  for (int n = tid; n < kC * Dp; n += kPrepThreads) {
    const int d = n / kC, j = n % kC;
    out[lay.kt() + n] = j < len ? bufA[j * ldk + d] * sD[j] : 0.f;
  }
  __syncthreads();   // Q is dead: A and T take its place
#pragma unroll
  for (int n = 0; n < 2; ++n) {
    const int t = wave + n * (kPrepThreads / 64);
#pragma unroll
    for (int s = 0; s < 4; ++s) mA[((t >> 2) * 16 + 4 * (lane >> 4) + s) * ldm + (t & 3) * 16 + (lane & 15)] = keep[n][s];
  }
  __syncthreads();
  // T = (I + A)^-1: diagonal 16 x 16 blocks by substitution, one column a lane
  if (wave < 4 && lane < 16) {
    const float* a = mA + wave * 16 * ldm + wave * 16;
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == lane ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) v -= a[i * ldm + j] * x[j];
      x[i] = v;
      mT[(wave * 16 + i) * ldm + wave * 16 + lane] = v;
    }
  }
  __syncthreads();
  for (int dist = 1; dist < 4; ++dist) {   // T_ij = -T_ii sum_k A_ik T_kj
    if (wave < 4 - dist) {
      const int tj = wave, ti = wave + dist;
      f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
      float fa[4], fb[4];
      for (int k = tj; k < ti; ++k) {
        frag_rows(mA + ti * 16 * ldm + k * 16, ldm, lane, fa);
        frag_cols(mT + k * 16 * ldm + tj * 16, ldm, lane, fb);
        acc = mma4(fa, fb, acc);
      }
      frag_rows(mT + ti * 16 * ldm + ti * 16, ldm, lane, fa);
      fb[0] = -acc[0], fb[1] = -acc[1], fb[2] = -acc[2], fb[3] = -acc[3];
      f32x4_t z = {0.f, 0.f, 0.f, 0.f};
      z = mma4(fa, fb, z);
#pragma unroll
      for (int s = 0; s < 4; ++s) mT[(ti * 16 + 4 * (lane >> 4) + s) * ldm + tj * 16 + (lane & 15)] = z[s];
    }
    __syncthreads();
  }
  // T diag(f) X, X [C][n] in bufA
  auto times = [&](const float* f, int ld, int np, float* dst) {
    const int nt = np / 16;
    for (int t = wave; t < 4 * nt; t += kPrepThreads / 64) {
      const int ti = t / nt, tn = t % nt;
      f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
      for (int k = 0; k <= ti; ++k) {
        float fa[4], fb[4];
        frag_rows(mT + ti * 16 * ldm + k * 16, ldm, lane, fa);
#pragma unroll
        for (int s = 0; s < 4; ++s) fa[s] *= f[k * 16 + 4 * (lane >> 4) + s];
        frag_cols(bufA + k * 16 * ld + tn * 16, ld, lane, fb);
        acc = mma4(fa, fb, acc);
      }
#pragma unroll
      for (int s = 0; s < 4; ++s) dst[(int64_t)(ti * 16 + 4 * (lane >> 4) + s) * np + tn * 16 + (lane & 15)] = acc[s];
    }
  };
  times(sE, ldk, Dp, out + lay.w());
  __syncthreads();
  conv_tile<T>(p, vec, bufA, ldv, Vp, 2 * p.K * p.D + h * p.V, p.V, row0, i0, len, start, ring);
  __syncthreads();
  times(sB, ldv, Vp, out + lay.u());
}

// LDS-only barrier: register loads in flight stay in flight
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// NV 16-column value tiles a workgroup: its four waves read every operand of a chunk once for all of them (the bound is the
// L2 traffic of those operands, each head's tiles reading the same ones)
template <int DT, int NV>
__global__ __launch_bounds__(256, 1) void gated_delta_scan_kernel(const DeltaParams p, float* ws, const ChunkLayout lay, int nvg) {
  scalar_cache_acquire();
  constexpr int Dp = DT * 16, LS = Dp + 4, LU = kC + 4, MT = (DT + 3) / 4;
  constexpr bool whole = DT % 4 == 0;      // every wave owns MT tiles of the state
  __shared__ __attribute__((aligned(16))) float sS[NV * 16 * LS];
  __shared__ __attribute__((aligned(16))) float sU[NV * 16 * LU];
  // the workgroups of a head on one XCD (workgroups go to the 8 XCDs in turn)
  const int bid = blockIdx.x;
  const int h = (bid / (8 * nvg)) * 8 + bid % 8, vg = (bid / 8) % nvg;
  const int r = p.req0 + blockIdx.y;
  const int s0 = p.qsl[r], L = p.qsl[r + 1] - s0;
  if (h >= p.H || L <= 0) return;
  const int start = p.seq_lens[r] - L;
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, lr = lane & 15, lg = lane >> 4;
  const int v0 = vg * 16 * NV + lr;        // + 16 n: this lane's value columns
  float* S = p.state + (((int64_t)p.slots[r] * p.H + h) * p.D) * p.V;
  f32x4_t st[NV][MT];
#pragma unroll
  for (int n = 0; n < NV; ++n)
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      const int mt = wave + 4 * m, v = v0 + 16 * n;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = mt * 16 + 4 * lg + i;
        st[n][m][i] = start > 0 && d < p.D && v < p.V ? S[(int64_t)d * p.V + v] : 0.f;
      }
      if (mt < DT) *reinterpret_cast<f32x4_t*>(sS + (16 * n + lr) * LS + mt * 16 + 4 * lg) = st[n][m];
    }
  const int nck = (L + kC - 1) / kC;
  float* base = ws + (chunk_base(p, r) * p.H + h) * lay.size();
  const int64_t step = p.H * lay.size();
  // one chunk's operands; the next chunk's are loaded a whole chunk ahead (the chain of chunks is the critical path, its
  // loads must not be).  Loads and stores are unconditional — past the last chunk the loads fetch what nobody uses, read-outs
  // replace U in the workspace — so that the number in flight is known at every wait: memory operations retire in order, and a
  // store that may or may not be there makes the wait for the loads behind it wait for its acknowledgement as well.
  struct Chunk {
    f32x4_t w[DT], q[DT], pm[4], kt[MT][4], u[NV];
    float g;
  };
  auto load = [&](Chunk& x, int c) {
    const float* b = base + c * step;
    const int64_t ro = (int64_t)(16 * wave + lr) * Dp + 4 * lg;
#pragma unroll
    for (int k = 0; k < DT; ++k) {
      x.w[k] = *reinterpret_cast<const f32x4_t*>(b + lay.w() + ro + 16 * k);
      x.q[k] = *reinterpret_cast<const f32x4_t*>(b + lay.q() + ro + 16 * k);
    }
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int i = 0; i < 4; ++i)
        x.u[n][i] = b[lay.u() + (int64_t)(16 * wave + 4 * lg + i) * lay.Vp + v0 + 16 * n];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      x.pm[k] = *reinterpret_cast<const f32x4_t*>(b + lay.pm() + (16 * wave + lr) * kC + 16 * k + 4 * lg);
#pragma unroll
      for (int m = 0; m < MT; ++m)
        x.kt[m][k] = *reinterpret_cast<const f32x4_t*>(b + lay.kt() + (int64_t)(min(wave + 4 * m, DT - 1) * 16 + lr) * kC + 16 * k + 4 * lg);
    }
    x.g = b[lay.g()];
  };
  auto work = [&](Chunk& x, int c) {
    f32x4_t d[NV] = {}, ao[NV] = {};
    f32x4_t sv[2][NV];       // the next k block's reads under this one's products
    auto get = [&](f32x4_t (&f)[NV], const float* b, int ld, int k) {
#pragma unroll
      for (int n = 0; n < NV; ++n) f[n] = *reinterpret_cast<const f32x4_t*>(b + (16 * n + lr) * ld + 16 * k + 4 * lg);
    };
    get(sv[0], sS, LS, 0);
#pragma unroll
    for (int k = 0; k < DT; ++k) {
      if (k + 1 < DT) get(sv[(k + 1) & 1], sS, LS, k + 1);
#pragma unroll
      for (int n = 0; n < NV; ++n)
#pragma unroll
        for (int s = 0; s < 4; ++s) {
          d[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w[k][s], sv[k & 1][n][s], d[n], 0, 0, 0);
          ao[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[k][s], sv[k & 1][n][s], ao[n], 0, 0, 0);
        }
      __builtin_amdgcn_sched_barrier(0);
    }
#pragma unroll
    for (int n = 0; n < NV; ++n) *reinterpret_cast<f32x4_t*>(sU + (16 * n + lr) * LU + 16 * wave + 4 * lg) = x.u[n] - d[n];
    lds_barrier();
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int m = 0; m < MT; ++m) st[n][m] *= x.g;
    get(sv[0], sU, LU, 0);
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      if (k < 3) get(sv[(k + 1) & 1], sU, LU, k + 1);
#pragma unroll
      for (int n = 0; n < NV; ++n)
#pragma unroll
        for (int s = 0; s < 4; ++s) {
          const float uv = sv[k & 1][n][s];
#pragma unroll
          for (int m = 0; m < MT; ++m)
            if (whole || wave + 4 * m < DT) st[n][m] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.kt[m][k][s], uv, st[n][m], 0, 0, 0);
          ao[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.pm[k][s], uv, ao[n], 0, 0, 0);
        }
      __builtin_amdgcn_sched_barrier(0);
    }
#pragma unroll
    for (int n = 0; n < NV; ++n) {
#pragma unroll
      for (int m = 0; m < MT; ++m)
        if (whole || wave + 4 * m < DT) *reinterpret_cast<f32x4_t*>(sS + (16 * n + lr) * LS + (wave + 4 * m) * 16 + 4 * lg) = st[n][m];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        base[c * step + lay.u() + (int64_t)(16 * wave + 4 * lg + i) * lay.Vp + v0 + 16 * n] = ao[n][i];
      }
    }
    lds_barrier();
  };
  Chunk a, b;
  load(a, 0);
  lds_barrier();
  for (int c = 0; c < nck; c += 2) {
    load(b, min(c + 1, nck - 1));
    work(a, c);
    if (c + 1 >= nck) break;
    load(a, min(c + 2, nck - 1));
    work(b, c + 1);
  }
#pragma unroll
  for (int n = 0; n < NV; ++n)
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = (wave + 4 * m) * 16 + 4 * lg + i, v = v0 + 16 * n;
        if (d < p.D && v < p.V) S[(int64_t)d * p.V + v] = st[n][m][i];
      }
}

// the read-out of (row, head), where the scan left it
__device__ __forceinline__ const float* readout(const DeltaParams& p, const float* ws, const ChunkLayout& lay, int nreq, int row, int h) {
  const int r = p.req0 + row_request(p.qsl + p.req0, nreq, row);
  const int i = row - p.qsl[r];
  return ws + ((chunk_base(p, r) + i / kC) * p.H + h) * lay.size() + lay.u() + (int64_t)(i % kC) * lay.Vp;
}

// out = o / rms(o) * norm * silu(gate), 16 lanes per (row, head), 8 values a lane at a time; vdim a multiple of 8, <= 128 U
template <typename T, int U>
__global__ __launch_bounds__(256) void gated_delta_finish8_kernel(const DeltaParams p, const float* ws, const ChunkLayout lay, int nreq, int row0, int rows) {
  scalar_cache_acquire();
  const int64_t item = (int64_t)blockIdx.x * 16 + (threadIdx.x >> 4);
  const int sub = threadIdx.x & 15;
  if (item >= (int64_t)rows * p.H) return;     // whole 16-lane groups leave
  const int64_t row = row0 + item / p.H;
  const int h = (int)(item % p.H);
  const float* x = readout(p, ws, lay, nreq, (int)row, h);
  const T* g = reinterpret_cast<const T*>(p.proj) + row * p.ld + p.off_g + h * p.V;
  float v[U][8], gt[U][8];
  float ss = 0.f;
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int c = 8 * (sub + 16 * u);
    if (c >= p.V) continue;
    Io<float>::ldv<8>(x + c, v[u]);
    Io<T>::template ldv<8>(g + c, gt[u]);
#pragma unroll
    for (int j = 0; j < 8; ++j) ss += v[u][j] * v[u][j];
  }
  const float inv = inv_rms(group_allreduce_sum<16>(ss), p.V, p.eps);
  T* out = reinterpret_cast<T*>(p.out) + (row * p.H + h) * (int64_t)p.V;
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int c = 8 * (sub + 16 * u);
    if (c >= p.V) continue;
    float w[8];
    Io<T>::template ldv<8>(reinterpret_cast<const T*>(p.norm_w) + c, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[u][j] *= inv * w[j] * silu_f(gt[u][j]);
    Io<T>::template stv<8>(out + c, v[u]);
  }
}

// the same for any vdim, one wave per (row, head)
template <typename T>
__global__ __launch_bounds__(256) void gated_delta_finish_kernel(const DeltaParams p, const float* ws, const ChunkLayout lay, int nreq, int row0, int rows) {
  scalar_cache_acquire();
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (item >= (int64_t)rows * p.H) return;
  const int64_t row = row0 + item / p.H;
  const int h = (int)(item % p.H);
  const float* x = readout(p, ws, lay, nreq, (int)row, h);
  float ss = 0.f;
  for (int v = lane; v < p.V; v += 64) ss += x[v] * x[v];
  const float inv = inv_rms(wave_allreduce_sum(ss), p.V, p.eps);
  const T* g = reinterpret_cast<const T*>(p.proj) + row * p.ld + p.off_g + h * p.V;
  const T* nw = reinterpret_cast<const T*>(p.norm_w);
  T* out = reinterpret_cast<T*>(p.out) + (row * p.H + h) * (int64_t)p.V;
  for (int v = lane; v < p.V; v += 64) Io<T>::st(out + v, x[v] * inv * Io<T>::ld(nw + v) * silu_f(Io<T>::ld(g + v)));
}

inline int round_tiles(int n) {   // 16-column tiles of the built scans: 2, 4, 8, 16
  const int t = (n + 15) / 16;
  return t <= 2 ? 2 : t <= 4 ? 4 : t <= 8 ? 8 : 16;
}

}  // namespace
}  // namespace mi

using namespace mi;

static bool chunk_layout(int32_t dim, int32_t vdim, ChunkLayout* lay) {
  if (dim <= 0 || vdim <= 0 || dim > 256 || vdim > 256) return false;
  lay->Dp = 16 * round_tiles(dim);
  lay->Vp = (vdim + 15) / 16 * 16;
  return true;
}

extern "C" int64_t mi_gated_delta_chunked_workspace_bytes(int32_t rows, int32_t num_reqs, int32_t heads, int32_t dim, int32_t vdim) {
  ChunkLayout lay;
  if (rows < 0 || num_reqs < 0 || heads <= 0 || !chunk_layout(dim, vdim, &lay)) return 0;
  const int64_t chunks = rows / kC + num_reqs;
  return chunks * heads * lay.size() * 4;
}

extern "C" int mi_gated_delta_chunked(const void* proj, int64_t proj_stride, const void* conv_w, const float* a_log,
                                      const float* dt_bias, const void* norm_w, float* state, void* ring, const int32_t* slots,
                                      const int32_t* query_start_loc, const int32_t* seq_lens, void* out, int32_t row0,
                                      int32_t rows, int32_t req0, int32_t num_reqs, int32_t max_query_len, int32_t heads,
                                      int32_t kv_heads, int32_t dim, int32_t vdim, int32_t taps, float eps, void* workspace,
                                      int64_t workspace_bytes, int dtype, void* stream) {
  if (num_reqs == 0 || rows == 0) return MI_OK;
  if (!proj || !conv_w || !a_log || !dt_bias || !norm_w || !state || !ring || !slots || !query_start_loc || !seq_lens || !out ||
      !workspace)
    return MI_ERR_INVALID_ARG;
  if (req0 < 0 || num_reqs < 0 || row0 < 0 || rows < 0 || max_query_len <= 0 || heads <= 0 || kv_heads <= 0 || taps <= 0 ||
      heads % kv_heads)
    return MI_ERR_INVALID_ARG;
  ChunkLayout lay;
  if (!chunk_layout(dim, vdim, &lay)) return MI_ERR_UNSUPPORTED;
  if (workspace_bytes < mi_gated_delta_chunked_workspace_bytes(rows, num_reqs, heads, dim, vdim)) return MI_ERR_WORKSPACE;
  const int CH = 2 * kv_heads * dim + heads * vdim;
  if (proj_stride < CH + heads * vdim + 2 * heads) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  const DeltaParams p{proj, conv_w, norm_w, ring, out, a_log, dt_bias, state, slots, query_start_loc, seq_lens, proj_stride, req0,
                      heads, kv_heads, dim, vdim, taps, CH, CH, CH + heads * vdim, CH + heads * vdim + heads, eps};
  hipStream_t s = (hipStream_t)stream;
  float* ws = (float*)workspace;
  const int ldk = lay.Dp + 4, ldv = lay.Vp + 4, ldm = kC + 4;
  const size_t lds = (size_t)(kC * (ldk > ldv ? ldk : ldv) + kC * (ldk > 2 * ldm ? ldk : 2 * ldm) + 5 * kC) * 4;
  const int al = (dtype == MI_DTYPE_BF16 ? 8 : 4);
  const bool vec = dim % 8 == 0 && vdim % 8 == 0 && proj_stride % al == 0 && CH % al == 0 && aligned16(proj) && aligned16(conv_w) &&
                   aligned16(ring);
  const dim3 pg((max_query_len + kC - 1) / kC, heads, num_reqs);
#define MI_PREP(T)                                                                                                        \
  do {                                                                                                                    \
    auto kern = gated_delta_prep_kernel<T>;                                                                               \
    if (hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) \
      return MI_ERR_LAUNCH;                                                                                               \
    hipLaunchKernelGGL(kern, pg, dim3(kPrepThreads), lds, s, p, ws, lay, vec);                                               \
  } while (0)
  if (dtype == MI_DTYPE_BF16) MI_PREP(uint16_t);
  else MI_PREP(float);
#undef MI_PREP
  // two value tiles a workgroup where that still leaves one for every CU
  const int nvt = lay.Vp / 16, nv = nvt % 2 == 0 && (int64_t)num_reqs * heads * (nvt / 2) >= 256 ? 2 : 1, nvg = nvt / nv;
  const dim3 sg((heads + 7) / 8 * 8 * nvg, num_reqs);
#define MI_SCAN(DT)                                                                                                            \
  do {                                                                                                                         \
    if (nv == 2) hipLaunchKernelGGL((gated_delta_scan_kernel<DT, 2>), sg, dim3(256), 0, s, p, ws, lay, nvg);                   \
    else hipLaunchKernelGGL((gated_delta_scan_kernel<DT, 1>), sg, dim3(256), 0, s, p, ws, lay, nvg);                           \
  } while (0)
  switch (lay.Dp / 16) {
    case 2: MI_SCAN(2); break;
    case 4: MI_SCAN(4); break;
    case 8: MI_SCAN(8); break;
    default: MI_SCAN(16); break;
  }
#undef MI_SCAN
  const dim3 fg((unsigned)(((int64_t)rows * heads + 3) / 4)), rg((CH + 255) / 256, num_reqs);
  const dim3 f8((unsigned)(((int64_t)rows * heads + 15) / 16));
  const bool vecf = vec && aligned16(out) && aligned16(norm_w);
#define MI_FINISH(T)                                                                                                              \
  do {                                                                                                                            \
    if (vecf && vdim <= 128) hipLaunchKernelGGL((gated_delta_finish8_kernel<T, 1>), f8, dim3(256), 0, s, p, ws, lay, num_reqs, row0, rows);   \
    else if (vecf) hipLaunchKernelGGL((gated_delta_finish8_kernel<T, 2>), f8, dim3(256), 0, s, p, ws, lay, num_reqs, row0, rows);             \
    else hipLaunchKernelGGL((gated_delta_finish_kernel<T>), fg, dim3(256), 0, s, p, ws, lay, num_reqs, row0, rows);                           \
  } while (0)
  if (dtype == MI_DTYPE_BF16) {
    MI_FINISH(uint16_t);
    hipLaunchKernelGGL((conv_ring_update_kernel<uint16_t>), rg, dim3(256), 0, s, p);
  } else {
    MI_FINISH(float);
    hipLaunchKernelGGL((conv_ring_update_kernel<float>), rg, dim3(256), 0, s, p);
  }
#undef MI_FINISH
  return launch_status();
}
