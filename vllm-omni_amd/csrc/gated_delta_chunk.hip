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
//   * finish: o / rms(o) * norm * gate.
// With one decay per key channel G_i is a vector: e^(G_i) and e^(G_C - G_i) scale the columns of K and Q, and A and P take
// sum_d k_id e^(G_id - G_jd) k_jd, whose exponential is split between j and i so that no factor exceeds one.
// All products run on v_mfma_f32_16x16x4_f32: q, k, decays and state are 32-bit quantities of the recurrence.  The k order
// inside 16 consecutive k is permuted alike in both operands (step s takes k = 4 (lane / 16) + s), so an operand whose k is
// contiguous is one 16-byte read for four steps, and an accumulator tile IS the B operand of a following product.
#include "chunk_scan.h"
#include "gated_delta.h"

namespace mi {
namespace {

// threads of a prep workgroup: two workgroups a CU, or one (whose cumulative decays take the LDS of the second) of twice the size
template <bool CHN>
constexpr int prep_threads() { return CHN ? 1024 : 512; }

// conv + silu of channels [ch0, ch0 + n) of the chunk's rows into buf [C][ld]; zeros in rows past len and columns past n
template <typename T, int NT>
__device__ __forceinline__ void conv_rows(const DeltaParams& p, float* buf, int ld, int np, int ch0, int n, int64_t row0, int i0,
                                          int len, int start, const T* ring) {
  const T* proj = reinterpret_cast<const T*>(p.proj);
  const T* cw = reinterpret_cast<const T*>(p.convw);
  const int segs = NT / np > 0 ? NT / np : 1;      // row segments worked on side by side
  const int rows_per = (kC + segs - 1) / segs;
  for (int item = threadIdx.x; item < segs * np; item += NT) {
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

// The same, 8 channels of two rows a thread, NB blocks of channels at once: all loads of a thread are unconditional (clamped
// addresses, values selected afterwards) and independent, so a trip costs one memory latency.  Needs n, the channel offsets
// and the row strides to be multiples of 8; the blocks share np and n.
template <typename T, int NT, int TAPS, int NB>
__device__ __forceinline__ void conv_rows8(const DeltaParams& p, float* const (&buf)[NB], const int (&ch0)[NB], int ld, int np, int n,
                                           int64_t row0, int i0, int len, int start, const T* ring) {
  const T* proj = reinterpret_cast<const T*>(p.proj) + row0 * p.ld;
  const T* cw = reinterpret_cast<const T*>(p.convw);
  const int per = np / 8;
  for (int item = threadIdx.x; item < kC / 2 * per; item += NT) {
    const int c = (item % per) * 8, i = item / per * 2;
    float wf[NB][8 * TAPS], x[NB][TAPS + 1][8];
    bool in[TAPS + 1];
#pragma unroll
    for (int t = 0; t <= TAPS; ++t) {
      const int k = min(i - (TAPS - 1) + t, len - 1), pos = start + i0 + k;
      in[t] = pos >= 0;
      const int64_t at = i0 + k >= 0 ? k * p.ld : 0, rat = (int64_t)(max(pos, 0) % TAPS) * p.CH;
#pragma unroll
      for (int b = 0; b < NB; ++b) {
        const int ch = ch0[b] + min(c, n - 8);
        Io<T>::template ldv<8>((i0 + k >= 0 ? proj + at : ring + rat) + ch, x[b][t]);
      }
    }
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
      for (int t = 0; t < TAPS; ++t)
        Io<T>::template ldv<8>(cw + (int64_t)(ch0[b] + min(c, n - 8)) * TAPS + 8 * t, *reinterpret_cast<float(*)[8]>(wf[b] + 8 * t));
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
      for (int r = 0; r < 2; ++r) {
        float acc[8] = {};
#pragma unroll
        for (int t = 0; t < TAPS; ++t)
#pragma unroll
          for (int j = 0; j < 8; ++j) acc[j] += in[t + r] ? wf[b][j * TAPS + t] * x[b][t + r][j] : 0.f;
        const bool live = c < n && i + r < len;
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[j] = live ? silu_f(acc[j]) : 0.f;
        Io<float>::stv<8>(buf[b] + (i + r) * ld + c, acc);
      }
  }
}

template <typename T, int NT, int NB>
__device__ __forceinline__ void conv_tiles(const DeltaParams& p, bool vec, float* const (&buf)[NB], const int (&ch0)[NB], int ld, int np, int n,
                                           int64_t row0, int i0, int len, int start, const T* ring) {
  if constexpr (sizeof(T) == 4 && NB > 1) {      // twice the registers a value: one block at a time
#pragma unroll
    for (int b = 0; b < NB; ++b) conv_tiles<T, NT, 1>(p, vec, {buf[b]}, {ch0[b]}, ld, np, n, row0, i0, len, start, ring);
    return;
  }
  if (vec && p.taps == 4) conv_rows8<T, NT, 4, NB>(p, buf, ch0, ld, np, n, row0, i0, len, start, ring);
  else if (vec && p.taps == 3) conv_rows8<T, NT, 3, NB>(p, buf, ch0, ld, np, n, row0, i0, len, start, ring);
  else if (vec && p.taps == 2) conv_rows8<T, NT, 2, NB>(p, buf, ch0, ld, np, n, row0, i0, len, start, ring);
  else
#pragma unroll
    for (int b = 0; b < NB; ++b) conv_rows<T, NT>(p, buf[b], ld, np, ch0[b], n, row0, i0, len, start, ring);
}

// rows of buf made unit vectors (16 lanes a row), then times mul
template <int NT>
__device__ __forceinline__ void unit_rows(float* buf, int ld, int np, float mul) {
  const int sub = threadIdx.x & 15;
  for (int i = threadIdx.x >> 4; i < kC; i += NT / 16) {
    float ss = 0.f;
    for (int c = sub; c < np; c += 16) ss += buf[i * ld + c] * buf[i * ld + c];
    ss = group_allreduce_sum<16>(ss);
    const float f = mul / sqrtf(ss + 1e-6f);
    for (int c = sub; c < np; c += 16) buf[i * ld + c] *= f;
  }
}

// A and P of one 16 x 16 tile (rows ti, columns tj < ti) with a decay per key channel.  e^(G_i - G_j) is split at the tile's
// entry: e^(sum of the row's tile up to i) on the row's side, what is left of tile tj behind j and the tiles between on the
// column's; all of these are sums of log decays, <= 0.  kb, qb, gb: [C][ld] keys, queries, log2 decays summed from the
// start of each 16-row tile (sums over a whole chunk would leave differences of large numbers).
__device__ __forceinline__ void channel_tile(const float* kb, const float* qb, const float* gb, int ld, int Dp, int ti,
                                             int tj, int lane, f32x4_t& aA, f32x4_t& aP) {
  for (int k = 0; k < Dp; k += 16) {
    float kf[4], qf[4], gf[4], cf[4], hf[4], lf[4], bf[4];
    frag_rows(kb + ti * 16 * ld + k, ld, lane, kf);
    frag_rows(qb + ti * 16 * ld + k, ld, lane, qf);
    frag_rows(gb + ti * 16 * ld + k, ld, lane, gf);
    frag_rows(kb + tj * 16 * ld + k, ld, lane, cf);
    frag_rows(gb + tj * 16 * ld + k, ld, lane, hf);
    frag_rows(gb + (tj * 16 + 15) * ld + k, 0, lane, lf);
    for (int s = 0; s < 4; ++s) bf[s] = 0.f;
    for (int t = tj + 1; t < ti; ++t) {
      float mf[4];
      frag_rows(gb + (t * 16 + 15) * ld + k, 0, lane, mf);
#pragma unroll
      for (int s = 0; s < 4; ++s) bf[s] += mf[s];
    }
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const float e = fast_exp2(gf[s]);
      kf[s] *= e, qf[s] *= e;
      cf[s] *= fast_exp2((lf[s] - hf[s]) + bf[s]);
    }
    aA = mma4(kf, cf, aA);
    aP = mma4(qf, cf, aP);
  }
}

// the same on the diagonal (ti == tj), by levels of halving: pairs (i, j) whose highest differing bit is `half` are split at the
// first row of the upper half of their block of 2 half rows.  A lane's token is in a row's role (upper half) or a column's
// (lower half) on each level, so one exponential per level serves both.  Levels lv0 and lv0 + 1; dg: q_i . k_i of the lane's token.
__device__ __forceinline__ void channel_diag(const float* kb, const float* qb, const float* gb, int ld, int Dp, int ti, int lv0, int lane,
                                             f32x4_t (&aA)[2], f32x4_t (&aP)[2], float& dg) {
  const int t = lane & 15;
  const float* g0 = gb + ti * 16 * ld;
  dg = 0.f;
  for (int k = 0; k < Dp; k += 16) {
    float kf[4], qf[4], gf[4];
    frag_rows(kb + ti * 16 * ld + k, ld, lane, kf);
    frag_rows(qb + ti * 16 * ld + k, ld, lane, qf);
    frag_rows(g0 + k, ld, lane, gf);
#pragma unroll
    for (int s = 0; s < 4; ++s) dg += qf[s] * kf[s];
#pragma unroll
    for (int l = 0; l < 2; ++l) {
      const int half = 1 << (lv0 + l), ref = (t & ~(2 * half - 1)) + half;
      const bool up = t & half;
      const float4 rv = *reinterpret_cast<const float4*>(g0 + ref * ld + k + 4 * (lane >> 4));
      const float rf[4] = {rv.x, rv.y, rv.z, rv.w};
      float rk[4], rq[4], ck[4];
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        const float d = gf[s] - rf[s], e = fast_exp2(up ? d : -d);
        rk[s] = up ? kf[s] * e : 0.f;
        rq[s] = up ? qf[s] * e : 0.f;
        ck[s] = up ? 0.f : kf[s] * e;
      }
      aA[l] = mma4(rk, ck, aA[l]);
      aP[l] = mma4(rq, ck, aP[l]);
    }
  }
  dg += __shfl_xor(dg, 16, 64);
  dg += __shfl_xor(dg, 32, 64);
}

// entry (4 (lane / 16) + s, lane % 16) of a diagonal tile belongs to the wave of levels lv0, lv0 + 1 (below the diagonal: their
// pairs; the wave of the lower levels also has the diagonal and what is above)
__device__ __forceinline__ bool diag_owner(int i, int j, int lv0) { return i > j ? ((i ^ j) >= 4) == (lv0 == 2) : lv0 == 0; }

// ln(1 + e^x), hardware exponential and logarithm; a series where 1 + e^-|x| would round the small term away
__device__ __forceinline__ float softplus_fast(float x) {
  const float e = fast_exp2(-fabsf(x) * kLog2e);
  const float s = e * (1.f - e * (0.5f - e * (0.33333334f - e * (0.25f - e * (0.2f - e * 0.16666667f)))));
  return fmaxf(x, 0.f) + (e < 0.0625f ? s : __builtin_amdgcn_logf(1.f + e) * 0.69314718f);
}

// CHN: one decay per head and key channel
template <typename T, bool CHN>
__global__ __launch_bounds__(prep_threads<CHN>(), 4) void gated_delta_prep_kernel(const DeltaParams p, float* ws, const ChunkLayout lay, bool vec) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) float lds[];
  constexpr int NT = prep_threads<CHN>();
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
  float* bufG = sD + kC;                   // CHN: log2 decays per channel, summed from the start of each 16-row tile
  float* sPre = bufG + kC * ldk;           // CHN: [4][Dp] sums of the tiles in front of a tile, and of those behind it
  float* sSuf = sPre + 4 * Dp;
  float* out = ws + ((chunk_base(p, r) + ck) * p.H + h) * lay.size();
  const T* ring = reinterpret_cast<const T*>(p.ring) + (int64_t)p.slots[r] * p.taps * p.CH;
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int kh = h / (p.H / p.K);
  // what the gates take, asked for in front of the convolutions
  const float raw_b = Io<T>::ld(reinterpret_cast<const T*>(p.b) + (row0 + min(lane, len - 1)) * p.ld_b + h);
  const float raw_a = CHN ? 0.f : Io<T>::ld(reinterpret_cast<const T*>(p.a) + (row0 + min(lane, len - 1)) * p.ld_a + h);
  conv_tiles<T, NT, 2>(p, vec, {bufA, bufB}, {p.K * p.D + kh * p.D, kh * p.D}, ldk, Dp, p.D, row0, i0, len, start, ring);
  if (!CHN && wave == 0) {   // gates: cumulative log decay over the 64 tokens of the chunk
    float lg = 0.f, b = 0.f;
    if (lane < len) {
      lg = -expf(p.a_log[h]) * softplus_f(raw_a + p.dt_bias[h]);
      b = sigmoid_f(raw_b);
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
    const float last = __shfl(e, 63, 64);
    for (int d = lane; d < Dp; d += 64) out[lay.g() + d] = last;
  }
  if constexpr (CHN) {
    const float neg_a = -expf(p.a_log[h]) * kLog2e;
    const T* ar = reinterpret_cast<const T*>(p.a) + row0 * p.ld_a + (int64_t)h * p.D;
    // (a decay below 2^-64 forgets as completely in 32 bits, and keeps the sums short)
    if (vec) {
      for (int n = tid; n < kC / 2 * Dp / 8; n += NT) {      // two rows a trip
        const int i = n / (Dp / 8), c = n % (Dp / 8) * 8;
        float v[2][8], dt[8];
#pragma unroll
        for (int r = 0; r < 2; ++r) Io<T>::template ldv<8>(ar + (int64_t)min(i + kC / 2 * r, len - 1) * p.ld_a + min(c, p.D - 8), v[r]);
        Io<float>::ldv<8>(p.dt_bias + h * p.D + min(c, p.D - 8), dt);
#pragma unroll
        for (int r = 0; r < 2; ++r) {
          const bool in = i + kC / 2 * r < len && c < p.D;
#pragma unroll
          for (int j = 0; j < 8; ++j) v[r][j] = in ? fmaxf(neg_a * softplus_fast(v[r][j] + dt[j]), -64.f) : 0.f;
          Io<float>::stv<8>(bufG + (i + kC / 2 * r) * ldk + c, v[r]);
        }
      }
    } else {
      for (int n = tid; n < kC * Dp; n += NT) {
        const int i = n / Dp, c = n % Dp;
        const bool in = i < len && c < p.D;
        const float v = Io<T>::ld(ar + (int64_t)min(i, len - 1) * p.ld_a + min(c, p.D - 1)) + p.dt_bias[h * p.D + min(c, p.D - 1)];
        bufG[i * ldk + c] = in ? fmaxf(neg_a * softplus_fast(v), -64.f) : 0.f;
      }
    }
    if (wave == 0) sB[lane] = lane < len ? sigmoid_f(raw_b) : 0.f;
    __syncthreads();
    // running sums over each 16-row tile, a segment of a tile's rows a thread, then the tile's segments in front
    const int segs = NT / Dp, c = tid % Dp, sg = tid / Dp, per = kC / segs;     // per <= 16: Dp <= 128
    float acc = 0.f;
    for (int i = sg * per; i < (sg + 1) * per; ++i) acc += bufG[i * ldk + c], bufG[i * ldk + c] = acc;
    __syncthreads();
    float before = 0.f;
    for (int n = sg * per / 16 * 16 / per; n < sg; ++n) before += bufG[(n * per + per - 1) * ldk + c];
    __syncthreads();
    for (int i = sg * per; i < (sg + 1) * per; ++i) bufG[i * ldk + c] += before;
    __syncthreads();
    if (tid < Dp) {
      float e[4], a = 0.f, b = 0.f;
#pragma unroll
      for (int t = 0; t < 4; ++t) e[t] = bufG[(16 * t + 15) * ldk + tid];
#pragma unroll
      for (int t = 0; t < 4; ++t) sPre[t * Dp + tid] = a, a += e[t];
#pragma unroll
      for (int t = 3; t >= 0; --t) sSuf[t * Dp + tid] = b, b += e[t];
      out[lay.g() + tid] = fast_exp2(a);
    }
  }
  __syncthreads();
  unit_rows<NT>(bufA, ldk, Dp, 1.0f);
  unit_rows<NT>(bufB, ldk, Dp, 1.0f / sqrtf((float)p.D));
  __syncthreads();
  // A and P, 16 tiles each, lower ones only: P goes out, A waits in registers until Q is dead
  f32x4_t keep[2] = {};
  if constexpr (CHN) {
    auto store = [&](int ti, int tj, int s, float a, float pv, f32x4_t& kp) {
      const int i = ti * 16 + 4 * (lane >> 4) + s, j = tj * 16 + (lane & 15);
      out[lay.pm() + i * kC + j] = pv;
      kp[s] = a * sB[i];
    };
    if (wave < 8) {          // a diagonal tile for two waves
      const int ti = wave & 3, lv0 = wave >> 2 << 1;
      f32x4_t aA[2] = {}, aP[2] = {};
      float dg;
      channel_diag(bufA, bufB, bufG, ldk, Dp, ti, lv0, lane, aA, aP, dg);
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        const int i = 4 * (lane >> 4) + s, j = lane & 15, x = i ^ j;
        const bool hi = x >= (lv0 ? 8 : 2);
        if (diag_owner(i, j, lv0)) store(ti, ti, s, hi ? aA[1][s] : aA[0][s], i > j ? (hi ? aP[1][s] : aP[0][s]) : i == j ? dg : 0.f, keep[0]);
      }
    } else if (wave < 14) {
      const int t = wave - 8, ti = t < 1 ? 1 : t < 3 ? 2 : 3, tj = t - ti * (ti - 1) / 2;
      f32x4_t aA = {}, aP = {};
      channel_tile(bufA, bufB, bufG, ldk, Dp, ti, tj, lane, aA, aP);
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        store(ti, tj, s, aA[s], aP[s], keep[0]);
        out[lay.pm() + (tj * 16 + 4 * (lane >> 4) + s) * kC + ti * 16 + (lane & 15)] = 0.f;   // its mirror: whole rows of P are multiplied
      }
    }
  }
#pragma unroll
  for (int n = 0; n < (CHN ? 0 : 4); ++n) {
    const int t = wave + n * (NT / 64);
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
  for (int n = tid; n < kC * Dp / 4; n += NT) {
    const int i = n / (Dp / 4), c = (n % (Dp / 4)) * 4;
    float4 v = *reinterpret_cast<const float4*>(bufB + i * ldk + c);
    if constexpr (CHN) {
      const float4 g = *reinterpret_cast<const float4*>(bufG + i * ldk + c), b = *reinterpret_cast<const float4*>(sPre + (i >> 4) * Dp + c);
      v = make_float4(v.x * fast_exp2(g.x + b.x), v.y * fast_exp2(g.y + b.y), v.z * fast_exp2(g.z + b.z), v.w * fast_exp2(g.w + b.w));
    } else {
      const float e = sQ[i];
      v = make_float4(v.x * e, v.y * e, v.z * e, v.w * e);
    }
    *reinterpret_cast<float4*>(out + lay.q() + (int64_t)i * Dp + c) = v;
  }
  for (int n = tid; n < kC * Dp; n += NT) {
    const int d = n / kC, j = n % kC;
    const float e = CHN ? fast_exp2((bufG[(j | 15) * ldk + d] - bufG[j * ldk + d]) + sSuf[(j >> 4) * Dp + d]) : sD[j];
    out[lay.kt() + n] = j < len ? bufA[j * ldk + d] * e : 0.f;
  }
  __syncthreads();   // Q is dead: A and T take its place
  if constexpr (CHN) {   // and nobody needs the plain keys again
    for (int n = tid; n < kC * Dp; n += NT) {
      const int i = n / Dp, c = n % Dp;
      bufA[i * ldk + c] *= fast_exp2(bufG[i * ldk + c] + sPre[(i >> 4) * Dp + c]);
    }
    if (wave < 14) {
      const int t = wave - 8, ti = wave < 8 ? wave & 3 : t < 1 ? 1 : t < 3 ? 2 : 3, tj = wave < 8 ? ti : t - ti * (ti - 1) / 2;
#pragma unroll
      for (int s = 0; s < 4; ++s) {
        const int i = 4 * (lane >> 4) + s, j = lane & 15;
        if (wave >= 8 || (i > j && diag_owner(i, j, wave >> 2 << 1))) mA[(ti * 16 + i) * ldm + tj * 16 + j] = keep[0][s];
      }
    }
  }
#pragma unroll
  for (int n = 0; n < (CHN ? 0 : 2); ++n) {
    const int t = wave + n * (NT / 64);
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
    for (int t = wave; t < 4 * nt; t += NT / 64) {
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
  times(CHN ? sB : sE, ldk, Dp, out + lay.w());
  __syncthreads();
  conv_tiles<T, NT, 1>(p, vec, {bufA}, {2 * p.K * p.D + h * p.V}, ldv, Vp, p.V, row0, i0, len, start, ring);
  __syncthreads();
  times(sB, ldv, Vp, out + lay.u());
}

// the read-out of (row, head), where the scan left it
__device__ __forceinline__ const float* readout(const DeltaParams& p, const float* ws, const ChunkLayout& lay, int nreq, int row, int h) {
  const int r = p.req0 + row_request(p.qsl + p.req0, nreq, row);
  const int i = row - p.qsl[r];
  return ws + ((chunk_base(p, r) + i / kC) * p.H + h) * lay.size() + lay.u() + (int64_t)(i % kC) * lay.Vp;
}

// out = o / rms(o) * norm * gate, 16 lanes per (row, head), 8 values a lane at a time; vdim a multiple of 8, <= 128 U
template <typename T, int U>
__global__ __launch_bounds__(256) void gated_delta_finish8_kernel(const DeltaParams p, const float* ws, const ChunkLayout lay, int nreq, int row0, int rows) {
  scalar_cache_acquire();
  const int64_t item = (int64_t)blockIdx.x * 16 + (threadIdx.x >> 4);
  const int sub = threadIdx.x & 15;
  if (item >= (int64_t)rows * p.H) return;     // whole 16-lane groups leave
  const int64_t row = row0 + item / p.H;
  const int h = (int)(item % p.H);
  const float* x = readout(p, ws, lay, nreq, (int)row, h);
  const T* g = reinterpret_cast<const T*>(p.gate) + row * p.ld_gate + h * p.V;
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
  T* out = reinterpret_cast<T*>(p.out) + row * p.ld_out + (int64_t)h * p.V;
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int c = 8 * (sub + 16 * u);
    if (c >= p.V) continue;
    float w[8];
    Io<T>::template ldv<8>(reinterpret_cast<const T*>(p.norm_w) + c, w);
#pragma unroll
    for (int j = 0; j < 8; ++j) v[u][j] *= inv * w[j] * out_gate(p, gt[u][j]);
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
  const T* g = reinterpret_cast<const T*>(p.gate) + row * p.ld_gate + h * p.V;
  const T* nw = reinterpret_cast<const T*>(p.norm_w);
  T* out = reinterpret_cast<T*>(p.out) + row * p.ld_out + (int64_t)h * p.V;
  for (int v = lane; v < p.V; v += 64) Io<T>::st(out + v, x[v] * inv * Io<T>::ld(nw + v) * out_gate(p, Io<T>::ld(g + v)));
}

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int64_t mi_gated_delta_chunked_workspace_bytes(int32_t rows, int32_t num_reqs, int32_t heads, int32_t dim, int32_t vdim,
                                                          int32_t channel_decay) {
  ChunkLayout lay;
  if (rows < 0 || num_reqs < 0 || heads <= 0 || !chunk_layout(dim, vdim, &lay)) return 0;
  if (channel_decay && dim > 128) return 0;      // K, Q and the cumulative decays of a chunk must fit the LDS together
  const int64_t chunks = rows / kC + num_reqs;
  return chunks * heads * lay.size() * 4;
}

extern "C" int mi_gated_delta_chunked(const mi_gated_delta_args* args, int32_t row0, int32_t rows, int32_t max_query_len,
                                      void* workspace, int64_t workspace_bytes, int dtype, void* stream) {
  if (args && (args->num_reqs == 0 || rows == 0)) return MI_OK;
  DeltaParams p;
  const int rc = delta_fill(p, args);
  if (rc != MI_OK) return rc;
  if (!workspace || row0 < 0 || rows < 0 || max_query_len <= 0) return MI_ERR_INVALID_ARG;
  const int heads = p.H, dim = p.D, vdim = p.V, num_reqs = args->num_reqs, CH = p.CH;
  ChunkLayout lay;
  if (!chunk_layout(dim, vdim, &lay) || (p.channel && dim > 128)) return MI_ERR_UNSUPPORTED;
  if (workspace_bytes < mi_gated_delta_chunked_workspace_bytes(rows, num_reqs, heads, dim, vdim, p.channel)) return MI_ERR_WORKSPACE;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  hipStream_t s = (hipStream_t)stream;
  float* ws = (float*)workspace;
  const int ldk = lay.Dp + 4, ldv = lay.Vp + 4, ldm = kC + 4;
  const size_t lds = (size_t)(kC * (ldk > ldv ? ldk : ldv) + kC * (ldk > 2 * ldm ? ldk : 2 * ldm) + 5 * kC + (p.channel ? kC * ldk + 8 * lay.Dp : 0)) * 4;
  const int al = (dtype == MI_DTYPE_BF16 ? 8 : 4);
  const bool vec = dim % 8 == 0 && vdim % 8 == 0 && p.ld % al == 0 && CH % al == 0 && aligned16(p.proj) && aligned16(p.convw) && aligned16(p.ring) &&
                   (!p.channel || (p.ld_a % al == 0 && aligned16(p.a) && aligned16(p.dt_bias)));
  const dim3 pg((max_query_len + kC - 1) / kC, heads, num_reqs);
#define MI_PREP(T)                                                                                                        \
  do {                                                                                                                    \
    auto kern = p.channel ? gated_delta_prep_kernel<T, true> : gated_delta_prep_kernel<T, false>;                                                                               \
    if (hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) \
      return MI_ERR_LAUNCH;                                                                                               \
    hipLaunchKernelGGL(kern, pg, dim3(p.channel ? prep_threads<true>() : prep_threads<false>()), lds, s, p, ws, lay, vec);                                               \
  } while (0)
  if (dtype == MI_DTYPE_BF16) MI_PREP(uint16_t);
  else MI_PREP(float);
#undef MI_PREP
  const int sc = launch_scan<true, false>(ScanParams{p.state, p.slots, p.qsl, p.seq_lens, p.req0, heads, dim, vdim}, ws, lay, num_reqs, s);
  if (sc != MI_OK) return sc;
  const dim3 fg((unsigned)(((int64_t)rows * heads + 3) / 4)), rg((CH + 255) / 256, num_reqs);
  const dim3 f8((unsigned)(((int64_t)rows * heads + 15) / 16));
  const bool vecf = vec && p.ld_gate % al == 0 && p.ld_out % al == 0 && aligned16(p.gate) && aligned16(p.out) && aligned16(p.norm_w);
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
