// Matrix-core kernels of attention with mixed heads (bf16, heads laid out to 64 or 128): see talking_attn.hip for the
// mechanism.  Scores are kept in units of log2; the cap is cap (1 - 2 / (e^(2 s / cap) + 1)), the bias r1 log2(1 + r2 d).
//
// Decode, one row per request:
//   * decode_scores: a workgroup per (keys, kv head, request): K rows straight into MFMA operands, scores of the group's heads
//     to a workspace (a thirtieth of the keys' bytes), with the part's maximum and sum.
//   * decode_values: a workgroup per (keys, request), all heads: weights from the scores and the whole softmax's sums, mixed by
//     fp32 MFMAs (T from the left), then V rows, 16 bytes a lane, times the fp32 mixed weights on the vector units.
//   * decode_reduce: parts summed, gate.
//   Bound: HBM, every visible K and V row once.
// Prompt portions, on the visible context gathered per request (64-row aligned: K by rows, V as [16 keys] columns per value
// dimension, so that both are operands without a detour):
//   * prefill_sums: log-sum-exp of every (row, head); a wave has 16 rows of up to HW heads, no cross-lane work in the loop.
//   * prefill_mix: a workgroup has 16 rows of ALL heads, a wave HW heads.  Per 16 keys: scores and weights again (now
//     normalised), exchanged through LDS, mixed (T from the right), exchanged again, times V.
//   Bound: the vector units (cap, bias and softmax are some fourteen operations, four of them transcendental at a quarter of
//   the rate, and both sweeps do them) well ahead of the matrix cores.
// Attention weights are 32-bit quantities: in MFMA products they are bf16 pairs hi + lo, and hi and lo halves of 16 keys
// fill the 32 of one K dimension.
#include "mfma_attn_common.h"
#include "row_io.h"

namespace mi {
namespace {

using E16 = Elem<bf16_tag>;

struct ScoreMul {
  float in, out;      // cap: e^(2 s / cap) = 2^(in s), out = cap log2(e); no cap: in = scale log2(e)
};

__device__ __forceinline__ float fast_log2(float x) { return __builtin_amdgcn_logf(x); }

// score in log2 units plus base - out, distance d as a float (>= 0 where the result counts)
template <bool CAP>
__device__ __forceinline__ float score_from(float base, float s, float d, float r1, float r2, const ScoreMul& m) {
  const float b = fmaf(-r1, fast_log2(fmaf(r2, d, 1.f)), base);
  if constexpr (CAP) {
    const float t = __builtin_amdgcn_rcpf(fast_exp2(s * m.in) + 1.f);
    return fmaf(-2.f * m.out, t, b);
  } else {
    return fmaf(s, m.in, b);
  }
}
template <bool CAP>
__device__ __forceinline__ float score_of(float s, float d, float r1, float r2, const ScoreMul& m) {
  return score_from<CAP>(m.out, s, d, r1, r2, m);
}

__device__ __forceinline__ float uniform(float v) {      // the same in all lanes: a scalar register
  return __builtin_bit_cast(float, __builtin_amdgcn_readfirstlane(__builtin_bit_cast(int, v)));
}

// 16 bytes that are read once
__device__ __forceinline__ uint4 load_once(const uint16_t* p) {
  return __builtin_bit_cast(uint4, __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(p)));
}

constexpr float kFloor = -1e30f;     // stands in for the maximum of no scores

// ------------------------------------------------------------------------------------------------ decode
struct DecodeParams {
  const uint16_t* q;
  const uint16_t* kc;
  const uint16_t* vc;
  const int32_t* table;
  const int32_t* seq_lens;
  const float* r1;         // nullptr: no bias
  const float* r2;
  const float* talk;
  const uint16_t* gate;    // nullptr: none
  uint16_t* out;
  float* scores;           // [reqs][H][pitch]
  float2* ml;              // [reqs][parts1][H]
  float* part;             // [reqs][parts2 * ksplit][H][V]
  int64_t q_stride, out_stride, gate_stride, block_stride, token_stride, head_stride, table_stride;
  int H, G, V, bs_log2, window, pitch, parts1, keys1, parts2, keys2, ksplit;
  ScoreMul mul;
};

// A wave has 16 NT keys of one kv head; neighbouring waves have neighbouring kv heads.  A group of at most CW heads stands in
// the products' 16 columns 16 / CW times, and a column's lanes go on with one of 16 / CW tiles: no score is formed twice.
template <int HD, int NT, int CW, bool CAP>
__global__ __launch_bounds__(256) void decode_scores_kernel(const DecodeParams p) {
  scalar_cache_acquire();
  constexpr int KS = HD / 32, NG = 16 / CW, NP = NT / NG;
  const int lane = threadIdx.x & 63, lr = lane & 15, lg = lane >> 4, col = lr % CW, group = lr / CW;
  const int unit = __builtin_amdgcn_readfirstlane(blockIdx.x * 4 + (threadIdx.x >> 6)), req = blockIdx.y;
  const int part = unit / p.G, kv = unit % p.G;
  const int L = p.seq_lens[req], lo = max(0, L - p.window), n = L - lo;
  const int t0 = part * (16 * NT);
  if (t0 >= n) return;
  const int R = p.H / p.G;
  const int32_t* tab = p.table + (int64_t)req * p.table_stride;
  const uint16_t* kc = p.kc + kv * p.head_stride + 8 * lg;
  uint4 kf[NT][KS];
#pragma unroll
  for (int u = 0; u < NT; ++u) {
    const int key = lo + min(t0 + 16 * u + lr, n - 1);
    const uint16_t* row = kc + (int64_t)tab[key >> p.bs_log2] * p.block_stride + (int64_t)(key & ((1 << p.bs_log2) - 1)) * p.token_stride;
#pragma unroll
    for (int k = 0; k < KS; ++k) kf[u][k] = *reinterpret_cast<const uint4*>(row + 32 * k);
  }
  for (int c0 = 0; c0 < R; c0 += CW) {
    const bool used = c0 + col < R;
    const int h = kv * R + min(c0 + col, R - 1);
    const uint16_t* q = p.q + req * p.q_stride + (int64_t)h * HD;
    uint4 qf[KS];
#pragma unroll
    for (int k = 0; k < KS; ++k) qf[k] = *reinterpret_cast<const uint4*>(q + 32 * k + 8 * lg);
    const float r1 = p.r1 ? p.r1[h] : 0.f, r2 = p.r1 ? p.r2[h] : 0.f;
    float* out = p.scores + ((int64_t)req * p.H + h) * p.pitch;
    float s[NP][4];
    float m = kFloor;
#pragma unroll
    for (int u = 0; u < NP; ++u) {
#pragma unroll
      for (int g = 0; g < NG; ++g) {
        f32x4_t a = {};
#pragma unroll
        for (int k = 0; k < KS; ++k) a = mfma16<bf16_tag>(kf[u * NG + g][k], qf[k], a);
#pragma unroll
        for (int j = 0; j < 4; ++j) s[u][j] = g == 0 || group == g ? a[j] : s[u][j];
      }
      const int at = t0 + 16 * (u * NG + group) + 4 * lg;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int d = n - 1 - at - j;
        s[u][j] = d >= 0 ? score_of<CAP>(s[u][j], (float)d, r1, r2, p.mul) : -INFINITY;
        m = max2f(m, s[u][j]);
      }
      if (used) *reinterpret_cast<float4*>(out + at) = make_float4(s[u][0], s[u][1], s[u][2], s[u][3]);
    }
    m = rows_allreduce_max(m);
#pragma unroll
    for (int o = CW; o < 16; o <<= 1) m = fmaxf(m, __shfl_xor(m, o, 64));
    float l = 0.f;
#pragma unroll
    for (int u = 0; u < NP; ++u)
#pragma unroll
      for (int j = 0; j < 4; ++j) l += fast_exp2(s[u][j] - m);
    l = rows_allreduce_sum(l);
#pragma unroll
    for (int o = CW; o < 16; o <<= 1) l += __shfl_xor(l, o, 64);
    if (lane < CW && used) p.ml[((int64_t)req * p.parts1 + part) * p.H + h] = make_float2(m, l);
  }
}

inline int decode_pad(int H) { return (H + 15) / 16 * 16 + 4; }       // floats a key's mixed weights take in LDS

// RM: heads a wave accumulates at a time; HT: 16-head tiles
template <int HD, int RM, int HT>
__global__ __launch_bounds__(256) void decode_values_kernel(const DecodeParams p) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) float lds[];
  constexpr int LPR = HD / 8, KPI = 64 / LPR, UN = 4;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, lr = lane & 15, lg = lane >> 4;
  const int part = blockIdx.x, req = blockIdx.y;
  const int L = p.seq_lens[req], lo = max(0, L - p.window), n = L - lo;
  const int k0 = part * p.keys2;
  if (k0 >= n) return;
  const int H = p.H, V = p.V, R = H / p.G, pad = (H + 15) / 16 * 16 + 4, kq = (H + 3) / 4, tp = 4 * kq + 1;
  float* pm = lds;                                     // [keys2][pad]
  float* st = pm + p.keys2 * pad + 16;                 // [16 HT][tp]
  float* lse = st + 16 * HT * tp;                      // [4 kq]
  int64_t* pages = reinterpret_cast<int64_t*>(lse + 4 * kq);      // where the part's pages start in the cache
  const int first_page = (lo + k0) >> p.bs_log2, nk = min(p.keys2, n - k0);
  const int last_page = (lo + k0 + nk - 1) >> p.bs_log2;
  const int32_t* tab = p.table + (int64_t)req * p.table_stride;
  for (int i = tid; i <= last_page - first_page; i += 256) pages[i] = (int64_t)tab[first_page + i] * p.block_stride;
  for (int i = tid; i < 16 * HT * 4 * kq; i += 256) {
    const int h = i / (4 * kq), g = i % (4 * kq);
    st[h * tp + g] = h < H && g < H ? p.talk[h * H + g] : 0.f;
  }
  const int np = (n + p.keys1 - 1) / p.keys1;
  for (int h0 = 0; h0 < 4 * kq; h0 += 32) {            // eight lanes per head
    const int h = h0 + (tid >> 3);
    float m = kFloor, l = 0.f;
    if (h < H)
      for (int i = tid & 7; i < np; i += 8) {
        const float2 e = p.ml[((int64_t)req * p.parts1 + i) * H + h];
        const float mn = fmaxf(m, e.x);
        l = l * fast_exp2(m - mn) + e.y * fast_exp2(e.x - mn);
        m = mn;
      }
#pragma unroll
    for (int o = 1; o < 8; o <<= 1) {
      const float m2 = __shfl_xor(m, o, 64), l2 = __shfl_xor(l, o, 64), mn = fmaxf(m, m2);
      l = l * fast_exp2(m - mn) + l2 * fast_exp2(m2 - mn);
      m = mn;
    }
    if ((tid & 7) == 0 && h < 4 * kq) lse[h] = h < H ? m + fast_log2(l) : 0.f;
  }
  __syncthreads();
  const float* sc = p.scores + (int64_t)req * H * p.pitch + k0;
  for (int j0 = wave * 16; j0 < p.keys2; j0 += 64) {
    f32x4_t acc[HT] = {};
    const int key = j0 + lr;
    if (j0 < nk)
      for (int k = 0; k < kq; ++k) {
        const int g = 4 * k + lg;
        const float w = g < H && key < nk ? fast_exp2(sc[(int64_t)g * p.pitch + key] - lse[g]) : 0.f;
#pragma unroll
        for (int t = 0; t < HT; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(st[(16 * t + lr) * tp + g], w, acc[t], 0, 0, 0);
      }
#pragma unroll
    for (int t = 0; t < HT; ++t)
      if (16 * t < H) *reinterpret_cast<float4*>(pm + key * pad + 16 * t + 4 * lg) = make_float4(acc[t][0], acc[t][1], acc[t][2], acc[t][3]);
  }
  __syncthreads();
  // values
  const int chunks = (R + RM - 1) / RM, units = p.G * chunks;
  const int dc = lane % LPR, sub = lane / LPR;
  const int ks = p.ksplit == 1 ? 0 : wave / units, wstep = p.ksplit == 1 ? 4 : units;
  if (ks >= p.ksplit) return;
  const int span = p.keys2 / p.ksplit, jb = ks * span, je = min(jb + span, nk);
  for (int unit = p.ksplit == 1 ? wave : wave % units; unit < units; unit += wstep) {
    const int kv = unit / chunks, r0 = (unit % chunks) * RM, h0 = kv * R + r0;
    const uint16_t* vc = p.vc + kv * p.head_stride + dc * 8;
    float acc[RM][8] = {};
    for (int j0 = jb; j0 < je; j0 += KPI * UN) {
      uint4 v[UN];
#pragma unroll
      for (int u = 0; u < UN; ++u) {
        const int key = lo + k0 + min(j0 + u * KPI + sub, nk - 1);
        v[u] = load_once(vc + pages[(key >> p.bs_log2) - first_page] + (int64_t)(key & ((1 << p.bs_log2) - 1)) * p.token_stride);
      }
#pragma unroll
      for (int u = 0; u < UN; ++u) {
        // (mixed weights of keys past the last are zeros; splits of the part are multiples of a round of loads)
        const float* w = pm + (j0 + u * KPI + sub) * pad + h0;
        const uint32_t a[4] = {v[u].x, v[u].y, v[u].z, v[u].w};
        float x[8];
#pragma unroll
        for (int i = 0; i < 4; ++i) x[2 * i] = E16::lo(a[i]), x[2 * i + 1] = E16::hi(a[i]);
#pragma unroll
        for (int r = 0; r < RM; ++r) {
#pragma unroll
          for (int i = 0; i < 8; ++i) acc[r][i] = fmaf(w[r], x[i], acc[r][i]);
        }
      }
    }
    float* out = p.part + (((int64_t)req * p.parts2 + part) * p.ksplit + ks) * H * V;
#pragma unroll
    for (int r = 0; r < RM; ++r) {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        float a = acc[r][i];
        if constexpr (HD == 64) a += __shfl_xor(a, 8, 64);
        acc[r][i] = rows_allreduce_sum(a);
      }
      if (sub == 0 && r0 + r < R) {
        float* o = out + (int64_t)(h0 + r) * V + dc * 8;
        if (V % 8 == 0) {
          if (dc * 8 < V) {
            *reinterpret_cast<float4*>(o) = make_float4(acc[r][0], acc[r][1], acc[r][2], acc[r][3]);
            *reinterpret_cast<float4*>(o + 4) = make_float4(acc[r][4], acc[r][5], acc[r][6], acc[r][7]);
          }
        } else {
#pragma unroll
          for (int i = 0; i < 8; ++i)
            if (dc * 8 + i < V) o[i] = acc[r][i];
        }
      }
    }
  }
}

__global__ __launch_bounds__(256) void decode_reduce_kernel(const DecodeParams p) {
  scalar_cache_acquire();
  const int i = blockIdx.x * 256 + threadIdx.x, req = blockIdx.y, hv = p.H * p.V;
  if (i >= hv) return;
  const int L = p.seq_lens[req], n = min(L, p.window);
  const int np = (n + p.keys2 - 1) / p.keys2 * p.ksplit;      // no keys (a padded row of a graph replay): zeros
  const float* x = p.part + (int64_t)req * p.parts2 * p.ksplit * hv + i;
  float s = 0.f;
  int k = 0;
  for (; k + 4 <= np; k += 4) {
    const float a = x[(int64_t)k * hv], b = x[(int64_t)(k + 1) * hv], c = x[(int64_t)(k + 2) * hv], d = x[(int64_t)(k + 3) * hv];
    s += (a + b) + (c + d);
  }
  for (; k < np; ++k) s += x[(int64_t)k * hv];
  if (p.gate) s *= sigmoid_f(E16::from_bits(p.gate[req * p.gate_stride + i]));
  p.out[req * p.out_stride + i] = E16::to_bits(s);
}

// ------------------------------------------------------------------------------------------------ prompt portions
struct PrefillParams {
  const uint16_t* q;       // [rows][q_stride], heads HD apart
  const uint16_t* k;       // [G][ctx_rows][HD]
  const uint16_t* vt;      // [G][ctx_rows / 16][HD][16]
  float* lse;              // [H][rows]
  const int32_t* ctx_start;
  const int32_t* seq_lens;
  const int32_t* qsl;
  const float* r1;         // nullptr: no bias
  const float* r2;
  const float* talk;
  const uint16_t* gate;    // nullptr: none
  uint16_t* out;
  int64_t q_stride, out_stride, gate_stride;
  int H, G, V, window, rows, ctx_rows, reqs, max_q;
  ScoreMul mul;
};

struct GatherParams {
  uint16_t* k;
  uint16_t* vt;
  const uint16_t* kc;
  const uint16_t* vc;
  const int32_t* ctx_start;
  const int32_t* table;
  const int32_t* seq_lens;
  const int32_t* qsl;
  int64_t block_stride, token_stride, head_stride, table_stride;
  int reqs, ctx_rows, bs_log2, window;
};

template <int HD>
__global__ __launch_bounds__(256) void gather_kernel(const GatherParams p) {
  scalar_cache_acquire();
  constexpr int LV = HD + 2, CH = HD / 8;
  __shared__ uint32_t sv[64 * LV / 2];
  uint16_t* s16 = reinterpret_cast<uint16_t*>(sv);
  const int i0 = blockIdx.x * 64, g = blockIdx.y, tid = threadIdx.x;
  const int r = row_request(p.ctx_start, p.reqs, i0);
  const int L = p.seq_lens[r], first = max(0, L - (p.qsl[r + 1] - p.qsl[r]) - p.window + 1);
  const int32_t* tab = p.table + r * p.table_stride;
#pragma unroll
  for (int it = 0; it < 64 * CH / 256; ++it) {
    const int item = it * 256 + tid, i = item / CH, c = item % CH * 8;
    const int pos = first + i0 + i - p.ctx_start[r];
    uint4 a = make_uint4(0, 0, 0, 0), b = a;
    if (pos < L) {
      const int64_t at = (int64_t)tab[pos >> p.bs_log2] * p.block_stride + (int64_t)(pos & ((1 << p.bs_log2) - 1)) * p.token_stride +
                         g * p.head_stride + c;
      a = *reinterpret_cast<const uint4*>(p.kc + at);
      b = *reinterpret_cast<const uint4*>(p.vc + at);
    }
    *reinterpret_cast<uint4*>(p.k + ((int64_t)g * p.ctx_rows + i0 + i) * HD + c) = a;
    uint32_t* d = sv + (i * LV + c) / 2;
    d[0] = b.x, d[1] = b.y, d[2] = b.z, d[3] = b.w;
  }
  __syncthreads();
  uint16_t* vt = p.vt + ((int64_t)g * p.ctx_rows + i0) * HD;      // four tiles of [HD][16]
#pragma unroll
  for (int it = 0; it < 64 * CH / 256; ++it) {
    const int item = it * 256 + tid, half = item & 1, d = (item >> 1) % HD, t = (item >> 1) / HD;
    uint32_t w[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int i = t * 16 + half * 8 + 2 * j;
      w[j] = (uint32_t)s16[i * LV + d] | (uint32_t)s16[(i + 1) * LV + d] << 16;
    }
    *reinterpret_cast<uint4*>(vt + ((int64_t)t * HD + d) * 16 + half * 8) = make_uint4(w[0], w[1], w[2], w[3]);
  }
}

// 16 query rows: where they are and which context rows they see
struct TileSpan {
  int s0, ql, tile0, start, first, c0, kb, ke;
  bool any;
};

__device__ __forceinline__ TileSpan tile_span(const PrefillParams& p, int r, int tile0) {
  TileSpan t;
  t.s0 = p.qsl[r], t.ql = p.qsl[r + 1] - t.s0, t.tile0 = tile0;
  t.any = tile0 < t.ql;
  const int L = p.seq_lens[r];
  t.start = L - t.ql;
  t.first = max(0, t.start - p.window + 1);
  t.c0 = p.ctx_start[r];
  const int q_lo = t.start + tile0;
  t.kb = max(0, q_lo - p.window + 1 - t.first) & ~15;
  t.ke = t.start + min(tile0 + 15, t.ql - 1) - t.first;
  return t;
}

// K operands of one 16-key tile
template <int HD>
__device__ __forceinline__ void load_k(uint4 (&kf)[HD / 32], const PrefillParams& p, int kv, int row, int lr, int lg) {
  const uint16_t* k = p.k + ((int64_t)kv * p.ctx_rows + row + lr) * HD + 8 * lg;
#pragma unroll
  for (int i = 0; i < HD / 32; ++i) kf[i] = *reinterpret_cast<const uint4*>(k + 32 * i);
}

template <int HD>
__device__ __forceinline__ f32x4_t qk(const uint4 (&kf)[HD / 32], const uint4 (&qf)[HD / 32]) {
  f32x4_t a = {};
#pragma unroll
  for (int i = 0; i < HD / 32; ++i) a = mfma16<bf16_tag>(kf[i], qf[i], a);
  return a;
}

// HW heads per wave; ONE: they share a kv head
template <int HD, int HW, bool ONE, bool CAP>
__global__ __launch_bounds__(256) void prefill_sums_kernel(const PrefillParams p) {
  scalar_cache_acquire();
  constexpr int KS = HD / 32;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lr = lane & 15, lg = lane >> 4;
  // late tiles (long rows) of all portions first; a group of heads stays on its XCD
  const int groups = (p.H + HW - 1) / HW, at = blockIdx.x / groups;
  const int h0 = (blockIdx.x % groups) * HW, r = at % p.reqs, R = p.H / p.G;
  const TileSpan t = tile_span(p, r, ((p.max_q + 63) / 64 - 1 - at / p.reqs) * 64 + wave * 16);
  if (!t.any) return;
  const int qi = min(t.tile0 + lr, t.ql - 1), qpos = t.start + t.tile0 + lr;
  const uint16_t* q = p.q + (int64_t)(t.s0 + qi) * p.q_stride + 8 * lg;
  uint4 qf[HW][KS];
  float m[HW], l[HW], r1[HW], r2[HW];
#pragma unroll
  for (int i = 0; i < HW; ++i) {
    const int h = min(h0 + i, p.H - 1);
#pragma unroll
    for (int k = 0; k < KS; ++k) qf[i][k] = *reinterpret_cast<const uint4*>(q + h * HD + 32 * k);
    m[i] = kFloor, l[i] = 0.f;
    r1[i] = uniform(p.r1 ? p.r1[h] : 0.f), r2[i] = uniform(p.r1 ? p.r2[h] : 0.f);
  }
  uint4 kf[KS];
  load_k<HD>(kf, p, h0 / R, t.c0 + t.kb, lr, lg);
  for (int k0 = t.kb; k0 <= t.ke; k0 += 16) {
    f32x4_t s[HW];
#pragma unroll
    for (int i = 0; i < HW; ++i) {
      if (!ONE && i > 0) load_k<HD>(kf, p, min(h0 + i, p.H - 1) / R, t.c0 + k0, lr, lg);
      s[i] = qk<HD>(kf, qf[i]);
    }
    if (k0 + 16 <= t.ke) load_k<HD>(kf, p, h0 / R, t.c0 + k0 + 16, lr, lg);
    const int key0 = t.first + k0, d0 = qpos - key0 - 4 * lg;
    const bool inside = key0 + 15 <= t.start + t.tile0 && t.start + t.tile0 + 15 - key0 < p.window;
    const float fd = (float)d0;
#pragma unroll
    for (int i = 0; i < HW; ++i) {
      float u[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) u[j] = score_of<CAP>(s[i][j], fd - (float)j, r1[i], r2[i], p.mul);
      if (!inside) {
        asm volatile("");      // stays a branch
#pragma unroll
        for (int j = 0; j < 4; ++j) u[j] = (unsigned)(d0 - j) < (unsigned)p.window ? u[j] : -INFINITY;
      }
      const float mn = max3f(max3f(m[i], u[0], u[1]), u[2], u[3]);
      l[i] = l[i] * fast_exp2(m[i] - mn) +
             ((fast_exp2(u[0] - mn) + fast_exp2(u[1] - mn)) + (fast_exp2(u[2] - mn) + fast_exp2(u[3] - mn)));
      m[i] = mn;
    }
  }
#pragma unroll
  for (int i = 0; i < HW; ++i) {
    const float mm = rows_allreduce_max(m[i]);
    const float ll = rows_allreduce_sum(l[i] * fast_exp2(m[i] - mm));
    if (lg == 0 && h0 + i < p.H && t.tile0 + lr < t.ql) p.lse[(int64_t)(h0 + i) * p.rows + t.s0 + t.tile0 + lr] = mm + fast_log2(ll);
  }
}

template <int HW>
__device__ __forceinline__ void store_heads(char* at, const uint32_t (&w)[(HW + 1) / 2]) {
  if constexpr (HW == 1) *reinterpret_cast<uint16_t*>(at) = (uint16_t)w[0];
  else if constexpr (HW == 2) *reinterpret_cast<uint32_t*>(at) = w[0];
  else if constexpr (HW == 4) *reinterpret_cast<uint2*>(at) = make_uint2(w[0], w[1]);
  else *reinterpret_cast<uint4*>(at) = make_uint4(w[0], w[1], w[2], w[3]);
}

// tiles of a portion that stay together
__host__ __device__ inline int mix_run(int reqs, int max_q) {
  const int n = (int)(((int64_t)reqs * ((max_q + 15) / 16)) >> 6);
  return n < 1 ? 1 : n > 16 ? 16 : n;
}

// LDS layout of the exchange (bytes).  A buffer has a region per row: the weights [hi, lo][16 keys][KP heads], which the one
// wave that mixes the row replaces by the mixed weights [16 HT heads][16 keys hi | lo].  Then talk [16 HT][KP] and the query
// operands that find no room in registers.
template <int HD, int HW>
struct MixLds {
  static constexpr int HT = HW == 8 ? 4 : HW == 4 ? 2 : 1, KP = HW == 8 ? 64 : 32;      // at most 8 HW heads
  static constexpr int kBufs = HW < 8 ? 2 : 1;         // two: values of a tile and weights of the next between the same barriers
  static constexpr int kKey = KP * 2 + 16, kHalf = 16 * kKey, kHead = 64 + 16;
  static constexpr int kRow = (2 * kHalf > 16 * HT * kHead ? 2 * kHalf : 16 * HT * kHead) + 16, kBuf = 16 * kRow;
  static constexpr int kTalkPitch = KP * 2 + 16, kTalk = kBufs * kBuf;
  static constexpr int QL = HD == 128 && HW == 4 ? 2 : 0;                                // heads of a wave with their q here
  static constexpr int kQ = kTalk + 16 * HT * kTalkPitch, kQWave = QL * (HD / 32) * 1024;
  static constexpr int bytes(int waves) { return kQ + waves * kQWave; }
};

template <int HD, int HW, bool ONE, bool CAP>
__global__ __launch_bounds__(512, 2) void prefill_mix_kernel(const PrefillParams p) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) char smem[];
  using M = MixLds<HD, HW>;
  constexpr int KS = HD / 32, VN = HD / 16, VH = VN / 2, HT = M::HT, QR = HW - M::QL;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lg = lane >> 4;
  const int NW = blockDim.x >> 6, R = p.H / p.G;
  // Workgroups go to the 8 XCDs in turn: `run` neighbouring tiles of a portion on one, where they walk the same keys; late
  // tiles (long rows) of all portions first.
  const int run = mix_run(p.reqs, p.max_q), tiles = (p.max_q + 15) / 16, b = blockIdx.x;
  const int unit = b / (8 * run) * 8 + (b & 7), r = unit % p.reqs;
  const int tile = tiles - 1 - (unit / p.reqs * run + (b >> 3) % run);
  if (tile < 0) return;
  const TileSpan t = tile_span(p, r, tile * 16);
  if (!t.any) return;
  for (int i = tid; i < M::kTalk / 16; i += blockDim.x) reinterpret_cast<uint4*>(smem)[i] = make_uint4(0, 0, 0, 0);
  for (int i = tid; i < 16 * HT * M::KP; i += blockDim.x) {
    const int h = i / M::KP, g = i % M::KP;
    reinterpret_cast<uint16_t*>(smem + M::kTalk + h * M::kTalkPitch)[g] = h < p.H && g < p.H ? E16::to_bits(p.talk[h * p.H + g]) : 0;
  }
  const int h0 = wave * HW, qi = min(t.tile0 + lr, t.ql - 1), qpos = t.start + t.tile0 + lr;
  const uint16_t* q = p.q + (int64_t)(t.s0 + qi) * p.q_stride + 8 * lg;
  uint4 qf[QR][KS];
  uint4* ql = reinterpret_cast<uint4*>(smem + M::kQ + wave * M::kQWave) + lane;
  float base[HW], r1[HW], r2[HW];      // base: what of the exponent depends on the row alone
  f32x4_t o[HW][VN] = {};
#pragma unroll
  for (int i = 0; i < HW; ++i) {
    const int h = min(h0 + i, p.H - 1);
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const uint4 v = *reinterpret_cast<const uint4*>(q + h * HD + 32 * k);
      if (i < QR) qf[i < QR ? i : 0][k] = v;
      else ql[((i - QR) * KS + k) * 64] = v;
    }
    const float lse = p.lse[(int64_t)h * p.rows + t.s0 + qi];
    base[i] = h0 + i < p.H ? p.mul.out - lse : -INFINITY;      // heads past the last: no weight
    r1[i] = uniform(p.r1 ? p.r1[h] : 0.f), r2[i] = uniform(p.r1 ? p.r2[h] : 0.f);
  }
  const int kv0 = min(h0, p.H - 1) / R;
  uint4 kf[KS], va[VH], vb[VH];
  load_k<HD>(kf, p, kv0, t.c0 + t.kb, lr, lg);

  // this wave's heads: weights of the keys at k0 (its K operands, and then those of the next tile, are in kf)
  auto weights = [&](int k0, char* buf) {
    f32x4_t s[HW];
#pragma unroll
    for (int i = 0; i < HW; ++i) {
      if (!ONE && i > 0) load_k<HD>(kf, p, min(h0 + i, p.H - 1) / R, t.c0 + k0, lr, lg);
      if (i < QR) {
        s[i] = qk<HD>(kf, qf[i < QR ? i : 0]);
      } else {
        uint4 x[KS];
#pragma unroll
        for (int k = 0; k < KS; ++k) x[k] = ql[((i - QR) * KS + k) * 64];
        s[i] = qk<HD>(kf, x);
      }
    }
    load_k<HD>(kf, p, kv0, t.c0 + min(k0 + 16, t.ke & ~15), lr, lg);
    const int key0 = t.first + k0, d0 = qpos - key0 - 4 * lg;
    const bool inside = key0 + 15 <= t.start + t.tile0 && t.start + t.tile0 + 15 - key0 < p.window;
    const float fd = (float)d0;
#pragma unroll
    for (int i = 0; i < HW; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j) s[i][j] = score_from<CAP>(base[i], s[i][j], fd - (float)j, r1[i], r2[i], p.mul);
    if (!inside) {
      asm volatile("");      // stays a branch: sixteen selects a tile for its edges only
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const bool seen = (unsigned)(d0 - j) < (unsigned)p.window;
#pragma unroll
        for (int i = 0; i < HW; ++i) s[i][j] = seen ? s[i][j] : -INFINITY;
      }
    }
    char* wr = buf + lr * M::kRow + 4 * lg * M::kKey + h0 * 2;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      float w[HW];
#pragma unroll
      for (int i = 0; i < HW; ++i) w[i] = fast_exp2(s[i][j]);
      uint32_t hi[(HW + 1) / 2], lo[(HW + 1) / 2];
      if constexpr (HW == 1) {
        hi[0] = E16::to_bits(w[0]);
        lo[0] = E16::to_bits(w[0] - E16::from_bits((uint16_t)hi[0]));
      } else {
#pragma unroll
        for (int i = 0; i < HW / 2; ++i) {
          hi[i] = E16::pack(w[2 * i], w[2 * i + 1]);
          lo[i] = E16::pack(w[2 * i] - E16::lo(hi[i]), w[2 * i + 1] - E16::hi(hi[i]));
        }
      }
      store_heads<HW>(wr + j * M::kKey, hi);
      store_heads<HW>(wr + j * M::kKey + M::kHalf, lo);
    }
  };
  // rows of the tile in turn: all heads' weights mixed, in place
  auto mix = [&](char* buf) {
    for (int row = wave; row < 16; row += NW) {
      char* at = buf + row * M::kRow;
      f32x4_t a[HT] = {};
#pragma unroll
      for (int k = 0; k < M::KP / 32; ++k) {
        const char* pr = at + lr * M::kKey + lg * 16 + 64 * k;
        const uint4 hi = *reinterpret_cast<const uint4*>(pr), lo = *reinterpret_cast<const uint4*>(pr + M::kHalf);
        uint4 tk[HT];
#pragma unroll
        for (int h = 0; h < HT; ++h)
          tk[h] = *reinterpret_cast<const uint4*>(smem + M::kTalk + (16 * h + lr) * M::kTalkPitch + 64 * k + lg * 16);
#pragma unroll
        for (int h = 0; h < HT; ++h) a[h] = mfma16<bf16_tag>(hi, tk[h], a[h]);
#pragma unroll
        for (int h = 0; h < HT; ++h) a[h] = mfma16<bf16_tag>(lo, tk[h], a[h]);
      }
#pragma unroll
      for (int h = 0; h < HT; ++h) {
        const f32x4_t& v = a[h];
        char* to = at + (16 * h + lr) * M::kHead + lg * 8;
        const uint2 hi = make_uint2(E16::pack(v[0], v[1]), E16::pack(v[2], v[3]));
        *reinterpret_cast<uint2*>(to) = hi;
        *reinterpret_cast<uint2*>(to + 32) = make_uint2(E16::pack(v[0] - E16::lo(hi.x), v[1] - E16::hi(hi.x)),
                                                        E16::pack(v[2] - E16::lo(hi.y), v[3] - E16::hi(hi.y)));
      }
    }
  };
  // value operands (columns past the values' size are zeros)
  auto load_v = [&](uint4 (&v)[VH], int kv, int k0, int n0) {
    const uint16_t* vt = p.vt + ((int64_t)kv * p.ctx_rows + t.c0 + k0) * HD + lr * 16 + (lg & 1) * 8 + n0 * 256;
#pragma unroll
    for (int n = 0; n < VH; ++n) v[n] = *reinterpret_cast<const uint4*>(vt + n * 256);
  };
  auto values = [&](int k0, const char* buf) {
    const char* rd = buf + lr * M::kRow + h0 * M::kHead + lg * 16;
    if constexpr (ONE) {       // the operands are in va and vb
#pragma unroll
      for (int i = 0; i < HW; ++i) {
        const uint4 w = *reinterpret_cast<const uint4*>(rd + i * M::kHead);
#pragma unroll
        for (int n = 0; n < VH; ++n) o[i][n] = mfma16<bf16_tag>(w, va[n], o[i][n]);
      }
#pragma unroll
      for (int i = 0; i < HW; ++i) {
        const uint4 w = *reinterpret_cast<const uint4*>(rd + i * M::kHead);
#pragma unroll
        for (int n = 0; n < VH; ++n) o[i][n + VH] = mfma16<bf16_tag>(w, vb[n], o[i][n + VH]);
      }
    } else {
#pragma unroll
      for (int i = 0; i < HW; ++i) {
        const uint4 w = *reinterpret_cast<const uint4*>(rd + i * M::kHead);
        const int kv = min(h0 + i, p.H - 1) / R;
        load_v(va, kv, k0, 0);
        load_v(vb, kv, k0, VH);
#pragma unroll
        for (int n = 0; n < VH; ++n) o[i][n] = mfma16<bf16_tag>(w, va[n], o[i][n]);
#pragma unroll
        for (int n = 0; n < VH; ++n) o[i][n + VH] = mfma16<bf16_tag>(w, vb[n], o[i][n + VH]);
      }
    }
  };
  __syncthreads();
  int at = 0;
  for (int k0 = t.kb; k0 <= t.ke; k0 += 16) {
    char* buf = smem + at;
    weights(k0, buf);
    if constexpr (ONE) load_v(va, kv0, k0, 0);
    __syncthreads();
    mix(buf);
    if constexpr (ONE) load_v(vb, kv0, k0, VH);
    __builtin_amdgcn_sched_barrier(0);      // the loads are on their way before the wait
    __syncthreads();
    values(k0, buf);
    if constexpr (M::kBufs == 2) at = M::kBuf - at;
    else __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < HW; ++i) {
    if (h0 + i >= p.H) continue;
#pragma unroll
    for (int n = 0; n < VN; ++n) {
      const int d = 16 * n + lr;
      if (d >= p.V) continue;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int row = t.tile0 + 4 * lg + j;
        if (row >= t.ql) continue;
        const int64_t at = (int64_t)(h0 + i) * p.V + d;
        float x = o[i][n][j];
        if (p.gate) x *= sigmoid_f(E16::from_bits(p.gate[(int64_t)(t.s0 + row) * p.gate_stride + at]));
        p.out[(int64_t)(t.s0 + row) * p.out_stride + at] = E16::to_bits(x);
      }
    }
  }
}

// ------------------------------------------------------------------------------------------------ host side
struct DecodePlan {
  int span, pitch, keys1, parts1, keys2, parts2, ksplit, rm;
  int64_t scores, ml, part;      // bytes
};

inline int ceil_div(int a, int b) { return (a + b - 1) / b; }

DecodePlan decode_plan(int reqs, int H, int G, int V, int window, int max_seq_len) {
  DecodePlan d;
  const int R = H / G;
  d.span = window < max_seq_len ? window : max_seq_len;
  if (d.span < 1) d.span = 1;
  d.pitch = ceil_div(d.span, 64) * 64;
  d.keys1 = (int64_t)reqs * G * ceil_div(d.span, 64) >= 1024 ? 64 : 16;
  d.parts1 = ceil_div(d.span, d.keys1);
  d.rm = R <= 1 ? 1 : R <= 2 ? 2 : R <= 4 ? 4 : 8;
  const int units = G * ceil_div(R, d.rm);
  d.ksplit = units == 1 ? 4 : units == 2 ? 2 : 1;
  d.keys2 = d.ksplit == 4 ? 128 : 64;      // a split is a multiple of 32 keys
  for (int k = 256; k > d.keys2; k >>= 1)
    if ((int64_t)reqs * ceil_div(d.span, k) >= 1024 && (k <= 128 || H <= 32)) { d.keys2 = k; break; }
  d.parts2 = ceil_div(d.span, d.keys2);
  auto up = [](int64_t n) { return (n + 255) / 256 * 256; };
  d.scores = up((int64_t)reqs * H * d.pitch * 4);
  d.ml = up((int64_t)reqs * d.parts1 * H * 8);
  d.part = up((int64_t)reqs * d.parts2 * d.ksplit * H * V * 4);
  return d;
}

inline int heads_per_wave(int H) {
  for (int w = 1; w <= 8; w <<= 1)
    if (ceil_div(H, w) <= 8) return w;
  return 16;
}

inline ScoreMul score_mul(float scale, float cap) {
  return cap > 0.f ? ScoreMul{2.f * scale * kLog2e / cap, cap * kLog2e} : ScoreMul{scale * kLog2e, 0.f};
}

inline int log2_of(int v) { return 31 - __builtin_clz(v); }

bool args_ok(const mi_talking_attn_args& a) {
  return a.out && a.q && a.k_cache && a.v_cache && a.block_table && a.seq_lens && a.query_start_loc && a.talk && !a.r1 == !a.r2 &&
         a.heads > 0 && a.kv_heads > 0 && a.heads % a.kv_heads == 0 && a.vdim > 0 && a.vdim <= a.head_dim && a.window > 0 &&
         a.q_stride >= (int64_t)a.heads * a.head_dim && a.out_stride >= (int64_t)a.heads * a.vdim &&
         (!a.gate || a.gate_stride >= (int64_t)a.heads * a.vdim);
}

bool sizes_built(const mi_talking_attn_args& a) {
  return mi_talking_attn_supported(a.heads, a.kv_heads, a.head_dim, a.vdim, a.block_size, a.softcap) && a.q_stride % 8 == 0 &&
         a.cache_block_stride % 8 == 0 && a.cache_token_stride % 8 == 0 && a.cache_head_stride % 8 == 0 && aligned16(a.q) &&
         aligned16(a.k_cache) && aligned16(a.v_cache);
}

template <typename K>
int allow_lds(K kern, int bytes) {
  if (bytes > 65536 &&
      hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, bytes) != hipSuccess)
    return MI_ERR_LAUNCH;
  return MI_OK;
}

template <int HD, int RM, int HT>
int launch_values(const DecodeParams& p, int reqs, hipStream_t s) {
  const int kq = (p.H + 3) / 4;
  const int bytes = (p.keys2 * decode_pad(p.H) + 16 + 16 * HT * (4 * kq + 1) + 4 * kq + 2 * ((p.keys2 >> p.bs_log2) + 2)) * 4;
  auto kern = decode_values_kernel<HD, RM, HT>;
  if (int e = allow_lds(kern, bytes)) return e;
  hipLaunchKernelGGL(kern, dim3(p.parts2, reqs), dim3(256), bytes, s, p);
  return launch_status();
}

template <int HD>
int launch_decode(const DecodeParams& p, int reqs, int rm, bool cap, hipStream_t s) {
  const dim3 g1(ceil_div(p.parts1 * p.G, 4), reqs), block(256);
#define MI_DS(NT, CW)                                                                                 \
  do {                                                                                                \
    if (cap) hipLaunchKernelGGL((decode_scores_kernel<HD, NT, CW, true>), g1, block, 0, s, p);        \
    else hipLaunchKernelGGL((decode_scores_kernel<HD, NT, CW, false>), g1, block, 0, s, p);           \
  } while (0)
  const int R = p.H / p.G;
  if (p.keys1 == 16) MI_DS(1, 16);
  else if (R <= 4) MI_DS(4, 4);
  else if (R <= 8) MI_DS(4, 8);
  else MI_DS(4, 16);
#undef MI_DS
  int e = launch_status();
  if (e) return e;
  if (p.H <= 32)
    e = rm == 1 ? launch_values<HD, 1, 2>(p, reqs, s) : rm == 2 ? launch_values<HD, 2, 2>(p, reqs, s)
        : rm == 4 ? launch_values<HD, 4, 2>(p, reqs, s) : launch_values<HD, 8, 2>(p, reqs, s);
  else
    e = rm == 1 ? launch_values<HD, 1, 4>(p, reqs, s) : rm == 2 ? launch_values<HD, 2, 4>(p, reqs, s)
        : rm == 4 ? launch_values<HD, 4, 4>(p, reqs, s) : launch_values<HD, 8, 4>(p, reqs, s);
  if (e) return e;
  hipLaunchKernelGGL(decode_reduce_kernel, dim3(ceil_div(p.H * p.V, 256), reqs), dim3(256), 0, s, p);
  return launch_status();
}

template <int HD, int HW, bool ONE, bool CAP>
int launch_prefill(const PrefillParams& p, int reqs, int max_q, hipStream_t s) {
  hipLaunchKernelGGL((prefill_sums_kernel<HD, HW, ONE, CAP>), dim3(ceil_div(p.H, HW) * ceil_div(max_q, 64) * reqs), dim3(256), 0, s, p);
  if (int e = launch_status()) return e;
  const int waves = ceil_div(p.H, HW), bytes = MixLds<HD, HW>::bytes(waves);
  auto kern = prefill_mix_kernel<HD, HW, ONE, CAP>;
  if (int e = allow_lds(kern, bytes)) return e;
  const int run = mix_run(reqs, max_q), units = ceil_div(ceil_div(max_q, 16), run) * reqs;
  hipLaunchKernelGGL(kern, dim3(ceil_div(units, 8) * 8 * run), dim3(64 * waves), bytes, s, p);
  return launch_status();
}

template <int HD, int HW>
int launch_prefill_of(const PrefillParams& p, int reqs, int max_q, bool cap, hipStream_t s) {
  if (HW == 1 || p.H / p.G % HW == 0)
    return cap ? launch_prefill<HD, HW, true, true>(p, reqs, max_q, s) : launch_prefill<HD, HW, true, false>(p, reqs, max_q, s);
  return cap ? launch_prefill<HD, HW, false, true>(p, reqs, max_q, s) : launch_prefill<HD, HW, false, false>(p, reqs, max_q, s);
}

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int mi_talking_attn_supported(int32_t heads, int32_t kv_heads, int32_t head_dim, int32_t vdim, int32_t block_size,
                                         float softcap) {
  return heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && (head_dim == 64 || head_dim == 128) && vdim > 0 && vdim <= head_dim &&
         heads <= (head_dim == 64 ? 64 : 32) && block_size >= 16 && is_pow2(block_size) && softcap <= 1024.f;
}

extern "C" int64_t mi_talking_decode_workspace_bytes(int32_t num_reqs, int32_t heads, int32_t kv_heads, int32_t vdim, int32_t window,
                                                     int32_t max_seq_len) {
  if (num_reqs <= 0 || heads <= 0 || kv_heads <= 0 || heads % kv_heads || vdim <= 0 || window <= 0) return 0;
  const DecodePlan d = decode_plan(num_reqs, heads, kv_heads, vdim, window, max_seq_len);
  return d.scores + d.ml + d.part;
}

extern "C" int mi_talking_decode(const mi_talking_attn_args* args, int32_t num_reqs, int32_t max_seq_len, void* workspace,
                                 int64_t workspace_bytes, void* stream) {
  if (num_reqs == 0) return MI_OK;
  if (!args || num_reqs < 0 || max_seq_len < 0 || !args_ok(*args)) return MI_ERR_INVALID_ARG;
  const mi_talking_attn_args& a = *args;
  if (!sizes_built(a) || num_reqs > 65535) return MI_ERR_UNSUPPORTED;
  const DecodePlan d = decode_plan(num_reqs, a.heads, a.kv_heads, a.vdim, a.window, max_seq_len);
  if (!workspace || workspace_bytes < d.scores + d.ml + d.part || !aligned16(workspace)) return MI_ERR_WORKSPACE;
  char* ws = (char*)workspace;
  const DecodeParams p{(const uint16_t*)a.q, (const uint16_t*)a.k_cache, (const uint16_t*)a.v_cache, a.block_table, a.seq_lens, a.r1,
                       a.r2, a.talk, (const uint16_t*)a.gate, (uint16_t*)a.out, (float*)ws, (float2*)(ws + d.scores),
                       (float*)(ws + d.scores + d.ml), a.q_stride, a.out_stride, a.gate_stride, a.cache_block_stride,
                       a.cache_token_stride, a.cache_head_stride, a.table_stride, a.heads, a.kv_heads, a.vdim, log2_of(a.block_size),
                       d.span, d.pitch, d.parts1, d.keys1, d.parts2, d.keys2, d.ksplit, score_mul(a.scale, a.softcap)};
  hipStream_t s = (hipStream_t)stream;
  return a.head_dim == 64 ? launch_decode<64>(p, num_reqs, d.rm, a.softcap > 0.f, s) : launch_decode<128>(p, num_reqs, d.rm, a.softcap > 0.f, s);
}

extern "C" int64_t mi_talking_prefill_workspace_bytes(int32_t rows, int32_t heads, int32_t kv_heads, int32_t head_dim, int32_t ctx_rows) {
  if (rows <= 0 || heads <= 0 || kv_heads <= 0 || head_dim <= 0 || ctx_rows <= 0) return 0;
  return 2ll * kv_heads * ctx_rows * head_dim * 2 + (int64_t)heads * rows * 4;
}

extern "C" int mi_talking_prefill(const mi_talking_attn_args* args, const int32_t* ctx_start, int32_t ctx_rows, int32_t num_reqs,
                                  int32_t rows, int32_t max_query_len, void* workspace, int64_t workspace_bytes, void* stream) {
  if (num_reqs == 0 || rows == 0 || max_query_len == 0) return MI_OK;
  if (!args || !ctx_start || num_reqs < 0 || rows < 0 || max_query_len < 0 || ctx_rows <= 0 || ctx_rows % 64 || !args_ok(*args))
    return MI_ERR_INVALID_ARG;
  const mi_talking_attn_args& a = *args;
  if (!sizes_built(a) || num_reqs > 65535) return MI_ERR_UNSUPPORTED;
  const int64_t kb = (int64_t)a.kv_heads * ctx_rows * a.head_dim * 2;
  if (!workspace || !aligned16(workspace) ||
      workspace_bytes < mi_talking_prefill_workspace_bytes(rows, a.heads, a.kv_heads, a.head_dim, ctx_rows))
    return MI_ERR_WORKSPACE;
  char* ws = (char*)workspace;
  hipStream_t s = (hipStream_t)stream;
  const GatherParams gp{(uint16_t*)ws, (uint16_t*)(ws + kb), (const uint16_t*)a.k_cache, (const uint16_t*)a.v_cache, ctx_start,
                        a.block_table, a.seq_lens, a.query_start_loc, a.cache_block_stride, a.cache_token_stride, a.cache_head_stride,
                        a.table_stride, num_reqs, ctx_rows, log2_of(a.block_size), a.window};
  const dim3 gg(ctx_rows / 64, a.kv_heads), block(256);
  if (a.head_dim == 64) hipLaunchKernelGGL(gather_kernel<64>, gg, block, 0, s, gp);
  else hipLaunchKernelGGL(gather_kernel<128>, gg, block, 0, s, gp);
  if (int e = launch_status()) return e;
  const PrefillParams p{(const uint16_t*)a.q, (const uint16_t*)ws, (const uint16_t*)(ws + kb), (float*)(ws + 2 * kb), ctx_start, a.seq_lens,
                        a.query_start_loc, a.r1, a.r2, a.talk, (const uint16_t*)a.gate, (uint16_t*)a.out, a.q_stride, a.out_stride,
                        a.gate_stride, a.heads, a.kv_heads, a.vdim, a.window, rows, ctx_rows, num_reqs, max_query_len, score_mul(a.scale, a.softcap)};
  const bool cap = a.softcap > 0.f;
  const int hw = heads_per_wave(a.heads);
  if (a.head_dim == 64) {
    if (hw == 1) return launch_prefill_of<64, 1>(p, num_reqs, max_query_len, cap, s);
    if (hw == 2) return launch_prefill_of<64, 2>(p, num_reqs, max_query_len, cap, s);
    if (hw == 4) return launch_prefill_of<64, 4>(p, num_reqs, max_query_len, cap, s);
    return launch_prefill_of<64, 8>(p, num_reqs, max_query_len, cap, s);
  }
  if (hw == 1) return launch_prefill_of<128, 1>(p, num_reqs, max_query_len, cap, s);
  if (hw == 2) return launch_prefill_of<128, 2>(p, num_reqs, max_query_len, cap, s);
  return launch_prefill_of<128, 4>(p, num_reqs, max_query_len, cap, s);
}
