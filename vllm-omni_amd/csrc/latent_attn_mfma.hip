// Matrix-core kernels of the latent attention (bf16): see latent_attn.hip for the mechanism.
//   * latent_decode:  absorbed form, one query token per request.  A cache tile of 64 rows x rank is staged once and serves
//     as keys (row reads) and values (transposed reads) of up to 32 heads; the context is split over workgroups.  Bound:
//     HBM, the window's cache rows read once per 32 heads.
//   * latent_prefill: prompt portions.  The portion's visible latents are gathered into a dense matrix per request (64-row
//     aligned), K = ctx W_uk^T and V^T = W_uv ctx^T come from library GEMMs, and this kernel runs windowed attention on
//     them, S^T = K Q^T and O^T = V^T P^T, so that a query is a lane and P is an operand without leaving registers.
//   * head_gemm_nt:   per-head products (absorb, and W_uv behind the decode attention).
// Attention weights are 32-bit quantities: P enters its product as a bf16 pair hi + lo.
#include "mfma_attn_common.h"
#include "row_io.h"

namespace mi {
namespace {

using E16 = Elem<bf16_tag>;

// ------------------------------------------------------------------------------------------------ per-head GEMM
// y[t][h][n] = sum_k x[t][h][k] w[h][n][k]; wave = 16 n x 16 TT t, operands straight from global memory, 128 k of them in
// flight.  Loads are unconditional on clamped addresses; FULL: Kd is a multiple of 32, nothing to blank out.
template <int TT, bool FULL>
__global__ __launch_bounds__(256) void head_gemm_nt_kernel(uint16_t* y, const uint16_t* x, const uint16_t* w, int rows, int N, int Kd,
                                                           int64_t y_row, int64_t x_row, int64_t w_head) {
  scalar_cache_acquire();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lr = lane & 15, lg = lane >> 4;
  const int h = blockIdx.y, n0 = blockIdx.x * 64 + wave * 16, t0 = blockIdx.z * 16 * TT;
  if (n0 >= N) return;
  const uint16_t* wr = w + h * w_head + (int64_t)min(n0 + lr, N - 1) * Kd;
  const uint16_t* xh = x + (int64_t)h * Kd;
  f32x4_t acc[TT] = {};
  for (int k0 = 0; k0 < Kd; k0 += 128) {
    u32x4_t a[4], b[4][TT];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int k = min(k0 + 32 * u + 8 * lg, Kd - 8);      // Kd is a multiple of 8
      a[u] = *reinterpret_cast<const u32x4_t*>(wr + k);
#pragma unroll
      for (int i = 0; i < TT; ++i) b[u][i] = *reinterpret_cast<const u32x4_t*>(xh + (int64_t)min(t0 + 16 * i + lr, rows - 1) * x_row + k);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      if (FULL && k0 + 32 * u >= Kd) break;
      if (!FULL && k0 + 32 * u + 8 * lg >= Kd) a[u] = u32x4_t{0, 0, 0, 0};
#pragma unroll
      for (int i = 0; i < TT; ++i) acc[i] = mfma16<bf16_tag>(__builtin_bit_cast(uint4, a[u]), __builtin_bit_cast(uint4, b[u][i]), acc[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < TT; ++i) {
    const int t = t0 + 16 * i + lr, n = n0 + 4 * lg;
    if (t < rows && n < N)      // N is a multiple of 4
      *reinterpret_cast<uint2*>(y + t * y_row + (int64_t)h * N + n) = make_uint2(E16::pack(acc[i][0], acc[i][1]), E16::pack(acc[i][2], acc[i][3]));
  }
}

// ------------------------------------------------------------------------------------------------ decode
struct LatentDecodeParams {
  uint16_t* out;         // [reqs][H][rank]
  const uint16_t* q;     // [reqs][H][rank]
  const uint16_t* cache;
  const int32_t* table;
  const int32_t* seq_lens;
  float* part;           // [reqs][nsplit][H][rank + 2] when nsplit > 1: sums, then m, l
  int64_t block_stride, token_stride, table_stride;
  int H, rank, bs_log2, window, nsplit;
  float scale;           // times log2(e)
};

__device__ __forceinline__ uint32_t lds_addr(const void* p) { return (uint32_t)(uintptr_t)(lds_void*)p; }

// transposed reads of the A operands (K = 32: two reads of 4 key rows x 16 dims) of one or four consecutive dim tiles, with
// one wait
template <int OFF>
__device__ __forceinline__ uint4 tr_pair(uint32_t addr) {
  u32x2_t a, b;
  asm volatile("ds_read_b64_tr_b16 %0, %2\n\tds_read_b64_tr_b16 %1, %2 offset:%3\n\ts_waitcnt lgkmcnt(0)"
               : "=&v"(a), "=&v"(b) : "v"(addr), "i"(OFF) : "memory");
  return make_uint4(a[0], a[1], b[0], b[1]);
}
template <int OFF>
__device__ __forceinline__ void tr_pair4(uint32_t addr, uint4 (&o)[4]) {
  u32x2_t a[4], b[4];
  asm volatile(
      "ds_read_b64_tr_b16 %0, %8\n\tds_read_b64_tr_b16 %4, %8 offset:%9\n\t"
      "ds_read_b64_tr_b16 %1, %8 offset:32\n\tds_read_b64_tr_b16 %5, %8 offset:%10\n\t"
      "ds_read_b64_tr_b16 %2, %8 offset:64\n\tds_read_b64_tr_b16 %6, %8 offset:%11\n\t"
      "ds_read_b64_tr_b16 %3, %8 offset:96\n\tds_read_b64_tr_b16 %7, %8 offset:%12\n\t"
      "s_waitcnt lgkmcnt(0)"
      : "=&v"(a[0]), "=&v"(a[1]), "=&v"(a[2]), "=&v"(a[3]), "=&v"(b[0]), "=&v"(b[1]), "=&v"(b[2]), "=&v"(b[3])
      : "v"(addr), "i"(OFF), "i"(OFF + 32), "i"(OFF + 64), "i"(OFF + 96)
      : "memory");
#pragma unroll
  for (int i = 0; i < 4; ++i) o[i] = make_uint4(a[i][0], a[i][1], b[i][0], b[i][1]);
}

template <int RN, int NHT>
__global__ __launch_bounds__(256 * NHT) void latent_decode_kernel(const LatentDecodeParams p) {
  scalar_cache_acquire();
  constexpr int Rp = 64 * RN, NT = 256 * NHT, LD = Rp + 8, PL = 64 + 8;
  constexpr int CH = 64 * (Rp / 8) / NT;            // 16-byte chunks of a tile per thread
  constexpr int MT = RN;                            // 16-dim tiles a wave accumulates (Rp / 4 dims)
  extern __shared__ __attribute__((aligned(16))) char smem[];
  uint16_t* sC = reinterpret_cast<uint16_t*>(smem);           // [64][LD]
  uint16_t* sP = sC + 64 * LD;                                // [2 (hi, lo)][16 NHT][PL]
  float* sR = reinterpret_cast<float*>(sP + 2 * 16 * NHT * PL);   // [4][16 NHT]
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lr = lane & 15, lg = lane >> 4;
  const int kw = wave & 3, ht = wave >> 2;          // key group / dim group, head tile
  const int split = blockIdx.x, r = blockIdx.z;
  const int hl = ht * 16 + lr, head = blockIdx.y * 16 * NHT + hl;
  const bool live = head < p.H;
  const int L = p.seq_lens[r];
  const int lo = max(0, L - p.window), n = max(0, L - lo);
  const int per = ((n + p.nsplit - 1) / p.nsplit + 63) / 64 * 64;
  const int k0 = lo + split * per, k1 = min(L, k0 + per);
  f32x4_t acc[MT] = {};
  float m = -INFINITY, l = 0.f;
  if (k0 < k1) {
    u32x4_t qv[2 * RN];
    const uint16_t* qr = p.q + ((int64_t)r * p.H + (live ? head : 0)) * p.rank;
#pragma unroll
    for (int k = 0; k < 2 * RN; ++k) qv[k] = *reinterpret_cast<const u32x4_t*>(qr + min(32 * k + 8 * lg, p.rank - 8));
    // a tile's block ids are loaded a tile ahead of its rows, its rows a tile ahead of their use.  Loads are unconditional on
    // clamped addresses (rows past the split get weight 0, columns past the rank meet zeros of q and are not stored): the
    // number in flight is known at every wait.
    const int32_t* tab = p.table + (int64_t)r * p.table_stride;
    const int bmask = (1 << p.bs_log2) - 1;
    u32x4_t pre[CH];
    int32_t blk[CH];
    auto ids = [&](int t0) {
#pragma unroll
      for (int i = 0; i < CH; ++i) blk[i] = tab[min(t0 + (tid + i * NT) / (Rp / 8), k1 - 1) >> p.bs_log2];
    };
    auto fetch = [&](int t0) {
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        const int c = tid + i * NT, key = min(t0 + c / (Rp / 8), k1 - 1), col = min((c % (Rp / 8)) * 8, p.rank - 8);
        pre[i] = *reinterpret_cast<const u32x4_t*>(p.cache + (int64_t)blk[i] * p.block_stride + (int64_t)(key & bmask) * p.token_stride + col);
      }
    };
    ids(k0);
    fetch(k0);
    ids(k0 + 64);
    uint4 qf[2 * RN];
#pragma unroll
    for (int k = 0; k < 2 * RN; ++k) {
      const bool in = 32 * k + 8 * lg < p.rank;
      qf[k] = make_uint4(in ? qv[k][0] : 0, in ? qv[k][1] : 0, in ? qv[k][2] : 0, in ? qv[k][3] : 0);
    }
    const uint32_t tr_base = lds_addr(sC) + (uint32_t)(((8 * lg + (lr >> 2)) * LD + kw * (Rp / 4) + 4 * (lr & 3)) * 2);
    for (int t0 = k0; t0 < k1; t0 += 64) {
      __syncthreads();        // the previous tile's readers are done
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        const int c = tid + i * NT, row = c / (Rp / 8), col = (c % (Rp / 8)) * 8;
        *reinterpret_cast<u32x4_t*>(sC + row * LD + col) = pre[i];
      }
      __syncthreads();
      fetch(t0 + 64);      // (past the end: the last row again)
      ids(t0 + 128);
      f32x4_t s = {}, s2 = {};
#pragma unroll
      for (int k = 0; k < 2 * RN; k += 2) {
        const uint4 a = *reinterpret_cast<const uint4*>(sC + (16 * kw + lr) * LD + 32 * k + 8 * lg);
        const uint4 b = *reinterpret_cast<const uint4*>(sC + (16 * kw + lr) * LD + 32 * k + 32 + 8 * lg);
        s = mfma16<bf16_tag>(a, qf[k], s);
        s2 = mfma16<bf16_tag>(b, qf[k + 1], s2);
      }
      s += s2;
      float mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        s[i] = t0 + 16 * kw + 4 * lg + i < k1 ? s[i] * p.scale : -INFINITY;
        mx = fmaxf(mx, s[i]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      if (lg == 0) sR[kw * 16 * NHT + hl] = mx;
      __syncthreads();
      float mn = m;
#pragma unroll
      for (int i = 0; i < 4; ++i) mn = fmaxf(mn, sR[i * 16 * NHT + hl]);
      const float f = fast_exp2(m - mn);
      m = mn;
      float e[4], lo4[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        e[i] = fast_exp2(s[i] - mn);
        lo4[i] = e[i] - E16::from_bits(E16::to_bits(e[i]));
      }
      l = l * f + ((e[0] + e[1]) + (e[2] + e[3]));
      uint16_t* ph = sP + hl * PL + 16 * kw + 4 * lg;
      *reinterpret_cast<uint2*>(ph) = make_uint2(E16::pack(e[0], e[1]), E16::pack(e[2], e[3]));
      *reinterpret_cast<uint2*>(ph + 16 * NHT * PL) = make_uint2(E16::pack(lo4[0], lo4[1]), E16::pack(lo4[2], lo4[3]));
#pragma unroll
      for (int i = 0; i < MT; ++i) acc[i] *= f;
      __syncthreads();
#pragma unroll
      for (int kb = 0; kb < 2; ++kb) {
        const uint4 bh = *reinterpret_cast<const uint4*>(sP + hl * PL + 32 * kb + 8 * lg);
        const uint4 bl = *reinterpret_cast<const uint4*>(sP + (16 * NHT + hl) * PL + 32 * kb + 8 * lg);
        const uint32_t base = tr_base + (uint32_t)(32 * kb * LD * 2);
        if constexpr (MT >= 4) {
#pragma unroll
          for (int i = 0; i < MT; i += 4) {
            uint4 a[4];
            tr_pair4<4 * LD * 2>(base + 32 * i, a);
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[i + j] = mfma16<bf16_tag>(a[j], bh, acc[i + j]);
#pragma unroll
            for (int j = 0; j < 4; ++j) acc[i + j] = mfma16<bf16_tag>(a[j], bl, acc[i + j]);
          }
        } else {
#pragma unroll
          for (int i = 0; i < MT; ++i) {
            const uint4 a = tr_pair<4 * LD * 2>(base + 32 * i);
            acc[i] = mfma16<bf16_tag>(a, bh, acc[i]);
            acc[i] = mfma16<bf16_tag>(a, bl, acc[i]);
          }
        }
      }
    }
    // l: over the lane groups, then the four key groups of the head tile
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    __syncthreads();
    if (lg == 0) sR[kw * 16 * NHT + hl] = l;
    __syncthreads();
    l = (sR[hl] + sR[16 * NHT + hl]) + (sR[2 * 16 * NHT + hl] + sR[3 * 16 * NHT + hl]);
  }
  if (!live) return;
  if (p.nsplit == 1) {
    const float inv = l > 0.f ? 1.0f / l : 0.f;     // no tokens (a padded row): zeros
    uint16_t* o = p.out + ((int64_t)r * p.H + head) * p.rank;
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const int d = kw * (Rp / 4) + 16 * i + 4 * lg;
      if (d < p.rank)
        *reinterpret_cast<uint2*>(o + d) = make_uint2(E16::pack(acc[i][0] * inv, acc[i][1] * inv), E16::pack(acc[i][2] * inv, acc[i][3] * inv));
    }
  } else {
    float* o = p.part + (((int64_t)r * p.nsplit + split) * p.H + head) * (p.rank + 4);
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const int d = kw * (Rp / 4) + 16 * i + 4 * lg;
      if (d < p.rank) *reinterpret_cast<f32x4_t*>(o + d) = acc[i];
    }
    if (kw == 0 && lg == 0) o[p.rank] = m, o[p.rank + 1] = l;
  }
}

__global__ __launch_bounds__(128) void latent_decode_merge_kernel(uint16_t* out, const float* part, int H, int rank, int nsplit) {
  scalar_cache_acquire();
  const int h = blockIdx.x, r = blockIdx.y, lane = threadIdx.x & 63;
  const int64_t st = (int64_t)H * (rank + 4);
  const float* b = part + ((int64_t)r * nsplit * H + h) * (rank + 4);
  const int d = threadIdx.x * 4;
  const float* bd = b + min(d, rank - 4);
  // lane s holds split s's maximum and sum (at most 64 splits); eight splits' values are in flight at a time
  f32x4_t v[8];
  auto fetch = [&](int s0) {
#pragma unroll
    for (int j = 0; j < 8; ++j) v[j] = *reinterpret_cast<const f32x4_t*>(bd + min(s0 + j, nsplit - 1) * st);
  };
  const float* bs = b + min(lane, nsplit - 1) * st + rank;
  const float ms = bs[0], ls = lane < nsplit ? bs[1] : 0.f;
  fetch(0);
  const float m = wave_allreduce_max(ls > 0.f ? ms : -INFINITY);
  const float w = ls > 0.f ? fast_exp2(ms - m) : 0.f;      // a split without tokens: 0
  const float l = wave_allreduce_sum(ls * w);
  f32x4_t a = {};
  for (int s0 = 0; s0 < nsplit; s0 += 8) {
#pragma unroll
    for (int j = 0; j < 8; ++j) a += v[j] * __shfl(w, s0 + j, 64);
    fetch(s0 + 8);
  }
  a *= l > 0.f ? 1.0f / l : 0.f;
  if (d < rank)
    *reinterpret_cast<uint2*>(out + ((int64_t)r * H + h) * rank + d) = make_uint2(E16::pack(a[0], a[1]), E16::pack(a[2], a[3]));
}

// ------------------------------------------------------------------------------------------------ prefill
// row i of the dense context: request r with ctx_start[r] <= i, position first(r) + i - ctx_start[r]; zeros past its end
__global__ __launch_bounds__(256) void latent_gather_kernel(uint16_t* ctx, const uint16_t* cache, const int32_t* ctx_start,
                                                            const int32_t* table, const int32_t* seq_lens, const int32_t* qsl,
                                                            int reqs, int rows, int rank, int block_size, int window,
                                                            int64_t block_stride, int64_t token_stride, int64_t table_stride) {
  scalar_cache_acquire();
  const int per = rank / 8;
  const int64_t item = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (item >= (int64_t)rows * per) return;
  const int i = (int)(item / per), c = (int)(item % per) * 8;
  const int r = row_request(ctx_start, reqs, i);
  const int L = seq_lens[r], first = max(0, L - (qsl[r + 1] - qsl[r]) - window + 1);
  const int pos = first + i - ctx_start[r];
  uint4 v = make_uint4(0, 0, 0, 0);
  if (pos < L)
    v = *reinterpret_cast<const uint4*>(cache + (int64_t)table[r * table_stride + pos / block_size] * block_stride +
                                        (int64_t)(pos % block_size) * token_stride + c);
  *reinterpret_cast<uint4*>(ctx + (int64_t)i * rank + c) = v;
}

struct LatentPrefillParams {
  uint16_t* out;         // [rows][H vdim]
  const uint16_t* q;     // [rows][H dim]
  const uint16_t* k;     // [ctx][H dim]
  const uint16_t* vt;    // [H vdim][ctx]
  const int32_t* ctx_start;
  const int32_t* seq_lens;
  const int32_t* qsl;
  int64_t q_stride, k_stride, out_stride, vt_stride;
  int H, dim, vdim, window;
  float scale;           // times log2(e)
};

template <int KT, int VN>   // dim padded to 16 KT, vdim to 32 VN
__global__ __launch_bounds__(256, KT <= 8 && VN <= 4 ? 2 : 1) void latent_prefill_kernel(const LatentPrefillParams p) {
  scalar_cache_acquire();
  constexpr int Dp = 16 * KT, Vp = 32 * VN, LK = Dp + 8, LV = 64 + 4;
  constexpr int KCH = 64 * (Dp / 8) / 256, VCH = Vp * 8 / 256;
  constexpr int STAGE = 64 * LK + Vp * LV;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  uint16_t* lds = reinterpret_cast<uint16_t*>(smem);
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lc = lane & 31, hh = lane >> 5;
  // heads spread over the XCDs (workgroups go to the 8 in turn), a head's query tiles follow each other on one
  const int hx = (p.H + 7) / 8;
  const int idx = blockIdx.x >> 3;
  const int head = (blockIdx.x & 7) + 8 * (idx % hx), r = blockIdx.y;
  const int s0 = p.qsl[r], ql = p.qsl[r + 1] - s0;
  const int tile0 = (idx / hx) * 128;
  if (head >= p.H || tile0 >= ql) return;
  const int L = p.seq_lens[r], start = L - ql;
  const int first = max(0, start - p.window + 1);       // position of the request's context row 0
  const int c0 = p.ctx_start[r];
  const int rows = min(128, ql - tile0);
  const int q_lo = start + tile0, q_hi = q_lo + rows - 1;
  const int qi = wave * 32 + lc, qpos = q_lo + qi;
  const bool valid = qi < rows;
  // 64-row tiles of the context, in context-row coordinates
  const int kb = (max(0, q_lo - p.window + 1 - first)) / 64 * 64, ke = q_hi - first + 1;
  // this wave's own key range: tiles outside it are staged with the others but not computed
  const int wq_lo = q_lo + wave * 32, wq_hi = min(q_lo + wave * 32 + 31, q_hi);
  uint4 qf[KT];
#pragma unroll
  for (int k = 0; k < KT; ++k) {
    const int c = 16 * k + 8 * hh;
    qf[k] = valid && c < p.dim ? *reinterpret_cast<const uint4*>(p.q + (int64_t)(s0 + tile0 + qi) * p.q_stride + (int64_t)head * p.dim + c)
                               : make_uint4(0, 0, 0, 0);
  }
  uint4 pk[KCH], pv[VCH];
  auto fetch = [&](int t) {
#pragma unroll
    for (int i = 0; i < KCH; ++i) {
      const int c = tid + i * 256, row = c / (Dp / 8), col = (c % (Dp / 8)) * 8;
      pk[i] = col < p.dim ? *reinterpret_cast<const uint4*>(p.k + (int64_t)(c0 + t + row) * p.k_stride + (int64_t)head * p.dim + col)
                          : make_uint4(0, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < VCH; ++i) {
      const int c = tid + i * 256, row = c >> 3, col = (c & 7) * 8;
      pv[i] = row < p.vdim ? *reinterpret_cast<const uint4*>(p.vt + ((int64_t)head * p.vdim + row) * p.vt_stride + c0 + t + col)
                           : make_uint4(0, 0, 0, 0);
    }
  };
  auto stage = [&](uint16_t* b) {
#pragma unroll
    for (int i = 0; i < KCH; ++i) {
      const int c = tid + i * 256, row = c / (Dp / 8), col = (c % (Dp / 8)) * 8;
      *reinterpret_cast<uint4*>(b + row * LK + col) = pk[i];
    }
    uint16_t* v = b + 64 * LK;
#pragma unroll
    for (int i = 0; i < VCH; ++i) {
      const int c = tid + i * 256, row = c >> 3, col = (c & 7) * 8;
      *reinterpret_cast<uint2*>(v + row * LV + col) = make_uint2(pv[i].x, pv[i].y);
      *reinterpret_cast<uint2*>(v + row * LV + col + 4) = make_uint2(pv[i].z, pv[i].w);
    }
  };
  f32x16_t acc[VN] = {};
  float m = -INFINITY, l = 0.f;
  fetch(kb);
  int cur = 0;
  for (int t = kb; t < ke; t += 64, cur ^= 1) {
    uint16_t* b = lds + cur * STAGE;
    stage(b);
    __syncthreads();      // (two stages: the buffer written next was last read before this barrier)
    if (t + 64 < ke) fetch(t + 64);
    const int p0 = first + t;                                   // position of the tile's first key
    if (p0 > wq_hi || p0 + 63 <= wq_lo - p.window) continue;    // wave-uniform: nothing of this tile is visible here
    const uint16_t* v = b + 64 * LK;
    f32x16_t s[2] = {};
#pragma unroll
    for (int mt = 0; mt < 2; ++mt)
#pragma unroll
      for (int k = 0; k < KT; ++k) {
        const uint4 a = *reinterpret_cast<const uint4*>(b + (32 * mt + lc) * LK + 16 * k + 8 * hh);
        s[mt] = mfma32<bf16_tag>(a, qf[k], s[mt]);
      }
    const bool inner = p0 + 63 <= wq_lo && p0 > wq_hi - p.window;   // every key visible to every query of the wave
    float mx = -INFINITY;
#pragma unroll
    for (int mt = 0; mt < 2; ++mt)
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        float x = s[mt][i] * p.scale;
        if (!inner) {
          const int d = qpos - (p0 + 32 * mt + 8 * (i >> 2) + 4 * hh + (i & 3));
          x = d >= 0 && d < p.window ? x : -INFINITY;
        }
        s[mt][i] = x;
        mx = fmaxf(mx, x);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m, mx);
    const float base = mn == -INFINITY ? 0.f : mn;              // a query that has seen nothing yet: all weights 0
    if (__any(mn > m)) {
      const float f = fast_exp2(m - base);
      l *= f;
#pragma unroll
      for (int n = 0; n < VN; ++n) acc[n] *= f;
      m = mn;
    }
    float ls = 0.f;
#pragma unroll
    for (int mt = 0; mt < 2; ++mt)
#pragma unroll
      for (int bk = 0; bk < 2; ++bk) {
        float e[8], el[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          e[j] = fast_exp2(s[mt][8 * bk + j] - base);
          ls += e[j];
        }
        const uint4 ph = make_uint4(E16::pack(e[0], e[1]), E16::pack(e[2], e[3]), E16::pack(e[4], e[5]), E16::pack(e[6], e[7]));
        const uint32_t w[4] = {ph.x, ph.y, ph.z, ph.w};
#pragma unroll
        for (int j = 0; j < 4; ++j) el[2 * j] = e[2 * j] - E16::lo(w[j]), el[2 * j + 1] = e[2 * j + 1] - E16::hi(w[j]);
        const uint4 pl = make_uint4(E16::pack(el[0], el[1]), E16::pack(el[2], el[3]), E16::pack(el[4], el[5]), E16::pack(el[6], el[7]));
#pragma unroll
        for (int n = 0; n < VN; ++n) {
          const uint16_t* vr = v + (32 * n + lc) * LV + 32 * mt + 16 * bk + 4 * hh;
          const uint2 a0 = *reinterpret_cast<const uint2*>(vr), a1 = *reinterpret_cast<const uint2*>(vr + 8);
          const uint4 a = make_uint4(a0.x, a0.y, a1.x, a1.y);
          acc[n] = mfma32<bf16_tag>(a, ph, acc[n]);
          acc[n] = mfma32<bf16_tag>(a, pl, acc[n]);
        }
      }
    l += ls;
  }
  l += __shfl_xor(l, 32, 64);
  if (!valid) return;
  const float inv = 1.0f / l;
  uint16_t* o = p.out + (int64_t)(s0 + tile0 + qi) * p.out_stride + (int64_t)head * p.vdim;
#pragma unroll
  for (int n = 0; n < VN; ++n)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int d = 32 * n + 8 * i + 4 * hh;
      if (d < p.vdim)   // vdim is a multiple of 8
        *reinterpret_cast<uint2*>(o + d) = make_uint2(E16::pack(acc[n][4 * i] * inv, acc[n][4 * i + 1] * inv),
                                                      E16::pack(acc[n][4 * i + 2] * inv, acc[n][4 * i + 3] * inv));
    }
}

template <int RN, int NHT>
int launch_decode(const LatentDecodeParams& p, int reqs, hipStream_t s) {
  constexpr int LD = 64 * RN + 8, PL = 72;
  constexpr int lds = (64 * LD + 2 * 16 * NHT * PL) * 2 + 4 * 16 * NHT * 4;
  auto kern = latent_decode_kernel<RN, NHT>;
  if (lds > 65536 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess)
    return MI_ERR_LAUNCH;
  hipLaunchKernelGGL(kern, dim3(p.nsplit, (p.H + 16 * NHT - 1) / (16 * NHT), reqs), dim3(256 * NHT), lds, s, p);
  return launch_status();
}

template <int KT, int VN>
int launch_prefill(const LatentPrefillParams& p, int reqs, int max_q, hipStream_t s) {
  constexpr int lds = 2 * (64 * (16 * KT + 8) + 32 * VN * 68) * 2;
  auto kern = latent_prefill_kernel<KT, VN>;
  if (lds > 65536 && hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess)
    return MI_ERR_LAUNCH;
  hipLaunchKernelGGL(kern, dim3((p.H + 7) / 8 * 8 * ((max_q + 127) / 128), reqs), dim3(256), lds, s, p);
  return launch_status();
}

inline int rank_tiles(int rank) { return rank <= 64 ? 1 : rank <= 128 ? 2 : rank <= 256 ? 4 : 8; }

inline int decode_splits(int reqs, int head_groups, int span) {
  // a workgroup for every CU, at least 128 cache rows each
  const int want = (256 + reqs * head_groups - 1) / (reqs * head_groups);
  const int most = (span + 127) / 128;
  const int n = want < most ? want : most;
  return n < 1 ? 1 : n > 64 ? 64 : n;
}

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int mi_head_gemm_nt(void* y, const void* x, const void* w, int32_t rows, int32_t heads, int32_t n, int32_t k,
                               int64_t y_row_stride, int64_t x_row_stride, int64_t w_head_stride, void* stream) {
  if (rows == 0) return MI_OK;
  if (!y || !x || !w || rows < 0 || heads <= 0 || n <= 0 || k <= 0) return MI_ERR_INVALID_ARG;
  if (y_row_stride < (int64_t)heads * n || x_row_stride < (int64_t)heads * k || w_head_stride < (int64_t)n * k) return MI_ERR_INVALID_ARG;
  if (k % 8 || n % 4 || x_row_stride % 8 || y_row_stride % 4 || w_head_stride % 8 || !aligned16(x) || !aligned16(w) || ((uintptr_t)y & 7))
    return MI_ERR_UNSUPPORTED;
#define MI_HG(TT, FULL)                                                                                                           \
  hipLaunchKernelGGL((head_gemm_nt_kernel<TT, FULL>), dim3((n + 63) / 64, heads, (rows + 16 * TT - 1) / (16 * TT)), dim3(256), 0, \
                     (hipStream_t)stream, (uint16_t*)y, (const uint16_t*)x, (const uint16_t*)w, rows, n, k, y_row_stride, x_row_stride, w_head_stride)
  if (k % 32 == 0) {
    if (rows <= 16) MI_HG(1, true);
    else if (rows <= 32) MI_HG(2, true);
    else MI_HG(4, true);
  } else {
    if (rows <= 16) MI_HG(1, false);
    else MI_HG(4, false);
  }
#undef MI_HG
  return launch_status();
}

extern "C" int64_t mi_latent_decode_workspace_bytes(int32_t num_reqs, int32_t heads, int32_t kv_rank, int32_t window, int32_t max_seq_len) {
  if (num_reqs <= 0 || heads <= 0 || kv_rank <= 0) return 0;
  const int groups = heads > 16 ? (heads + 31) / 32 : 1;
  const int ns = decode_splits(num_reqs, groups, window < max_seq_len ? window : max_seq_len);
  return ns == 1 ? 0 : (int64_t)num_reqs * ns * heads * (kv_rank + 4) * 4;
}

extern "C" int mi_latent_decode(void* out, const void* q, const void* cache, const int32_t* block_table, const int32_t* seq_lens,
                                int32_t num_reqs, int32_t heads, int32_t kv_rank, int32_t block_size, int32_t window,
                                int32_t max_seq_len, float scale, int64_t cache_block_stride, int64_t cache_token_stride,
                                int64_t table_stride, void* workspace, int64_t workspace_bytes, void* stream) {
  if (num_reqs == 0) return MI_OK;
  if (!out || !q || !cache || !block_table || !seq_lens) return MI_ERR_INVALID_ARG;
  if (num_reqs < 0 || heads <= 0 || kv_rank <= 0 || block_size <= 0 || window <= 0 || max_seq_len <= 0) return MI_ERR_INVALID_ARG;
  if (kv_rank > 512 || kv_rank % 8 || !is_pow2(block_size) || cache_block_stride % 8 || cache_token_stride % 8 || !aligned16(out) ||
      !aligned16(q) || !aligned16(cache))
    return MI_ERR_UNSUPPORTED;
  const int64_t need = mi_latent_decode_workspace_bytes(num_reqs, heads, kv_rank, window, max_seq_len);
  if (need > workspace_bytes || (need && (!workspace || !aligned16(workspace)))) return MI_ERR_WORKSPACE;
  const int groups = heads > 16 ? (heads + 31) / 32 : 1;
  int bs_log2 = 0;
  while ((1 << bs_log2) < block_size) ++bs_log2;
  LatentDecodeParams p{(uint16_t*)out, (const uint16_t*)q, (const uint16_t*)cache, block_table, seq_lens, (float*)workspace,
                       cache_block_stride, cache_token_stride, table_stride, heads, kv_rank, bs_log2, window,
                       decode_splits(num_reqs, groups, window < max_seq_len ? window : max_seq_len), scale * kLog2e};
  hipStream_t s = (hipStream_t)stream;
  int rc;
#define MI_LD(RN) (heads > 16 ? launch_decode<RN, 2>(p, num_reqs, s) : launch_decode<RN, 1>(p, num_reqs, s))
  switch (rank_tiles(kv_rank)) {
    case 1: rc = MI_LD(1); break;
    case 2: rc = MI_LD(2); break;
    case 4: rc = MI_LD(4); break;
    default: rc = MI_LD(8); break;
  }
#undef MI_LD
  if (rc != MI_OK || p.nsplit == 1) return rc;
  hipLaunchKernelGGL(latent_decode_merge_kernel, dim3(heads, num_reqs), dim3(128), 0, s, (uint16_t*)out, (const float*)workspace, heads,
                     kv_rank, p.nsplit);
  return launch_status();
}

extern "C" int mi_latent_gather(void* ctx, const void* cache, const int32_t* ctx_start, const int32_t* block_table,
                                const int32_t* seq_lens, const int32_t* query_start_loc, int32_t num_reqs, int32_t ctx_rows,
                                int32_t kv_rank, int32_t block_size, int32_t window, int64_t cache_block_stride,
                                int64_t cache_token_stride, int64_t table_stride, void* stream) {
  if (num_reqs == 0 || ctx_rows == 0) return MI_OK;
  if (!ctx || !cache || !ctx_start || !block_table || !seq_lens || !query_start_loc) return MI_ERR_INVALID_ARG;
  if (num_reqs < 0 || ctx_rows < 0 || kv_rank <= 0 || block_size <= 0 || window <= 0) return MI_ERR_INVALID_ARG;
  if (kv_rank % 8 || cache_block_stride % 8 || cache_token_stride % 8 || !aligned16(ctx) || !aligned16(cache)) return MI_ERR_UNSUPPORTED;
  const int64_t items = (int64_t)ctx_rows * (kv_rank / 8);
  hipLaunchKernelGGL(latent_gather_kernel, dim3((unsigned)((items + 255) / 256)), dim3(256), 0, (hipStream_t)stream, (uint16_t*)ctx,
                     (const uint16_t*)cache, ctx_start, block_table, seq_lens, query_start_loc, num_reqs, ctx_rows, kv_rank, block_size,
                     window, cache_block_stride, cache_token_stride, table_stride);
  return launch_status();
}

extern "C" int mi_latent_prefill(void* out, const void* q, const void* k, const void* vt, const int32_t* ctx_start,
                                 const int32_t* seq_lens, const int32_t* query_start_loc, int32_t num_reqs, int32_t max_query_len,
                                 int32_t heads, int32_t dim, int32_t vdim, int32_t window, float scale, int64_t out_stride,
                                 int64_t q_stride, int64_t k_stride, int64_t vt_stride, void* stream) {
  if (num_reqs == 0) return MI_OK;
  if (!out || !q || !k || !vt || !ctx_start || !seq_lens || !query_start_loc) return MI_ERR_INVALID_ARG;
  if (num_reqs < 0 || max_query_len <= 0 || heads <= 0 || dim <= 0 || vdim <= 0 || window <= 0) return MI_ERR_INVALID_ARG;
  if (dim % 8 || vdim % 8 || dim > 256 || vdim > 256 || out_stride % 4 || q_stride % 8 || k_stride % 8 || vt_stride % 8 || !aligned16(q) ||
      !aligned16(k) || !aligned16(vt) || ((uintptr_t)out & 7))
    return MI_ERR_UNSUPPORTED;
  const LatentPrefillParams p{(uint16_t*)out, (const uint16_t*)q, (const uint16_t*)k, (const uint16_t*)vt, ctx_start, seq_lens,
                              query_start_loc, q_stride, k_stride, out_stride, vt_stride, heads, dim, vdim, window, scale * kLog2e};
  hipStream_t s = (hipStream_t)stream;
#define MI_LP(KT)                                                                       \
  (vdim <= 64 ? launch_prefill<KT, 2>(p, num_reqs, max_query_len, s)                    \
   : vdim <= 128 ? launch_prefill<KT, 4>(p, num_reqs, max_query_len, s) : launch_prefill<KT, 8>(p, num_reqs, max_query_len, s))
  return dim <= 64 ? MI_LP(4) : dim <= 128 ? MI_LP(8) : MI_LP(16);
#undef MI_LP
}
