// The chain of chunks shared by the chunked forms of linear recurrences with a matrix state: 64 tokens at a time on the
// fp32 matrix cores.  A "prep" kernel of each recurrence leaves, per (chunk, head), operands Q, Kt, P, U, a decay per state
// row and, for delta rules, W in a workspace; the scan then walks a request's chunks with the state S in registers:
//   V' = U - W S   (DELTA; else V' = U)        O = Q S + P V'        S <- diag(g) S + Kt V'
// O replaces U in the workspace.
#pragma once
#include "mfma_attn_common.h"
#include "row_io.h"

namespace mi {
namespace {

constexpr int kC = 64;             // tokens per chunk

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

// workspace of one (chunk, head): W [C][Dp], Q [C][Dp], Kt [Dp][C], P [C][C], U [C][Vp], then e^(G_C) per state row [Dp]
struct ChunkLayout {
  int Dp, Vp;
  __host__ __device__ int64_t w() const { return 0; }
  __host__ __device__ int64_t q() const { return (int64_t)kC * Dp; }
  __host__ __device__ int64_t kt() const { return 2 * (int64_t)kC * Dp; }
  __host__ __device__ int64_t pm() const { return 3 * (int64_t)kC * Dp; }
  __host__ __device__ int64_t u() const { return 3 * (int64_t)kC * Dp + kC * kC; }
  __host__ __device__ int64_t g() const { return u() + (int64_t)kC * Vp; }
  __host__ __device__ int64_t size() const { return g() + Dp; }
};

struct ScanParams {
  float* state;          // [slots][H][D][V]
  const int32_t* slots;
  const int32_t* qsl;
  const int32_t* seq_lens;
  int req0, H, D, V;
  // segments (recurrences without a delta term and one decay per head): a request's chunks in runs of seg_chunks
  const float* log2_decay = nullptr;   // [H]
  float* seg_state = nullptr;          // [requests][nseg][H][D][V]: end state of each run but the last, from zeros except the
                                       // first; the last place holds what the request started from
  int nseg = 1, seg_chunks = 1 << 28;
};
constexpr int kMaxSegments = 8;

template <typename P>
__device__ __forceinline__ int64_t chunk_base(const P& p, int r) {
  return (p.qsl[r] - p.qsl[p.req0]) / kC + (r - p.req0);
}

// LDS-only barrier: register loads in flight stay in flight
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// NV 16-column value tiles a workgroup: its four waves read every operand of a chunk once for all of them (the bound is the
// L2 traffic of those operands, each head's tiles reading the same ones).  ENDS: only the end state of a segment.
template <int DT, int NV, bool DELTA, bool ENDS = false>
__global__ __launch_bounds__(256, 1) void chunk_scan_kernel(const ScanParams p, float* ws, const ChunkLayout lay, int nvg) {
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
  const int all = (L + kC - 1) / kC;                                   // the request's chunks
  const int seg = DELTA ? 0 : blockIdx.z, segs = DELTA ? 1 : (all + p.seg_chunks - 1) / p.seg_chunks;
  if (!DELTA && (ENDS ? seg >= segs - 1 : seg >= segs)) return;
  const int first = DELTA ? 0 : seg * p.seg_chunks;
  const int nck = DELTA ? all : min(p.seg_chunks, all - first);
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, lr = lane & 15, lg = lane >> 4;
  const int v0 = vg * 16 * NV + lr;        // + 16 n: this lane's value columns
  float* S = p.state + (((int64_t)p.slots[r] * p.H + h) * p.D) * p.V;
  auto seg_at = [&](int k) { return p.seg_state + ((((int64_t)(r - p.req0) * p.nseg + k) * p.H + h) * p.D) * p.V; };
  f32x4_t st[NV][MT] = {};
  auto add_state = [&](const float* src, float keep) {      // st <- keep st + src
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int d = (wave + 4 * m) * 16 + 4 * lg + i, v = v0 + 16 * n;
          const bool in = d < p.D && v < p.V;
          const float x = src[in ? (int64_t)d * p.V + v : 0];
          st[n][m][i] = st[n][m][i] * keep + (in ? x : 0.f);
        }
  };
  auto put_state = [&](float* dst) {
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int d = (wave + 4 * m) * 16 + 4 * lg + i, v = v0 + 16 * n;
          if (d < p.D && v < p.V) dst[(int64_t)d * p.V + v] = st[n][m][i];
        }
  };
  if (DELTA || segs == 1) {
    if (start > 0) add_state(S, 0.f);
  } else if constexpr (ENDS) {
    // the first segment starts from the request's state and leaves a copy of it: the pass behind this one overwrites it
    if (seg == 0) {
      if (start > 0) add_state(S, 0.f);
      put_state(seg_at(p.nseg - 1));
    }
  } else {
    if (seg == 0) add_state(seg_at(p.nseg - 1), 0.f);
    const float keep = seg > 1 ? fast_exp2(p.log2_decay[h] * (float)(p.seg_chunks * kC)) : 0.f;
    for (int k = 0; k < seg; ++k) add_state(seg_at(k), keep);
  }
#pragma unroll
  for (int n = 0; n < NV; ++n)
#pragma unroll
    for (int m = 0; m < MT; ++m)
      if (wave + 4 * m < DT) *reinterpret_cast<f32x4_t*>(sS + (16 * n + lr) * LS + (wave + 4 * m) * 16 + 4 * lg) = st[n][m];
  float* base = ws + ((chunk_base(p, r) + first) * p.H + h) * lay.size();
  const int64_t step = p.H * lay.size();
  // one chunk's operands; the next chunk's are loaded a whole chunk ahead (the chain of chunks is the critical path, its
  // loads must not be).  Loads and stores are unconditional — past the last chunk the loads fetch what nobody uses, read-outs
  // replace U in the workspace — so that the number in flight is known at every wait: memory operations retire in order, and a
  // store that may or may not be there makes the wait for the loads behind it wait for its acknowledgement as well.
  struct Chunk {
    f32x4_t w[DELTA ? DT : 1], q[ENDS ? 1 : DT], pm[ENDS ? 1 : 4], kt[MT][4], u[NV], g[MT];
  };
  auto load = [&](Chunk& x, int c) {
    const float* b = base + c * step;
    const int64_t ro = (int64_t)(16 * wave + lr) * Dp + 4 * lg;
#pragma unroll
    for (int k = 0; k < DT; ++k) {
      if constexpr (DELTA) x.w[k] = *reinterpret_cast<const f32x4_t*>(b + lay.w() + ro + 16 * k);
      if constexpr (!ENDS) x.q[k] = *reinterpret_cast<const f32x4_t*>(b + lay.q() + ro + 16 * k);
    }
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int i = 0; i < 4; ++i)
        x.u[n][i] = b[lay.u() + (int64_t)(16 * wave + 4 * lg + i) * lay.Vp + v0 + 16 * n];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      if constexpr (!ENDS) x.pm[k] = *reinterpret_cast<const f32x4_t*>(b + lay.pm() + (16 * wave + lr) * kC + 16 * k + 4 * lg);
#pragma unroll
      for (int m = 0; m < MT; ++m)
        x.kt[m][k] = *reinterpret_cast<const f32x4_t*>(b + lay.kt() + (int64_t)(min(wave + 4 * m, DT - 1) * 16 + lr) * kC + 16 * k + 4 * lg);
    }
#pragma unroll
    for (int m = 0; m < MT; ++m) x.g[m] = *reinterpret_cast<const f32x4_t*>(b + lay.g() + min(wave + 4 * m, DT - 1) * 16 + 4 * lg);
  };
  auto work = [&](Chunk& x, int c) {
    f32x4_t d[NV] = {}, ao[NV] = {};
    f32x4_t sv[2][NV];       // the next k block's reads under this one's products
    auto get = [&](f32x4_t (&f)[NV], const float* b, int ld, int k) {
#pragma unroll
      for (int n = 0; n < NV; ++n) f[n] = *reinterpret_cast<const f32x4_t*>(b + (16 * n + lr) * ld + 16 * k + 4 * lg);
    };
    if constexpr (!ENDS) {
    get(sv[0], sS, LS, 0);
#pragma unroll
    for (int k = 0; k < DT; ++k) {
      if (k + 1 < DT) get(sv[(k + 1) & 1], sS, LS, k + 1);
#pragma unroll
      for (int n = 0; n < NV; ++n)
#pragma unroll
        for (int s = 0; s < 4; ++s) {
          if constexpr (DELTA) d[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w[k][s], sv[k & 1][n][s], d[n], 0, 0, 0);
          ao[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[k][s], sv[k & 1][n][s], ao[n], 0, 0, 0);
        }
      __builtin_amdgcn_sched_barrier(0);
    }
    }
#pragma unroll
    for (int n = 0; n < NV; ++n) *reinterpret_cast<f32x4_t*>(sU + (16 * n + lr) * LU + 16 * wave + 4 * lg) = x.u[n] - d[n];
    lds_barrier();
#pragma unroll
    for (int n = 0; n < NV; ++n)
#pragma unroll
      for (int m = 0; m < MT; ++m) st[n][m] *= x.g[m];
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
          if constexpr (!ENDS) ao[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.pm[k][s], uv, ao[n], 0, 0, 0);
        }
      __builtin_amdgcn_sched_barrier(0);
    }
    if constexpr (!ENDS) {
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
  if constexpr (ENDS) put_state(seg_at(seg));
  else if (seg == segs - 1) put_state(S);
}

inline int round_tiles(int n) {   // 16-column tiles of the built scans: 2, 4, 8, 16
  const int t = (n + 15) / 16;
  return t <= 2 ? 2 : t <= 4 ? 4 : t <= 8 ? 8 : 16;
}

template <bool DELTA, bool ENDS>
int launch_scan(const ScanParams& p, float* ws, const ChunkLayout& lay, int num_reqs, hipStream_t s) {
  // two value tiles a workgroup where that still leaves one for every CU
  const int nvt = lay.Vp / 16, nv = nvt % 2 == 0 && (int64_t)num_reqs * p.H * p.nseg * (nvt / 2) >= 256 ? 2 : 1, nvg = nvt / nv;
  const dim3 sg((p.H + 7) / 8 * 8 * nvg, num_reqs, ENDS ? p.nseg - 1 : p.nseg);
#define MI_SCAN(DT)                                                                                                            \
  do {                                                                                                                         \
    if (nv == 2) hipLaunchKernelGGL((chunk_scan_kernel<DT, 2, DELTA, ENDS>), sg, dim3(256), 0, s, p, ws, lay, nvg);            \
    else hipLaunchKernelGGL((chunk_scan_kernel<DT, 1, DELTA, ENDS>), sg, dim3(256), 0, s, p, ws, lay, nvg);                    \
  } while (0)
  switch (lay.Dp / 16) {
    case 2: MI_SCAN(2); break;
    case 4: MI_SCAN(4); break;
    case 8: MI_SCAN(8); break;
    default: MI_SCAN(16); break;
  }
#undef MI_SCAN
  return launch_status();
}

// recurrences without a delta term: where heads and requests leave CUs idle, a request's chunks run in segments side by side —
// one pass for the segments' end states, one for the read-outs
inline int launch_linear_scan(ScanParams p, float* ws, const ChunkLayout& lay, int num_reqs, int max_chunks, hipStream_t s) {
  const int64_t tiles = (int64_t)num_reqs * p.H * (lay.Vp / 16);
  int n = (int)(1024 / tiles);
  if (n > max_chunks / 8) n = max_chunks / 8;
  if (n > kMaxSegments) n = kMaxSegments;
  if (n > 1) {
    p.seg_chunks = (max_chunks + n - 1) / n;
    p.nseg = (max_chunks + p.seg_chunks - 1) / p.seg_chunks;
  }
  if (p.nseg > 1) {
    const int rc = launch_scan<false, true>(p, ws, lay, num_reqs, s);
    if (rc != MI_OK) return rc;
  }
  return launch_scan<false, false>(p, ws, lay, num_reqs, s);
}

inline bool chunk_layout(int32_t dim, int32_t vdim, ChunkLayout* lay) {
  if (dim <= 0 || vdim <= 0 || dim > 256 || vdim > 256) return false;
  lay->Dp = 16 * round_tiles(dim);
  lay->Vp = (vdim + 15) / 16 * 16;
  return true;
}

}  // namespace
}  // namespace mi
