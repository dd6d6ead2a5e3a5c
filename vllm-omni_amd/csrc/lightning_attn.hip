// Decayed linear attention ("lightning attention"): per head, with q, k, v = silu of the projections,
//   S_t = d S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,   d a constant of the head;
// the heads of a token are normed together: out = o / rms(o) * norm * sigmoid(gate) * mul.
// The projections of a row arrive side by side as q | k | v (heads x dim, heads x dim, heads x vdim).  The state
// [heads][dim][vdim] is fp32 per request slot; a request whose first token is position 0 starts from zeros.
//   * lightning_step:  a workgroup per (head, 64 value columns, request), the state in registers, token after token:
//     decode (HBM bound: the state is read and written once) and sizes outside the chunked form;
//   * prompt portions in chunks of 64 tokens: prep here, the chain of chunks in chunk_scan.h (no delta term):
//     O = diag(d^(i+1)) Q S0 + P V,  P_ij = d^(i-j) q_i . k_j (j <= i),  S1 = d^C S0 + sum_j d^(C-1-j) k_j v_j^T;
//     few heads and requests: a request's chunks in segments side by side, their end states first;
//   * finish: norm and gate, one workgroup per token.
#include "chunk_scan.h"

namespace mi {
namespace {

struct LightningParams {
  const void* qkv;          // [rows][ld]
  const float* decay;       // [H]
  const float* log2_decay;  // [H]
  float* state;
  const int32_t* slots;
  const int32_t* qsl;
  const int32_t* seq_lens;
  float* o;                 // step: read-outs [rows of the requests][H V]
  int64_t ld;
  int req0, row0, H, D, V;
};

constexpr int kCols = 64;   // value columns of a step workgroup
constexpr int kPrep = 512;

// thread: VEC columns x R rows of the state; q, k of a token are staged for everybody
template <typename T, int VEC, int R>
__global__ __launch_bounds__(256) void lightning_step_kernel(const LightningParams p) {
  scalar_cache_acquire();
  constexpr int LV = kCols / VEC, GR = 256 / LV;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int D = p.D, V = p.V;
  float* sq = lds;                 // [D]
  float* sk = sq + D;              // [D]
  float* red = sk + D;             // [GR][kCols]
  const int h = blockIdx.x, r = p.req0 + blockIdx.z, c0 = blockIdx.y * kCols;
  const int s0 = p.qsl[r], L = p.qsl[r + 1] - s0, start = p.seq_lens[r] - L;   // start < 0: a padded row of a graph replay
  if (L <= 0) return;
  const int tid = threadIdx.x, g = tid / LV, c = c0 + (tid % LV) * VEC;
  float* S = p.state + ((int64_t)p.slots[r] * p.H + h) * D * (int64_t)V;
  const bool cols = c < V;         // VEC divides V
  float st[R][VEC];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const float* src = S + (int64_t)min(g + i * GR, D - 1) * V + (cols ? c : 0);
    if constexpr (VEC == 4) {
      const f32x4_t a = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t*>(src));
      st[i][0] = a[0], st[i][1] = a[1], st[i][2] = a[2], st[i][3] = a[3];
    } else {
      st[i][0] = *src;
    }
  }
#pragma unroll
  for (int i = 0; i < R; ++i)
#pragma unroll
    for (int j = 0; j < VEC; ++j) st[i][j] = start > 0 && g + i * GR < D ? st[i][j] : 0.f;
  const float dec = p.decay[h];
  for (int i = 0; i < L; ++i) {
    const int64_t row = s0 + i;
    const T* q = reinterpret_cast<const T*>(p.qkv) + row * p.ld + (int64_t)h * D;
    const T* k = q + (int64_t)p.H * D;
    const T* v = reinterpret_cast<const T*>(p.qkv) + row * p.ld + 2 * (int64_t)p.H * D + (int64_t)h * V + (cols ? c : 0);
    float vv[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) vv[j] = silu_f(Io<T>::ld(v + j));
    for (int d = tid; d < D; d += 256) {
      const float a = Io<T>::ld(q + d), b = Io<T>::ld(k + d);
      sq[d] = silu_f(a), sk[d] = silu_f(b);
    }
    __syncthreads();
    float acc[VEC] = {};
#pragma unroll
    for (int n = 0; n < R; ++n) {
      const int d = min(g + n * GR, D - 1);
      const bool in = g + n * GR < D;
      const float kk = in ? sk[d] : 0.f, qq = in ? sq[d] : 0.f;
#pragma unroll
      for (int j = 0; j < VEC; ++j) st[n][j] = st[n][j] * dec + kk * vv[j], acc[j] += st[n][j] * qq;
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) red[g * kCols + (tid % LV) * VEC + j] = acc[j];
    __syncthreads();      // (also: every reader of sq, sk is done)
    if (tid < kCols && c0 + tid < V) {
      float t = 0.f;
#pragma unroll
      for (int n = 0; n < GR; ++n) t += red[n * kCols + tid];
      p.o[(row - p.row0) * p.H * V + (int64_t)h * V + c0 + tid] = t;
    }
  }
  if (!cols) return;
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int d = g + i * GR;
    if (d >= D) continue;
    if constexpr (VEC == 4) {
      const f32x4_t a = {st[i][0], st[i][1], st[i][2], st[i][3]};
      __builtin_nontemporal_store(a, reinterpret_cast<f32x4_t*>(S + (int64_t)d * V + c));
    } else {
      S[(int64_t)d * V + c] = st[i][0];
    }
  }
}

// silu of a chunk's q, k (to LDS) and v (to the workspace); zeros in rows past len and columns past dim / vdim
template <typename T>
__device__ __forceinline__ void silu_rows(const LightningParams& p, bool vec, float* bq, float* bk, float* bv, const ChunkLayout& lay, int h,
                                          int64_t row0, int len) {
  const int Dp = lay.Dp, Vp = lay.Vp, ldk = Dp + 4;
  const T* base = reinterpret_cast<const T*>(p.qkv) + row0 * p.ld;
  const int64_t cq = (int64_t)h * p.D, ck = (int64_t)(p.H + h) * p.D, cv = 2 * (int64_t)p.H * p.D + (int64_t)h * p.V;
  if (vec) {      // sizes, columns and the row stride are multiples of 8: six loads of a thread in flight
    const int per = (2 * Dp + Vp) / 8, total = kC * per;
    for (int it0 = threadIdx.x; it0 < total; it0 += 6 * kPrep) {
      float x[6][8];
#pragma unroll
      for (int u = 0; u < 6; ++u) {
        const int it = min(it0 + u * kPrep, total - 1), i = it / per, c = it % per * 8;
        const int64_t col = c < Dp ? cq + min(c, p.D - 8) : c < 2 * Dp ? ck + min(c - Dp, p.D - 8) : cv + min(c - 2 * Dp, p.V - 8);
        Io<T>::template ldv<8>(base + (int64_t)min(i, len - 1) * p.ld + col, x[u]);
      }
#pragma unroll
      for (int u = 0; u < 6; ++u) {
        const int it = it0 + u * kPrep, i = it / per, c = it % per * 8;
        if (it >= total) continue;
        const int cc = c < Dp ? c : c < 2 * Dp ? c - Dp : c - 2 * Dp;
        const bool in = i < len && cc < (c < 2 * Dp ? p.D : p.V);
#pragma unroll
        for (int j = 0; j < 8; ++j) x[u][j] = in ? silu_f(x[u][j]) : 0.f;
        float* dst = c < Dp ? bq + i * ldk + cc : c < 2 * Dp ? bk + i * ldk + cc : bv + i * Vp + cc;
        Io<float>::stv<8>(dst, x[u]);
      }
    }
  } else {
    for (int it = threadIdx.x; it < kC * Dp; it += kPrep) {
      const int i = it / Dp, c = it % Dp;
      const bool in = i < len && c < p.D;
      bq[i * ldk + c] = in ? silu_f(Io<T>::ld(base + (int64_t)i * p.ld + cq + c)) : 0.f;
      bk[i * ldk + c] = in ? silu_f(Io<T>::ld(base + (int64_t)i * p.ld + ck + c)) : 0.f;
    }
    for (int it = threadIdx.x; it < kC * Vp; it += kPrep) {
      const int i = it / Vp, c = it % Vp;
      bv[i * Vp + c] = i < len && c < p.V ? silu_f(Io<T>::ld(base + (int64_t)i * p.ld + cv + c)) : 0.f;
    }
  }
}

template <typename T>
__global__ __launch_bounds__(kPrep, 4) void lightning_prep_kernel(const LightningParams p, float* ws, const ChunkLayout lay, bool vec) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int r = p.req0 + blockIdx.z, h = blockIdx.y, ck = blockIdx.x;
  const int s0 = p.qsl[r], L = p.qsl[r + 1] - s0;
  const int i0 = ck * kC;
  if (i0 >= L) return;
  const int len = min(kC, L - i0);
  const int64_t row0 = s0 + i0;
  const int Dp = lay.Dp, ldk = Dp + 4, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  float* bufK = lds;
  float* bufQ = bufK + kC * ldk;
  const float lg = p.log2_decay[h];
  float* out = ws + ((chunk_base(p, r) + ck) * p.H + h) * lay.size();
  silu_rows<T>(p, vec, bufQ, bufK, out + lay.u(), lay, h, row0, len);
  for (int d = tid; d < Dp; d += kPrep) out[lay.g() + d] = fast_exp2(lg * len);
  __syncthreads();
#pragma unroll
  for (int n = 0; n < 2; ++n) {
    const int t = wave + n * (kPrep / 64), ti = t >> 2, tj = t & 3;
    f32x4_t acc = {};
    if (tj <= ti)
      for (int k = 0; k < Dp; k += 16) {
        float fa[4], fb[4];
        frag_rows(bufQ + ti * 16 * ldk + k, ldk, lane, fa);
        frag_rows(bufK + tj * 16 * ldk + k, ldk, lane, fb);
        acc = mma4(fa, fb, acc);
      }
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int i = ti * 16 + 4 * (lane >> 4) + s, j = tj * 16 + (lane & 15);
      out[lay.pm() + i * kC + j] = j <= i ? acc[s] * fast_exp2(lg * (i - j)) : 0.f;
    }
  }
  for (int n = tid; n < kC * Dp / 4; n += kPrep) {
    const int i = n / (Dp / 4), c = (n % (Dp / 4)) * 4;
    const float e = fast_exp2(lg * (i + 1));
    const float4 v = *reinterpret_cast<const float4*>(bufQ + i * ldk + c);
    *reinterpret_cast<float4*>(out + lay.q() + (int64_t)i * Dp + c) = make_float4(v.x * e, v.y * e, v.z * e, v.w * e);
  }
  for (int n = tid; n < kC * Dp; n += kPrep) {
    const int d = n / kC, j = n % kC;
    out[lay.kt() + n] = j < len ? bufK[j * ldk + d] * fast_exp2(lg * (len - 1 - j)) : 0.f;
  }
}

struct LightningFinish {
  void* out;                // [rows][ld_out]
  const void* gate;         // [rows][ld_gate]
  const void* norm_w;       // [H V]
  const float* o;           // read-outs: [rows - row0][H V] of the step, or nullptr: in the workspace of the scan
  const float* ws;
  const int32_t* qsl;
  int64_t ld_out, ld_gate;
  int req0, nreq, row0, H, V;
  float eps, mul;
  ChunkLayout lay;
};

template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void lightning_finish_kernel(const LightningFinish p) {
  scalar_cache_acquire();
  __shared__ float smem[16];
  const int64_t row = p.row0 + blockIdx.x;
  const int n = p.H * p.V;
  const float* src;
  int64_t head;             // distance of the heads' read-outs
  if (p.o) {
    src = p.o + (row - p.row0) * n;
    head = p.V;
  } else {
    const int r = p.req0 + row_request(p.qsl + p.req0, p.nreq, (int)row);
    const int i = (int)row - p.qsl[r];
    src = p.ws + (chunk_base(p, r) + i / kC) * p.H * p.lay.size() + p.lay.u() + (int64_t)(i % kC) * p.lay.Vp;
    head = p.lay.size();
  }
  float x[MAXC][VEC];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= n) continue;
    Io<float>::ldv<VEC>(src + (c / p.V) * head + c % p.V, x[k]);
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += x[k][j] * x[k][j];
  }
  const float inv = inv_rms(wg_sum(ss, smem), n, p.eps) * p.mul;
  const T* gr = reinterpret_cast<const T*>(p.gate) + row * p.ld_gate;
  T* out = reinterpret_cast<T*>(p.out) + row * p.ld_out;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= n) continue;
    float w[VEC], g[VEC];
    Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.norm_w) + c, w);
    Io<T>::template ldv<VEC>(gr + c, g);
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[k][j] *= inv * w[j] * sigmoid_f(g[j]);
    Io<T>::template stv<VEC>(out + c, x[k]);
  }
}

template <typename T>
int finish(const LightningFinish& f, int rows, hipStream_t s) {
  const int n = f.H * f.V, al = 16 / sizeof(T);
  const bool vec = f.V % 8 == 0 && f.ld_out % al == 0 && f.ld_gate % al == 0 && aligned16(f.out) && aligned16(f.gate) &&
                   aligned16(f.norm_w);
  const dim3 grid(rows), block(256);
  if (vec) {
    if (n <= 2048) hipLaunchKernelGGL((lightning_finish_kernel<T, 8, 1>), grid, block, 0, s, f);
    else if (n <= 4096) hipLaunchKernelGGL((lightning_finish_kernel<T, 8, 2>), grid, block, 0, s, f);
    else if (n <= 16384) hipLaunchKernelGGL((lightning_finish_kernel<T, 8, 8>), grid, block, 0, s, f);
    else return MI_ERR_UNSUPPORTED;
  } else {
    if (n <= 1024) hipLaunchKernelGGL((lightning_finish_kernel<T, 1, 4>), grid, block, 0, s, f);
    else if (n <= 8192) hipLaunchKernelGGL((lightning_finish_kernel<T, 1, 32>), grid, block, 0, s, f);
    else return MI_ERR_UNSUPPORTED;
  }
  return launch_status();
}

template <typename T>
int step(const LightningParams& p, int nreq, hipStream_t s) {
  const bool v4 = p.V % 4 == 0;
  const int gr = v4 ? 16 : 4, need = (p.D + gr - 1) / gr;
  const dim3 grid(p.H, (p.V + kCols - 1) / kCols, nreq), block(256);
  const size_t lds = (size_t)(2 * p.D + gr * kCols) * sizeof(float);
#define MI_LS(VEC, R) hipLaunchKernelGGL((lightning_step_kernel<T, VEC, R>), grid, block, lds, s, p)
  if (v4) {
    if (need <= 4) MI_LS(4, 4);
    else if (need <= 8) MI_LS(4, 8);
    else if (need <= 16) MI_LS(4, 16);
    else if (need <= 32) MI_LS(4, 32);
    else return MI_ERR_UNSUPPORTED;
  } else {
    if (need <= 16) MI_LS(1, 16);
    else if (need <= 64) MI_LS(1, 64);
    else if (need <= 128) MI_LS(1, 128);
    else return MI_ERR_UNSUPPORTED;
  }
#undef MI_LS
  return launch_status();
}

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int64_t mi_lightning_workspace_bytes(int32_t rows, int32_t num_reqs, int32_t heads, int32_t dim, int32_t vdim, int32_t chunked) {
  if (rows < 0 || num_reqs < 0 || heads <= 0 || dim <= 0 || vdim <= 0) return 0;
  if (!chunked) return (int64_t)rows * heads * vdim * 4;
  ChunkLayout lay;
  if (!chunk_layout(dim, vdim, &lay)) return 0;
  return ((int64_t)rows / kC + num_reqs) * heads * lay.size() * 4 + (int64_t)num_reqs * kMaxSegments * heads * dim * vdim * 4;
}

extern "C" int mi_lightning_attn(const mi_lightning_args* a, int32_t row0, int32_t rows, int32_t max_query_len, int32_t chunked,
                                 void* workspace, int64_t workspace_bytes, int dtype, void* stream) {
  if (a && (a->num_reqs == 0 || rows == 0)) return MI_OK;
  if (!a || !a->qkv || !a->gate || !a->decay || !a->log2_decay || !a->norm_w || !a->state || !a->slots || !a->query_start_loc || !a->seq_lens ||
      !a->out || !workspace)
    return MI_ERR_INVALID_ARG;
  const int H = a->heads, D = a->dim, V = a->vdim, nreq = a->num_reqs;
  if (a->req0 < 0 || nreq < 0 || row0 < 0 || rows < 0 || max_query_len <= 0 || H <= 0 || D <= 0 || V <= 0) return MI_ERR_INVALID_ARG;
  if (a->qkv_stride < (int64_t)H * (2 * D + V) || a->gate_stride < H * V || a->out_stride < H * V) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  ChunkLayout lay{0, 0};
  if (chunked && !chunk_layout(D, V, &lay)) return MI_ERR_UNSUPPORTED;
  if (workspace_bytes < mi_lightning_workspace_bytes(rows, nreq, H, D, V, chunked)) return MI_ERR_WORKSPACE;
  hipStream_t s = (hipStream_t)stream;
  float* ws = (float*)workspace;
  const LightningParams p{a->qkv, a->decay, a->log2_decay, a->state, a->slots, a->query_start_loc, a->seq_lens, ws, a->qkv_stride,
                          a->req0, row0, H, D, V};
  int rc;
  if (!chunked) {
    rc = dtype == MI_DTYPE_BF16 ? step<uint16_t>(p, nreq, s) : step<float>(p, nreq, s);
  } else {
    const int al = dtype == MI_DTYPE_BF16 ? 8 : 4;
    const bool vec = D % 8 == 0 && V % 8 == 0 && a->qkv_stride % al == 0 && aligned16(a->qkv);
    const size_t lds = (size_t)2 * kC * (lay.Dp + 4) * 4;
    const dim3 pg((max_query_len + kC - 1) / kC, H, nreq);
#define MI_PREP(T)                                                                                                        \
  do {                                                                                                                    \
    auto kern = lightning_prep_kernel<T>;                                                                                 \
    if (hipFuncSetAttribute(reinterpret_cast<const void*>(kern), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) \
      return MI_ERR_LAUNCH;                                                                                               \
    hipLaunchKernelGGL(kern, pg, dim3(kPrep), lds, s, p, ws, lay, vec);                                                   \
  } while (0)
    if (dtype == MI_DTYPE_BF16) MI_PREP(uint16_t);
    else MI_PREP(float);
#undef MI_PREP
    ScanParams sp{p.state, p.slots, p.qsl, p.seq_lens, p.req0, H, D, V};
    sp.log2_decay = p.log2_decay;
    sp.seg_state = ws + ((int64_t)rows / kC + nreq) * H * lay.size();
    rc = launch_linear_scan(sp, ws, lay, nreq, (max_query_len + kC - 1) / kC, s);
  }
  if (rc != MI_OK) return rc;
  const LightningFinish f{a->out, a->gate, a->norm_w, chunked ? nullptr : ws, ws, a->query_start_loc, a->out_stride, a->gate_stride,
                          a->req0, nreq, row0, H, V, a->eps, a->mul, lay};
  return dtype == MI_DTYPE_BF16 ? finish<uint16_t>(f, rows, s) : finish<float>(f, rows, s);
}
