// Attention over a cached latent: a token's cache entry is ONE row c [rank] shared by all heads; per head k = W_uk c and
// v = W_uv c.  No positions are encoded; a query sees the `window` tokens that end at itself.
//
// Kernels in this file work on the ABSORBED form — q' = W_uk^T q, score = q' . c * scale, o' = sum p c, o = W_uv o' — where
// the cache row is key and value at once:
//   * latent_norm_cache: RMS norm of the query latent and of the new cache row, the row written at its slot
//   * head_gemm:         y[row, head, :] = W[head] x[row, head, :] (absorb, and W_uv behind the attention)
//   * latent_attn_rows:  one workgroup per (row, head), any sizes and types (32-bit models; the exact reference of the
//     matrix-core kernels)
#include "row_io.h"

namespace mi {
namespace {

struct LatentNormParams {
  const void* x;         // [rows][ld]: query latent (nq) | cache latent (nc, may be 0)
  const void* wq;
  const void* wc;
  void* q_out;           // [rows][nq]
  void* cache;           // slot s: block s / block_size, row s % block_size
  const int64_t* slots;
  int64_t ld, block_stride, token_stride;
  int nq, nc, block_size;
  float eps;
};

template <typename T, int VEC, int MAXC>
__device__ __forceinline__ void norm_segment(const T* x, const T* w, T* out, int n, float eps, float* smem) {
  float v[MAXC][VEC];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= n) continue;
    Io<T>::template ldv<VEC>(x + c, v[k]);
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += v[k][j] * v[k][j];
  }
  const float inv = inv_rms(wg_sum(ss, smem), n, eps);
  if (out == nullptr) return;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= n) continue;
    float ww[VEC];
    Io<T>::template ldv<VEC>(w + c, ww);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[k][j] *= inv * ww[j];
    Io<T>::template stv<VEC>(out + c, v[k]);
  }
}

template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void latent_norm_cache_kernel(const LatentNormParams p) {
  scalar_cache_acquire();
  __shared__ float smem[16];
  const int64_t row = blockIdx.x;
  const T* x = reinterpret_cast<const T*>(p.x) + row * p.ld;
  if (blockIdx.y == 0) {
    norm_segment<T, VEC, MAXC>(x, reinterpret_cast<const T*>(p.wq), reinterpret_cast<T*>(p.q_out) + row * p.nq, p.nq, p.eps, smem);
  } else {
    const int64_t slot = p.slots[row];
    T* dst = slot < 0 ? nullptr
                      : reinterpret_cast<T*>(p.cache) + (slot / p.block_size) * p.block_stride + (slot % p.block_size) * p.token_stride;
    norm_segment<T, VEC, MAXC>(x + p.nq, reinterpret_cast<const T*>(p.wc), dst, p.nc, p.eps, smem);
  }
}

// y[row][h][n] = sum_k x[row][h][k] w(h, n, k), element strides of w given; one thread per output column
template <typename T>
__global__ __launch_bounds__(64) void head_gemm_kernel(T* y, const T* x, const T* w, int N, int Kd, int64_t y_row, int64_t x_row,
                                                       int64_t w_head, int64_t w_n, int64_t w_k) {
  scalar_cache_acquire();
  const int h = blockIdx.y;
  const int64_t row = blockIdx.x;
  const int n = blockIdx.z * 64 + threadIdx.x;
  if (n >= N) return;
  const T* xr = x + row * x_row + (int64_t)h * Kd;
  const T* wr = w + h * w_head + n * w_n;
  float acc = 0.f;
  for (int k = 0; k < Kd; ++k) acc += Io<T>::ld(xr + k) * Io<T>::ld(wr + k * w_k);
  Io<T>::st(y + row * y_row + (int64_t)h * N + n, acc);
}

struct LatentRowsParams {
  void* out;             // [rows][H][rank]
  const void* q;         // [rows][H][rank]
  const void* cache;
  const int32_t* table;  // [reqs][table_stride]
  const int32_t* seq_lens;
  const int32_t* qsl;
  int64_t block_stride, token_stride, table_stride;
  int row0, reqs, H, rank, block_size, window;
  float scale;
};

constexpr int kRowTile = 256;   // keys per pass

template <typename T, int RC>
__global__ __launch_bounds__(256) void latent_attn_rows_kernel(const LatentRowsParams p) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* sq = lds;                 // [rank]
  float* sp = sq + p.rank;         // [kRowTile]
  float* smem = sp + kRowTile;     // [16]
  const int h = blockIdx.x, t = p.row0 + blockIdx.y, tid = threadIdx.x;
  const int r = row_request(p.qsl, p.reqs, t);
  const int pos = p.seq_lens[r] - p.qsl[r + 1] + t;
  const int64_t io = ((int64_t)t * p.H + h) * p.rank;
  T* out = reinterpret_cast<T*>(p.out) + io;
  const T* q = reinterpret_cast<const T*>(p.q) + io;
  if (pos < 0) {   // padded row of a graph replay
    for (int i = tid; i < p.rank; i += 256) Io<T>::st(out + i, 0.f);
    return;
  }
  for (int i = tid; i < p.rank; i += 256) sq[i] = Io<T>::ld(q + i);
  __syncthreads();
  const T* cache = reinterpret_cast<const T*>(p.cache);
  const int32_t* tab = p.table + (int64_t)r * p.table_stride;
  float acc[RC];
#pragma unroll
  for (int i = 0; i < RC; ++i) acc[i] = 0.f;
  float m = -INFINITY, l = 0.f;
  const int wave = tid >> 6, lane = tid & 63;
  for (int k0 = max(0, pos - p.window + 1); k0 <= pos; k0 += kRowTile) {
    const int n = min(kRowTile, pos - k0 + 1);
    for (int j = wave; j < n; j += 4) {
      const int key = k0 + j;
      const T* c = cache + (int64_t)tab[key / p.block_size] * p.block_stride + (int64_t)(key % p.block_size) * p.token_stride;
      float s = 0.f;
      for (int i = lane; i < p.rank; i += 64) s += sq[i] * Io<T>::ld(c + i);
      s = wave_allreduce_sum(s);
      if (lane == 0) sp[j] = s * p.scale;
    }
    __syncthreads();
    float mx = tid < n ? sp[tid] : -INFINITY;
    mx = wave_allreduce_max(mx);
    if (lane == 0) smem[wave] = mx;
    __syncthreads();
    const float mn = fmaxf(m, fmaxf(fmaxf(smem[0], smem[1]), fmaxf(smem[2], smem[3])));
    const float e = tid < n ? expf(sp[tid] - mn) : 0.f;
    __syncthreads();
    sp[tid] = e;
    const float f = expf(m - mn);
    l = l * f + wg_sum(e, smem);   // its barriers also publish sp
    m = mn;
#pragma unroll
    for (int i = 0; i < RC; ++i) acc[i] *= f;
    for (int j = 0; j < n; ++j) {
      const int key = k0 + j;
      const T* c = cache + (int64_t)tab[key / p.block_size] * p.block_stride + (int64_t)(key % p.block_size) * p.token_stride;
      const float w = sp[j];
#pragma unroll
      for (int i = 0; i < RC; ++i)
        if (tid + i * 256 < p.rank) acc[i] += w * Io<T>::ld(c + tid + i * 256);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < RC; ++i)
    if (tid + i * 256 < p.rank) Io<T>::st(out + tid + i * 256, acc[i] / l);
}

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int mi_latent_norm_cache(const void* x, int64_t x_stride, const void* q_weight, int32_t q_rank, void* q_out,
                                    const void* c_weight, int32_t kv_rank, void* cache, const int64_t* slot_mapping,
                                    int32_t block_size, int64_t cache_block_stride, int64_t cache_token_stride, float eps,
                                    int32_t rows, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!x || !q_weight || !q_out || rows < 0 || q_rank <= 0 || kv_rank < 0) return MI_ERR_INVALID_ARG;
  if (kv_rank && (!c_weight || !cache || !slot_mapping || block_size <= 0)) return MI_ERR_INVALID_ARG;
  if (x_stride < q_rank + kv_rank) return MI_ERR_INVALID_ARG;
  LatentNormParams p{x, q_weight, c_weight, q_out, cache, slot_mapping, x_stride, cache_block_stride, cache_token_stride,
                     q_rank, kv_rank, block_size, eps};
  const bool vec = q_rank % 8 == 0 && kv_rank % 8 == 0 && x_stride % 8 == 0 && cache_block_stride % 8 == 0 &&
                   cache_token_stride % 8 == 0 && aligned16(x) && aligned16(q_weight) && aligned16(c_weight) && aligned16(q_out) &&
                   aligned16(cache);
  const int n = q_rank > kv_rank ? q_rank : kv_rank;
  if (n > (vec ? 8192 : 4096)) return MI_ERR_UNSUPPORTED;
  const dim3 grid(rows, kv_rank ? 2 : 1), block(256);
  hipStream_t s = (hipStream_t)stream;
#define MI_LN(T)                                                                                 \
  do {                                                                                           \
    if (vec && n <= 2048) hipLaunchKernelGGL((latent_norm_cache_kernel<T, 8, 1>), grid, block, 0, s, p); \
    else if (vec) hipLaunchKernelGGL((latent_norm_cache_kernel<T, 8, 4>), grid, block, 0, s, p); \
    else hipLaunchKernelGGL((latent_norm_cache_kernel<T, 1, 16>), grid, block, 0, s, p);         \
  } while (0)
  if (dtype == MI_DTYPE_BF16) MI_LN(uint16_t);
  else if (dtype == MI_DTYPE_F32) MI_LN(float);
  else return MI_ERR_UNSUPPORTED;
#undef MI_LN
  return launch_status();
}

extern "C" int mi_head_gemm(void* y, const void* x, const void* w, int32_t rows, int32_t heads, int32_t n, int32_t k,
                            int64_t y_row_stride, int64_t x_row_stride, int64_t w_head_stride, int64_t w_n_stride,
                            int64_t w_k_stride, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!y || !x || !w || rows < 0 || heads <= 0 || n <= 0 || k <= 0) return MI_ERR_INVALID_ARG;
  if (y_row_stride < (int64_t)heads * n || x_row_stride < (int64_t)heads * k) return MI_ERR_INVALID_ARG;
  const dim3 grid(rows, heads, (n + 63) / 64), block(64);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MI_DTYPE_BF16)
    hipLaunchKernelGGL((head_gemm_kernel<uint16_t>), grid, block, 0, s, (uint16_t*)y, (const uint16_t*)x, (const uint16_t*)w, n, k,
                       y_row_stride, x_row_stride, w_head_stride, w_n_stride, w_k_stride);
  else if (dtype == MI_DTYPE_F32)
    hipLaunchKernelGGL((head_gemm_kernel<float>), grid, block, 0, s, (float*)y, (const float*)x, (const float*)w, n, k,
                       y_row_stride, x_row_stride, w_head_stride, w_n_stride, w_k_stride);
  else return MI_ERR_UNSUPPORTED;
  return launch_status();
}

extern "C" int mi_latent_attn_rows(void* out, const void* q, const void* cache, const int32_t* block_table, const int32_t* seq_lens,
                                   const int32_t* query_start_loc, int32_t row0, int32_t rows, int32_t num_reqs, int32_t heads,
                                   int32_t kv_rank, int32_t block_size, int32_t window, float scale, int64_t cache_block_stride,
                                   int64_t cache_token_stride, int64_t table_stride, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!out || !q || !cache || !block_table || !seq_lens || !query_start_loc) return MI_ERR_INVALID_ARG;
  if (row0 < 0 || rows < 0 || num_reqs <= 0 || heads <= 0 || kv_rank <= 0 || block_size <= 0 || window <= 0) return MI_ERR_INVALID_ARG;
  if (kv_rank > 2048) return MI_ERR_UNSUPPORTED;
  LatentRowsParams p{out, q, cache, block_table, seq_lens, query_start_loc, cache_block_stride, cache_token_stride, table_stride,
                     row0, num_reqs, heads, kv_rank, block_size, window, scale};
  const dim3 grid(heads, rows), block(256);
  const size_t lds = (size_t)(kv_rank + kRowTile + 16) * sizeof(float);
  hipStream_t s = (hipStream_t)stream;
#define MI_LR(T)                                                                                      \
  do {                                                                                                \
    if (kv_rank <= 512) hipLaunchKernelGGL((latent_attn_rows_kernel<T, 2>), grid, block, lds, s, p);  \
    else hipLaunchKernelGGL((latent_attn_rows_kernel<T, 8>), grid, block, lds, s, p);                 \
  } while (0)
  if (dtype == MI_DTYPE_BF16) MI_LR(uint16_t);
  else if (dtype == MI_DTYPE_F32) MI_LR(float);
  else return MI_ERR_UNSUPPORTED;
#undef MI_LR
  return launch_status();
}
