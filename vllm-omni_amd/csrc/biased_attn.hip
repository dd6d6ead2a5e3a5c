// Attention with per-head query / key norms, a query temperature that grows with the position, a distance bias and a sink:
//   q = rms_norm(q; wq) * (1 + coef ln(floor((p + 1) / every) + 1)),   k = rms_norm(k; wk)
//   score_ij = scale q_i . k_j - slope_h (i - j);   the softmax's denominator also holds exp(sink_h)
// The framework's paged-attention kernels take the bias and the sink (16-bit, head sizes 64 and 128); this file has
//   * head_norm_cache: norms, temperature and the K / V cache write of a step's tokens in one launch.  Heads are laid out
//     `hd` apart in q and in the cache (hd >= dim, vdim): smaller heads are padded with zeros to the sizes those kernels
//     are built for;
//   * attn_rows: one workgroup per (row, head), any sizes and types (32-bit models and other head sizes).
#include "row_io.h"

namespace mi {
namespace {

struct HeadNormParams {
  const void* x;         // [rows][ld]: q (H dim) | k (G dim) | v (G vdim)
  const void* wq;        // nullptr: no norm
  const void* wk;
  void* q_out;           // [rows][H hd]
  void* kc;
  void* vc;
  const int64_t* slots;
  const int64_t* positions;
  int64_t ld, q_stride, block_stride, token_stride, head_stride;
  int rows, H, G, dim, vdim, hd, block_size;
  int64_t every;
  float coef, eps;
};

__device__ __forceinline__ float temperature(const HeadNormParams& p, int64_t row) {
  if (p.coef == 0.f) return 1.f;
  const int64_t n = (p.positions[row] + 1) / p.every;
  return 1.f + p.coef * logf((float)n + 1.f);
}

// LPH lanes per head, VEC values a lane at a time (U times)
template <typename T, int LPH, int VEC, int U>
__global__ __launch_bounds__(256) void head_norm_cache_kernel(const HeadNormParams p) {
  scalar_cache_acquire();
  const int units = p.H + 2 * p.G;
  const int64_t item = ((int64_t)blockIdx.x * 256 + threadIdx.x) / LPH;
  if (item >= (int64_t)p.rows * units) return;      // whole lane groups leave
  const int sub = threadIdx.x % LPH;
  const int64_t row = item / units;
  const int u = (int)(item % units);
  const T* x = reinterpret_cast<const T*>(p.x) + row * p.ld;
  const bool is_q = u < p.H, is_v = u >= p.H + p.G;
  const int n = is_v ? p.vdim : p.dim;
  T* dst;
  const T* w = nullptr;
  if (is_q) {
    x += (int64_t)u * p.dim;
    w = reinterpret_cast<const T*>(p.wq);
    dst = reinterpret_cast<T*>(p.q_out) + row * p.q_stride + (int64_t)u * p.hd;
  } else {
    const int kh = is_v ? u - p.H - p.G : u - p.H;
    x += (int64_t)(p.H + (is_v ? p.G : 0)) * p.dim + (int64_t)kh * n;
    if (!is_v) w = reinterpret_cast<const T*>(p.wk);
    const int64_t slot = p.slots[row];
    if (slot < 0) return;
    dst = reinterpret_cast<T*>(is_v ? p.vc : p.kc) + (slot / p.block_size) * p.block_stride + (slot % p.block_size) * p.token_stride +
          kh * p.head_stride;
  }
  float v[U][VEC];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < U; ++k) {
    const int c = (sub + k * LPH) * VEC;
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[k][j] = 0.f;
    if (c < n) Io<T>::template ldv<VEC>(x + c, v[k]);
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += v[k][j] * v[k][j];
  }
  if (w) {
#pragma unroll
    for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
    const float inv = inv_rms(ss, n, p.eps) * (is_q ? temperature(p, row) : 1.f);
#pragma unroll
    for (int k = 0; k < U; ++k) {
      const int c = (sub + k * LPH) * VEC;
      if (c >= n) continue;
      float ww[VEC];
      Io<T>::template ldv<VEC>(w + c, ww);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[k][j] *= inv * ww[j];
    }
  }
#pragma unroll
  for (int k = 0; k < U; ++k) {
    const int c = (sub + k * LPH) * VEC;
    if (c < p.hd) Io<T>::template stv<VEC>(dst + c, v[k]);      // zeros behind the head's own values
  }
}

struct AttnRowsParams {
  void* out;             // [rows][out_stride], heads hd apart
  const void* q;         // [rows][q_stride], heads hd apart
  const void* kc;
  const void* vc;
  const int32_t* table;
  const int32_t* seq_lens;
  const int32_t* qsl;
  const float* slopes;   // nullptr: no distance bias
  const float* sink;     // nullptr: none
  int64_t q_stride, out_stride, block_stride, token_stride, head_stride, table_stride;
  int row0, reqs, H, G, hd, block_size;
  float scale, out_scale;
};

constexpr int kRowTile = 256;   // keys per pass

template <typename T, int RC>
__global__ __launch_bounds__(256) void attn_rows_kernel(const AttnRowsParams p) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* sq = lds;                 // [hd]
  float* sp = sq + p.hd;           // [kRowTile]
  float* smem = sp + kRowTile;     // [16]
  const int h = blockIdx.x, t = p.row0 + blockIdx.y, tid = threadIdx.x, kh = h / (p.H / p.G);
  const int r = row_request(p.qsl, p.reqs, t);
  const int pos = p.seq_lens[r] - p.qsl[r + 1] + t;
  T* out = reinterpret_cast<T*>(p.out) + (int64_t)t * p.out_stride + (int64_t)h * p.hd;
  const T* q = reinterpret_cast<const T*>(p.q) + (int64_t)t * p.q_stride + (int64_t)h * p.hd;
  if (pos < 0) {   // padded row of a graph replay
    for (int i = tid; i < p.hd; i += 256) Io<T>::st(out + i, 0.f);
    return;
  }
  for (int i = tid; i < p.hd; i += 256) sq[i] = Io<T>::ld(q + i);
  __syncthreads();
  const T* kc = reinterpret_cast<const T*>(p.kc) + kh * p.head_stride;
  const T* vc = reinterpret_cast<const T*>(p.vc) + kh * p.head_stride;
  const int32_t* tab = p.table + (int64_t)r * p.table_stride;
  auto at = [&](int key) { return (int64_t)tab[key / p.block_size] * p.block_stride + (int64_t)(key % p.block_size) * p.token_stride; };
  const float slope = p.slopes ? p.slopes[h] : 0.f;
  float acc[RC];
#pragma unroll
  for (int i = 0; i < RC; ++i) acc[i] = 0.f;
  // the sink is a term of the denominator with no value: the sums start from it
  float m = p.sink ? p.sink[h] : -INFINITY, l = p.sink ? 1.f : 0.f;
  const int wave = tid >> 6, lane = tid & 63;
  for (int k0 = 0; k0 <= pos; k0 += kRowTile) {
    const int n = min(kRowTile, pos - k0 + 1);
    for (int j = wave; j < n; j += 4) {
      const T* c = kc + at(k0 + j);
      float s = 0.f;
      for (int i = lane; i < p.hd; i += 64) s += sq[i] * Io<T>::ld(c + i);
      s = wave_allreduce_sum(s);
      if (lane == 0) sp[j] = s * p.scale - slope * (float)(pos - k0 - j);
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
      const T* c = vc + at(k0 + j);
      const float w = sp[j];
#pragma unroll
      for (int i = 0; i < RC; ++i)
        if (tid + i * 256 < p.hd) acc[i] += w * Io<T>::ld(c + tid + i * 256);
    }
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < RC; ++i)
    if (tid + i * 256 < p.hd) Io<T>::st(out + tid + i * 256, acc[i] * (p.out_scale / l));
}

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int mi_head_norm_cache(const void* x, int64_t x_stride, const void* q_weight, const void* k_weight, void* q_out,
                                  int64_t q_stride, void* k_cache, void* v_cache, const int64_t* slot_mapping,
                                  const int64_t* positions, int32_t rows, int32_t num_q_heads, int32_t num_kv_heads, int32_t dim,
                                  int32_t vdim, int32_t head_dim, int32_t block_size, int64_t cache_block_stride,
                                  int64_t cache_token_stride, int64_t cache_head_stride, float temp_coef, int64_t temp_every,
                                  float eps, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!x || !q_out || !k_cache || !v_cache || !slot_mapping || !positions || rows < 0 || num_q_heads <= 0 || num_kv_heads <= 0 ||
      dim <= 0 || vdim <= 0 || head_dim < dim || head_dim < vdim || block_size <= 0 || temp_every <= 0)
    return MI_ERR_INVALID_ARG;
  if (x_stride < (int64_t)(num_q_heads + num_kv_heads) * dim + (int64_t)num_kv_heads * vdim || q_stride < (int64_t)num_q_heads * head_dim)
    return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  const HeadNormParams p{x, q_weight, k_weight, q_out, k_cache, v_cache, slot_mapping, positions, x_stride, q_stride,
                         cache_block_stride, cache_token_stride, cache_head_stride, rows, num_q_heads, num_kv_heads, dim, vdim,
                         head_dim, block_size, temp_every, temp_coef, eps};
  const int al = dtype == MI_DTYPE_BF16 ? 8 : 4;
  const bool vec = dim % 8 == 0 && vdim % 8 == 0 && head_dim % 8 == 0 && x_stride % al == 0 && q_stride % al == 0 &&
                   cache_block_stride % al == 0 && cache_token_stride % al == 0 && cache_head_stride % al == 0 && aligned16(x) &&
                   aligned16(q_out) && aligned16(k_cache) && aligned16(v_cache) && aligned16(q_weight) && aligned16(k_weight);
  const int64_t items = (int64_t)rows * (num_q_heads + 2 * num_kv_heads);
  hipStream_t s = (hipStream_t)stream;
#define MI_HN(T, LPH, VEC, U) \
  hipLaunchKernelGGL((head_norm_cache_kernel<T, LPH, VEC, U>), dim3((unsigned)((items * LPH + 255) / 256)), dim3(256), 0, s, p)
#define MI_HN_T(T)                                        \
  do {                                                    \
    if (vec && head_dim <= 64) MI_HN(T, 8, 8, 1);         \
    else if (vec && head_dim <= 128) MI_HN(T, 16, 8, 1);  \
    else if (head_dim <= 256) MI_HN(T, 64, 1, 4);         \
    else if (head_dim <= 1024) MI_HN(T, 64, 1, 16);       \
    else return MI_ERR_UNSUPPORTED;                       \
  } while (0)
  if (dtype == MI_DTYPE_BF16) MI_HN_T(uint16_t);
  else MI_HN_T(float);
#undef MI_HN_T
#undef MI_HN
  return launch_status();
}

extern "C" int mi_attn_rows(void* out, const void* q, const void* k_cache, const void* v_cache, const int32_t* block_table,
                            const int32_t* seq_lens, const int32_t* query_start_loc, const float* slopes, const float* sink,
                            float out_scale, int32_t row0, int32_t rows, int32_t num_reqs, int32_t num_q_heads, int32_t num_kv_heads, int32_t head_dim,
                            int32_t block_size, float scale, int64_t q_stride, int64_t out_stride, int64_t cache_block_stride,
                            int64_t cache_token_stride, int64_t cache_head_stride, int64_t table_stride, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!out || !q || !k_cache || !v_cache || !block_table || !seq_lens || !query_start_loc) return MI_ERR_INVALID_ARG;
  if (row0 < 0 || rows < 0 || num_reqs <= 0 || num_q_heads <= 0 || num_kv_heads <= 0 || num_q_heads % num_kv_heads || head_dim <= 0 ||
      block_size <= 0 || q_stride < (int64_t)num_q_heads * head_dim || out_stride < (int64_t)num_q_heads * head_dim)
    return MI_ERR_INVALID_ARG;
  if (head_dim > 1024) return MI_ERR_UNSUPPORTED;
  const AttnRowsParams p{out, q, k_cache, v_cache, block_table, seq_lens, query_start_loc, slopes, sink, q_stride, out_stride,
                         cache_block_stride, cache_token_stride, cache_head_stride, table_stride, row0, num_reqs, num_q_heads,
                         num_kv_heads, head_dim, block_size, scale, out_scale};
  const dim3 grid(num_q_heads, rows), block(256);
  const size_t lds = (size_t)(head_dim + kRowTile + 16) * sizeof(float);
  hipStream_t s = (hipStream_t)stream;
#define MI_AR(T)                                                                              \
  do {                                                                                        \
    if (head_dim <= 256) hipLaunchKernelGGL((attn_rows_kernel<T, 1>), grid, block, lds, s, p); \
    else hipLaunchKernelGGL((attn_rows_kernel<T, 4>), grid, block, lds, s, p);                \
  } while (0)
  if (dtype == MI_DTYPE_BF16) MI_AR(uint16_t);
  else if (dtype == MI_DTYPE_F32) MI_AR(float);
  else return MI_ERR_UNSUPPORTED;
#undef MI_AR
  return launch_status();
}
