// Attention whose heads mix their softmax weights ("talking heads", after the softmax), with a soft cap and a distance bias
// that grows with the logarithm of the distance, over the last `window` keys:
//   s_h(i, j) = cap tanh(scale q_h(i) . k(j) / cap) - r1_h ln(1 + r2_h (i - j)),   p_h = softmax_j s_h
//   o_h(i) = sum_j (sum_g T[h, g] p_g(i, j)) v(j),   out = o * sigmoid(gate)
// The mixed weights of a head need every head's normalised weights, so the softmax's sums come first and the weights are
// formed in a second sweep over the keys.  This file has the forms for any sizes and types:
//   * row_norm_cache: RMS norms of the whole q and the whole k projection + K / V cache write, one workgroup per row;
//   * talking_attn_rows: one workgroup per row, all heads (32-bit models and sizes the matrix-core forms are not built for).
#include "row_io.h"

namespace mi {
namespace {

struct RowNormParams {
  const void* x;         // [rows][ld]: q (H dim) | k (G dim) | v (G vdim)
  const void* wq;        // nullptr: no norm
  const void* wk;
  void* q_out;           // [rows][H hd]
  void* kc;
  void* vc;
  const int64_t* slots;
  int64_t ld, q_stride, block_stride, token_stride, head_stride;
  int H, G, dim, vdim, hd, block_size;
  float eps;
};

template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void row_norm_cache_kernel(const RowNormParams p) {
  scalar_cache_acquire();
  __shared__ float smem[8];
  const int64_t row = blockIdx.x;
  const T* x = reinterpret_cast<const T*>(p.x) + row * p.ld;
  const int nq = p.H * p.dim, nk = p.G * p.dim, n = nq + nk + p.G * p.vdim;
  const int64_t slot = p.slots[row];
  const int64_t at = slot < 0 ? 0 : (slot / p.block_size) * p.block_stride + (slot % p.block_size) * p.token_stride;
  float v[MAXC][VEC];
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int m = 0; m < MAXC; ++m) {
    const int c = (threadIdx.x + m * 256) * VEC;
    if (c >= n) continue;
    Io<T>::template ldv<VEC>(x + c, v[m]);
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += v[m][j] * v[m][j];
    if (c < nq) sq += ss;
    else if (c < nq + nk) sk += ss;
  }
  sq = wave_allreduce_sum(sq);
  sk = wave_allreduce_sum(sk);
  if ((threadIdx.x & 63) == 0) smem[threadIdx.x >> 6] = sq, smem[4 + (threadIdx.x >> 6)] = sk;
  __syncthreads();
  const float iq = inv_rms(smem[0] + smem[1] + smem[2] + smem[3], nq, p.eps);
  const float ik = inv_rms(smem[4] + smem[5] + smem[6] + smem[7], nk, p.eps);
  T* q = reinterpret_cast<T*>(p.q_out) + row * p.q_stride;
  T* kc = reinterpret_cast<T*>(p.kc) + at;
  T* vc = reinterpret_cast<T*>(p.vc) + at;
#pragma unroll
  for (int m = 0; m < MAXC; ++m) {
    const int c = (threadIdx.x + m * 256) * VEC;
    if (c >= n) continue;
    float w[VEC];
    if (c < nq + nk) {
      const bool is_q = c < nq;
      const int e = is_q ? c : c - nq;
      const T* wp = reinterpret_cast<const T*>(is_q ? p.wq : p.wk);
      if (wp) {
        Io<T>::template ldv<VEC>(wp + e, w);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[m][j] *= (is_q ? iq : ik) * w[j];
      }
      const int h = e / p.dim, d = e % p.dim;
      if (is_q) Io<T>::template stv<VEC>(q + (int64_t)h * p.hd + d, v[m]);
      else if (slot >= 0) Io<T>::template stv<VEC>(kc + (int64_t)h * p.head_stride + d, v[m]);
    } else if (slot >= 0) {
      const int e = c - nq - nk;
      Io<T>::template stv<VEC>(vc + (int64_t)(e / p.vdim) * p.head_stride + e % p.vdim, v[m]);
    }
  }
  // zeros behind the heads' own values
  const int pk = p.hd - p.dim, pv = p.hd - p.vdim;
  for (int i = threadIdx.x; i < p.H * pk; i += 256) Io<T>::st(q + (int64_t)(i / pk) * p.hd + p.dim + i % pk, 0.f);
  if (slot < 0) return;
  for (int i = threadIdx.x; i < p.G * pk; i += 256) Io<T>::st(kc + (int64_t)(i / pk) * p.head_stride + p.dim + i % pk, 0.f);
  for (int i = threadIdx.x; i < p.G * pv; i += 256) Io<T>::st(vc + (int64_t)(i / pv) * p.head_stride + p.vdim + i % pv, 0.f);
}

constexpr int kRowKeys = 64;      // keys per tile of the any-size kernel

struct RowsParams {
  mi_talking_attn_args a;
  int row0, reqs;
};

inline size_t rows_lds_bytes(const mi_talking_attn_args& a) {
  return ((size_t)a.heads * a.head_dim + 2ull * a.heads * kRowKeys + (size_t)a.heads * a.vdim + 2ull * a.heads) * sizeof(float);
}

template <typename T>
__global__ __launch_bounds__(256) void talking_attn_rows_kernel(const RowsParams p) {
  scalar_cache_acquire();
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const mi_talking_attn_args& a = p.a;
  const int H = a.heads, hd = a.head_dim, V = a.vdim, tid = threadIdx.x, per = H / a.kv_heads;
  float* sq = lds;                      // [H][hd]
  float* sp = sq + H * hd;              // [H][kRowKeys] scores, then weights
  float* sm = sp + H * kRowKeys;        // [H][kRowKeys] mixed weights
  float* so = sm + H * kRowKeys;        // [H][V]
  float* ml = so + H * V;               // [H] running maximum, [H] running sum
  const int t = p.row0 + blockIdx.x;
  const int r = row_request(a.query_start_loc, p.reqs, t);
  const int pos = a.seq_lens[r] - a.query_start_loc[r + 1] + t;
  T* out = reinterpret_cast<T*>(a.out) + (int64_t)t * a.out_stride;
  if (pos < 0) {   // padded row of a graph replay
    for (int i = tid; i < H * V; i += 256) Io<T>::st(out + i, 0.f);
    return;
  }
  const T* q = reinterpret_cast<const T*>(a.q) + (int64_t)t * a.q_stride;
  for (int i = tid; i < H * hd; i += 256) sq[i] = Io<T>::ld(q + i);
  for (int i = tid; i < H * V; i += 256) so[i] = 0.f;
  for (int i = tid; i < 2 * H; i += 256) ml[i] = i < H ? -INFINITY : 0.f;
  const int32_t* tab = a.block_table + (int64_t)r * a.table_stride;
  auto at = [&](int key) {
    return (int64_t)tab[key / a.block_size] * a.cache_block_stride + (int64_t)(key % a.block_size) * a.cache_token_stride;
  };
  const int lo = pos - a.window + 1 > 0 ? pos - a.window + 1 : 0;
  const int grp = tid >> 4, sub = tid & 15, wave = tid >> 6, lane = tid & 63;
  for (int sweep = 0; sweep < 2; ++sweep) {
    for (int k0 = lo; k0 <= pos; k0 += kRowKeys) {
      const int n = min(kRowKeys, pos - k0 + 1);
      __syncthreads();
      for (int item = grp; item < H * n; item += 16) {      // sixteen lanes per product
        const int h = item / n, j = item % n;
        const T* k = reinterpret_cast<const T*>(a.k_cache) + at(k0 + j) + (h / per) * a.cache_head_stride;
        float s = 0.f;
        for (int i = sub; i < hd; i += 16) s += sq[h * hd + i] * Io<T>::ld(k + i);
        s = group_allreduce_sum<16>(s);
        if (sub == 0) {
          s *= a.scale;
          if (a.softcap > 0.f) s = a.softcap * tanhf(s / a.softcap);
          if (a.r1) s -= a.r1[h] * logf(1.f + a.r2[h] * (float)(pos - k0 - j));
          sp[h * kRowKeys + j] = sweep ? expf(s - ml[h]) / ml[H + h] : s;
        }
      }
      __syncthreads();
      if (sweep == 0) {
        for (int h = wave; h < H; h += 4) {
          const float s = lane < n ? sp[h * kRowKeys + lane] : -INFINITY;
          const float m0 = ml[h], m = fmaxf(m0, wave_allreduce_max(s));
          const float l = wave_allreduce_sum(lane < n ? expf(s - m) : 0.f);
          if (lane == 0) ml[h] = m, ml[H + h] = ml[H + h] * expf(m0 - m) + l;
        }
        continue;
      }
      for (int i = tid; i < H * n; i += 256) {
        const int h = i / n, j = i % n;
        float s = 0.f;
        for (int g = 0; g < H; ++g) s += a.talk[(int64_t)h * H + g] * sp[g * kRowKeys + j];
        sm[h * kRowKeys + j] = s;
      }
      __syncthreads();
      for (int i = tid; i < H * V; i += 256) {
        const int h = i / V;
        const T* v = reinterpret_cast<const T*>(a.v_cache) + (h / per) * a.cache_head_stride + i % V;
        float s = so[i];
        for (int j = 0; j < n; ++j) s += sm[h * kRowKeys + j] * Io<T>::ld(v + at(k0 + j));
        so[i] = s;
      }
    }
  }
  const T* gate = reinterpret_cast<const T*>(a.gate) + (int64_t)t * a.gate_stride;
  for (int i = tid; i < H * V; i += 256) {      // every thread reads the sums it wrote
    float o = so[i];
    if (a.gate) o *= sigmoid_f(Io<T>::ld(gate + i));
    Io<T>::st(out + i, o);
  }
}

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int mi_row_norm_cache(const void* x, int64_t x_stride, const void* q_weight, const void* k_weight, void* q_out,
                                 int64_t q_stride, void* k_cache, void* v_cache, const int64_t* slot_mapping, int32_t rows,
                                 int32_t num_q_heads, int32_t num_kv_heads, int32_t dim, int32_t vdim, int32_t head_dim,
                                 int32_t block_size, int64_t cache_block_stride, int64_t cache_token_stride,
                                 int64_t cache_head_stride, float eps, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!x || !q_out || !k_cache || !v_cache || !slot_mapping || rows < 0 || num_q_heads <= 0 || num_kv_heads <= 0 || dim <= 0 ||
      vdim <= 0 || head_dim < dim || head_dim < vdim || block_size <= 0)
    return MI_ERR_INVALID_ARG;
  const int64_t n = (int64_t)(num_q_heads + num_kv_heads) * dim + (int64_t)num_kv_heads * vdim;
  if (x_stride < n || q_stride < (int64_t)num_q_heads * head_dim) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  const RowNormParams p{x, q_weight, k_weight, q_out, k_cache, v_cache, slot_mapping, x_stride, q_stride, cache_block_stride,
                        cache_token_stride, cache_head_stride, num_q_heads, num_kv_heads, dim, vdim, head_dim, block_size, eps};
  const int al = dtype == MI_DTYPE_BF16 ? 8 : 4;
  const bool vec = dim % 8 == 0 && vdim % 8 == 0 && head_dim % 8 == 0 && x_stride % al == 0 && q_stride % al == 0 &&
                   cache_block_stride % al == 0 && cache_token_stride % al == 0 && cache_head_stride % al == 0 && aligned16(x) &&
                   aligned16(q_out) && aligned16(k_cache) && aligned16(v_cache) && aligned16(q_weight) && aligned16(k_weight);
  const dim3 grid(rows), block(256);
  hipStream_t s = (hipStream_t)stream;
#define MI_RN(T, VEC, MAXC) hipLaunchKernelGGL((row_norm_cache_kernel<T, VEC, MAXC>), grid, block, 0, s, p)
#define MI_RN_T(T)                               \
  do {                                           \
    if (vec && n <= 2048) MI_RN(T, 8, 1);        \
    else if (vec && n <= 4096) MI_RN(T, 8, 2);   \
    else if (vec && n <= 8192) MI_RN(T, 8, 4);   \
    else if (vec && n <= 16384) MI_RN(T, 8, 8);  \
    else if (vec && n <= 32768) MI_RN(T, 8, 16); \
    else if (n <= 1024) MI_RN(T, 1, 4);          \
    else if (n <= 8192) MI_RN(T, 1, 32);         \
    else return MI_ERR_UNSUPPORTED;              \
  } while (0)
  if (dtype == MI_DTYPE_BF16) MI_RN_T(uint16_t);
  else MI_RN_T(float);
#undef MI_RN_T
#undef MI_RN
  return launch_status();
}

extern "C" int mi_talking_attn_rows(const mi_talking_attn_args* args, int32_t row0, int32_t rows, int32_t num_reqs, int dtype,
                                    void* stream) {
  if (rows == 0) return MI_OK;
  if (!args) return MI_ERR_INVALID_ARG;
  const mi_talking_attn_args& a = *args;
  if (!a.out || !a.q || !a.k_cache || !a.v_cache || !a.block_table || !a.seq_lens || !a.query_start_loc || !a.talk || !a.r1 != !a.r2)
    return MI_ERR_INVALID_ARG;
  if (row0 < 0 || rows < 0 || num_reqs <= 0 || a.heads <= 0 || a.kv_heads <= 0 || a.heads % a.kv_heads || a.head_dim <= 0 ||
      a.vdim <= 0 || a.vdim > a.head_dim || a.block_size <= 0 || a.window <= 0 || a.q_stride < (int64_t)a.heads * a.head_dim ||
      a.out_stride < (int64_t)a.heads * a.vdim || (a.gate && a.gate_stride < (int64_t)a.heads * a.vdim))
    return MI_ERR_INVALID_ARG;
  const size_t bytes = rows_lds_bytes(a);
  if (bytes > 160 * 1024) return MI_ERR_UNSUPPORTED;
  const RowsParams p{a, row0, num_reqs};
  hipStream_t s = (hipStream_t)stream;
#define MI_TR(T)                                                                                                           \
  do {                                                                                                                     \
    if (bytes > 65536 && hipFuncSetAttribute(reinterpret_cast<const void*>(talking_attn_rows_kernel<T>),                   \
                                             hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) != hipSuccess)        \
      return MI_ERR_LAUNCH;                                                                                                \
    hipLaunchKernelGGL((talking_attn_rows_kernel<T>), dim3(rows), dim3(256), bytes, s, p);                                 \
  } while (0)
  if (dtype == MI_DTYPE_BF16) MI_TR(uint16_t);
  else if (dtype == MI_DTYPE_F32) MI_TR(float);
  else return MI_ERR_UNSUPPORTED;
#undef MI_TR
  return launch_status();
}
