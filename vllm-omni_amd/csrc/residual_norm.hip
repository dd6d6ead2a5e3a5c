// Row kernels of decoders whose residual stream is 32-bit, and the small gates of such decoders:
//   * residual_norm:   post-norm of a sublayer's output + residual add + pre-norm (or plain cast) for the next one
//     (sublayers normed on both sides: x <- x + norm_b(f(norm_a(x))))
//   * residual_add_norm: residual add of a layer's output (and of its routed experts' rows, weighted) + pre-norm or cast
//     for what follows; also starts a stream from a projection (no add)
//   * embed_norm:      token embedding + the first pre-norm or cast
//   * stream_norm2:    residual add times a multiplier, what a pass of looped layers adds, and TWO norms of the sum (mixer and
//     feed-forward each read a norm of their own); also starts a stream from the embedding
//   * pair_embed_norm: scaled token embedding + the row of the (previous, current) token pair + the first pre-norm
//   * gelu_lookup_mul: gelu_tanh(z) * (a slice of a per-token table row)
//   * clamped_glu:     g sigmoid(alpha g) (u + 1) on clamped g, u
//   * glu:             act(g) * u, act silu or the tanh form of gelu
//   * activation:      act(z) of one projection, act the square of relu; also from a projection's split-K partials
//   * input_conv:      h + a causal filter per channel over h's last rows (what a sublayer reads); for one-token rows it
//     rides in residual_add_norm
// One workgroup per row, the row stays in registers; fp32 arithmetic, one rounding to the output type.  All of them
// stream: the bound is HBM (or launch latency at decode sizes).
#include "row_io.h"

namespace mi {
namespace {

struct ResidualNormParams {
  float* x;
  const void* y;        // T rows, or fp32 split-K partials [split][rows][width] (split >= 1)
  const void* w_post;
  const void* w_pre;    // nullptr: h = x cast
  void* h;              // nullptr: no output
  int64_t x_stride, y_stride, h_stride;
  int rows, width, split;
  float eps;
};

template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void residual_norm_kernel(const ResidualNormParams p) {
  scalar_cache_acquire();
  __shared__ float smem[16];
  const int64_t row = blockIdx.x;
  float* xr = p.x + row * p.x_stride;
  float y[MAXC][VEC], x[MAXC][VEC];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= p.width) continue;
    Io<float>::ldv<VEC>(xr + c, x[k]);
    if (p.split) {
      const float* yp = reinterpret_cast<const float*>(p.y) + row * p.width + c;
      Io<float>::ldv<VEC>(yp, y[k]);
      for (int s = 1; s < p.split; ++s) {
        float t[VEC];
        Io<float>::ldv<VEC>(yp + (int64_t)s * p.rows * p.width, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) y[k][j] += t[j];
      }
    } else {
      Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.y) + row * p.y_stride + c, y[k]);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += y[k][j] * y[k][j];
  }
  const float inv = inv_rms(wg_sum(ss, smem), p.width, p.eps);
  ss = 0.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= p.width) continue;
    float w[VEC];
    Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.w_post) + c, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      x[k][j] += y[k][j] * inv * w[j];
      ss += x[k][j] * x[k][j];
    }
    Io<float>::stv<VEC>(xr + c, x[k]);
  }
  if (p.h == nullptr) return;
  const bool pre = p.w_pre != nullptr;
  const float inv2 = pre ? inv_rms(wg_sum(ss, smem), p.width, p.eps) : 1.f;
  T* hr = reinterpret_cast<T*>(p.h) + row * p.h_stride;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= p.width) continue;
    if (pre) {
      float w[VEC];
      Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.w_pre) + c, w);
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[k][j] *= inv2 * w[j];
    }
    Io<T>::template stv<VEC>(hr + c, x[k]);
  }
}

// a causal filter over the normed rows, one per channel: the last taps - 1 rows of a sequence live in its ring, row of
// position p in place p % (taps - 1)
struct ConvParams {
  const void* w;            // [taps][width], the last one for the row itself; nullptr: no filter
  void* ring;               // [slots][taps - 1][width]
  const int32_t* slots;     // per row (one-token rows) or per request (portions)
  const int64_t* positions;
  int taps;
};

// the one-token form: every row is its sequence's only new one.  h: the thread's normed values
template <typename T, int VEC>
__device__ __forceinline__ void conv_one_row(float (&h)[VEC], const ConvParams& cv, int64_t row, int c, int width) {
  const T* w = reinterpret_cast<const T*>(cv.w) + c;
  const int back = cv.taps - 1;
  float cur[VEC], t[VEC], wt[VEC];
#pragma unroll
  for (int j = 0; j < VEC; ++j) {
    T bits;
    Io<T>::st(&bits, h[j]);        // the filter reads rows of the storage type, like the portions' form
    cur[j] = Io<T>::ld(&bits);
  }
  Io<T>::template ldv<VEC>(w + (int64_t)back * width, wt);
#pragma unroll
  for (int j = 0; j < VEC; ++j) h[j] = cur[j] + wt[j] * cur[j];
  if (back == 0) return;
  const int64_t pos = cv.positions[row];
  T* ring = reinterpret_cast<T*>(cv.ring) + (int64_t)cv.slots[row] * back * width + c;
  for (int b = 1; b <= back && b <= pos; ++b) {
    Io<T>::template ldv<VEC>(ring + (pos - b) % back * width, t);
    Io<T>::template ldv<VEC>(w + (int64_t)(back - b) * width, wt);
#pragma unroll
    for (int j = 0; j < VEC; ++j) h[j] += wt[j] * t[j];
  }
  Io<T>::template stv<VEC>(ring + pos % back * width, cur);     // the place of the row taps - 1 back, read above
}

// h = norm(x) w, norm(x) (1 + w) or x itself, of a row whose sum of squares over the thread's values is ss; then the
// one-token filter over it if there is one
template <typename T, int VEC, int MAXC, bool CONV = false>
__device__ __forceinline__ void store_normed(float (&x)[MAXC][VEC], float ss, const void* w_pre, float w_shift, void* h, int width,
                                             float eps, float* smem, const ConvParams* cv = nullptr, int64_t row = 0) {
  const bool pre = w_pre != nullptr;
  const float inv = pre ? inv_rms(wg_sum(ss, smem), width, eps) : 1.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= width) continue;
    if (pre) {
      float w[VEC];
      Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(w_pre) + c, w);
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[k][j] *= inv * (w[j] + w_shift);
    }
    if constexpr (CONV) {
      if (cv->w) conv_one_row<T, VEC>(x[k], *cv, row, c, width);
    }
    Io<T>::template stv<VEC>(reinterpret_cast<T*>(h) + c, x[k]);
  }
}

struct ResidualAddParams {
  float* x;
  const void* y;                // T rows, fp32 rows, or fp32 split-K partials [split][rows][width]
  const void* part;             // routed experts' output rows, T; nullptr: none
  const int32_t* row_of_pair;   // [rows][top] -> row of `part`; nullptr: pair t * top + j is its row t * top + j
  const float* weights;         // [rows][top]
  const void* w_pre;            // nullptr: h = x cast
  void* h;
  int64_t x_stride, y_stride, h_stride, part_stride;
  int rows, width, split, top, start;      // start: x is not read, the sum starts the stream
  float w_shift, eps;
  const void* add_row;          // EXT: [width] added to every row; nullptr: none
  ConvParams conv;              // EXT
};

template <typename T, int VEC, int MAXC, bool EXT>
__device__ __forceinline__ void residual_add_norm_row(const ResidualAddParams& p) {
  __shared__ float smem[16];
  const int64_t row = blockIdx.x;
  float* xr = p.x + row * p.x_stride;
  float x[MAXC][VEC];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= p.width) continue;
    float t[VEC];
    if (p.start) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[k][j] = 0.f;
    } else {
      Io<float>::ldv<VEC>(xr + c, x[k]);
    }
    if (p.split) {
      const float* yp = reinterpret_cast<const float*>(p.y) + row * p.y_stride + c;
      for (int s = 0; s < p.split; ++s) {
        Io<float>::ldv<VEC>(yp + (int64_t)s * p.rows * p.y_stride, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) x[k][j] += t[j];
      }
    } else {
      Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.y) + row * p.y_stride + c, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[k][j] += t[j];
    }
    if (p.part) {
      float e[VEC] = {};
      for (int j0 = 0; j0 < p.top; ++j0) {
        const int64_t pair = row * p.top + j0;
        const int64_t pr = p.row_of_pair ? p.row_of_pair[pair] : pair;
        const float w = p.weights[pair];
        Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.part) + pr * p.part_stride + c, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) e[j] += w * t[j];
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[k][j] += e[j];
    }
    if constexpr (EXT) {
      if (p.add_row) {
        Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.add_row) + c, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) x[k][j] += t[j];
      }
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += x[k][j] * x[k][j];
    Io<float>::stv<VEC>(xr + c, x[k]);
  }
  store_normed<T, VEC, MAXC, EXT>(x, ss, p.w_pre, p.w_shift, reinterpret_cast<T*>(p.h) + row * p.h_stride, p.width, p.eps, smem,
                                  &p.conv, row);
}

template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void residual_add_norm_kernel(const ResidualAddParams p) {
  scalar_cache_acquire();
  residual_add_norm_row<T, VEC, MAXC, false>(p);
}
template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void residual_add_norm_conv_kernel(const ResidualAddParams p) {
  scalar_cache_acquire();
  residual_add_norm_row<T, VEC, MAXC, true>(p);
}

// The filter over prompt portions (and one-token rows among them): a workgroup takes kConvRows rows of a request, a thread
// VEC channels of them.  The threads of a request's first rows are the ones that read its ring, and they alone write it
// when they are done: the places of a portion's last rows may be those its first rows read.
struct InputConvParams {
  const void* h;
  void* out;
  ConvParams conv;              // slots per request
  const int32_t* qsl;
  const int32_t* seq_lens;
  int64_t h_stride, out_stride;
  int req0, width;
};

constexpr int kConvRows = 16;

template <typename T, int VEC>
__global__ __launch_bounds__(256) void input_conv_kernel(const InputConvParams p) {
  scalar_cache_acquire();
  const int r = p.req0 + blockIdx.y, c = (blockIdx.z * 256 + threadIdx.x) * VEC;
  const int s0 = p.qsl[r], n = p.qsl[r + 1] - s0, t0 = blockIdx.x * kConvRows;
  if (t0 >= n || c >= p.width) return;
  const int first = p.seq_lens[r] - n;            // position of the portion's first row
  if (first < 0) return;
  const int back = p.conv.taps - 1;
  const T* w = reinterpret_cast<const T*>(p.conv.w) + c;
  const T* h = reinterpret_cast<const T*>(p.h) + (int64_t)s0 * p.h_stride + c;
  T* out = reinterpret_cast<T*>(p.out) + (int64_t)s0 * p.out_stride + c;
  T* ring = reinterpret_cast<T*>(p.conv.ring) + (int64_t)p.conv.slots[r] * back * p.width + c;
  constexpr int kHeld = 3;                        // filters up to four taps keep rows and weights in registers
  float prev[kHeld][VEC], wt[kHeld + 1][VEC], v[VEC], t[VEC], u[VEC];
  auto load = [&](int i, float (&d)[VEC]) {       // row i of the portion (negative: before it)
    if (i >= 0) {
      Io<T>::template ldv<VEC>(h + (int64_t)i * p.h_stride, d);
    } else if (first + i >= 0) {
      Io<T>::template ldv<VEC>(ring + (int64_t)((first + i) % back) * p.width, d);
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) d[j] = 0.f;
    }
  };
  const int end = min(n, t0 + kConvRows);
  if (back <= kHeld) {
#pragma unroll
    for (int b = 0; b <= kHeld; ++b) {
      if (b <= back) Io<T>::template ldv<VEC>(w + (int64_t)(back - b) * p.width, wt[b]);
      if (b >= 1 && b <= back) load(t0 - b, prev[b - 1]);
    }
    for (int i = t0; i < end; ++i) {
      Io<T>::template ldv<VEC>(h + (int64_t)i * p.h_stride, v);
#pragma unroll
      for (int j = 0; j < VEC; ++j) u[j] = v[j] + wt[0][j] * v[j];
#pragma unroll
      for (int b = 1; b <= kHeld; ++b)
        if (b <= back) {
#pragma unroll
          for (int j = 0; j < VEC; ++j) u[j] += wt[b][j] * prev[b - 1][j];
        }
#pragma unroll
      for (int b = kHeld - 1; b > 0; --b)
#pragma unroll
        for (int j = 0; j < VEC; ++j) prev[b][j] = prev[b - 1][j];
#pragma unroll
      for (int j = 0; j < VEC; ++j) prev[0][j] = v[j];
      Io<T>::template stv<VEC>(out + (int64_t)i * p.out_stride, u);
    }
  } else {
    for (int i = t0; i < end; ++i) {
#pragma unroll
      for (int j = 0; j < VEC; ++j) u[j] = 0.f;
      for (int b = 0; b <= back; ++b) {
        load(i - b, t);
        Io<T>::template ldv<VEC>(w + (int64_t)(back - b) * p.width, v);
#pragma unroll
        for (int j = 0; j < VEC; ++j) u[j] += (b == 0 ? 1.f + v[j] : v[j]) * t[j];
      }
      Io<T>::template stv<VEC>(out + (int64_t)i * p.out_stride, u);
    }
  }
  if (t0 != 0) return;      // (taps - 1 <= kConvRows, checked on the host: later workgroups read no ring)
  for (int i = max(0, n - back); i < n; ++i) {
    Io<T>::template ldv<VEC>(h + (int64_t)i * p.h_stride, v);
    Io<T>::template stv<VEC>(ring + (int64_t)((first + i) % back) * p.width, v);
  }
}

struct EmbedNormParams {
  float* x;
  void* h;
  void* copy;              // nullptr: none; the row in the table's type (a loop's second input)
  const void* table;
  const void* w_pre;       // nullptr: h = x cast
  const int64_t* ids;
  int64_t x_stride, h_stride, copy_stride;
  int width, vocab;
  float w_shift, eps;
  // POS: x = scale * table[id] + pos_table[position] + add_row
  const void* pos_table;   // nullptr: none
  const int64_t* positions;
  const void* add_row;     // nullptr: none
  int max_positions;
  float scale;
  ConvParams conv;
};

template <typename T, int VEC, int MAXC, bool POS>
__device__ __forceinline__ void embed_norm_row(const EmbedNormParams& p) {
  __shared__ float smem[16];
  const int64_t row = blockIdx.x;
  const int64_t id = p.ids[row];
  const bool known = id >= 0 && id < p.vocab;   // an id outside the table reads as a zero row
  const T* er = reinterpret_cast<const T*>(p.table) + (known ? id : 0) * p.width;
  float x[MAXC][VEC];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= p.width) continue;
    Io<T>::template ldv<VEC>(er + c, x[k]);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      x[k][j] = known ? x[k][j] : 0.f;
      if constexpr (POS) x[k][j] *= p.scale;
      else ss += x[k][j] * x[k][j];
    }
    if constexpr (POS) {
      float t[VEC];
      if (p.pos_table) {
        const int64_t at = p.positions[row];
        if (at >= 0 && at < p.max_positions) {      // a position outside the table reads as a zero row
          Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.pos_table) + at * p.width + c, t);
#pragma unroll
          for (int j = 0; j < VEC; ++j) x[k][j] += t[j];
        }
      }
      if (p.add_row) {
        Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.add_row) + c, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) x[k][j] += t[j];
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss += x[k][j] * x[k][j];
    }
    Io<float>::stv<VEC>(p.x + row * p.x_stride + c, x[k]);
    if (p.copy) Io<T>::template stv<VEC>(reinterpret_cast<T*>(p.copy) + row * p.copy_stride + c, x[k]);
  }
  store_normed<T, VEC, MAXC, POS>(x, ss, p.w_pre, p.w_shift, reinterpret_cast<T*>(p.h) + row * p.h_stride, p.width, p.eps, smem,
                                  &p.conv, row);
}

template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void embed_norm_kernel(const EmbedNormParams p) {
  scalar_cache_acquire();
  embed_norm_row<T, VEC, MAXC, false>(p);
}
template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void embed_pos_norm_kernel(const EmbedNormParams p) {
  scalar_cache_acquire();
  embed_norm_row<T, VEC, MAXC, true>(p);
}

struct StreamParams {
  float* x;
  const void* y;                // T rows, or fp32 slabs [split][rows][y_stride]; nullptr: x = table[id]
  const void* part;             // routed experts' output rows, T; nullptr: none
  const int32_t* row_of_pair;   // nullptr: pair t * top + j is its row t * top + j
  const float* weights;         // [rows][top]; nullptr: 1
  const void* table;            // nullptr: none; with y: table[id] is added once more
  const int64_t* ids;
  const void* add_row;          // [width] added to every row; nullptr: none
  const void* w1;
  const void* w2;               // nullptr: one norm only
  void* h1;
  void* h2;
  int64_t x_stride, y_stride, part_stride, h1_stride, h2_stride;
  int rows, width, split, top, vocab;
  float mult, w_shift, eps;
};

template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void stream_norm2_kernel(const StreamParams p) {
  scalar_cache_acquire();
  __shared__ float smem[16];
  const int64_t row = blockIdx.x;
  const int64_t id = p.table ? p.ids[row] : 0;
  const bool known = id >= 0 && id < p.vocab;   // an id outside the table reads as a zero row
  const T* er = reinterpret_cast<const T*>(p.table) + (known ? id : 0) * p.width;
  float* xr = p.x + row * p.x_stride;
  float x[MAXC][VEC] = {};
  // slabs and experts' rows four at a time: their loads are on their way together (past the last one: it again, times zero)
  if (p.split) {
    const float* yp = reinterpret_cast<const float*>(p.y) + row * p.y_stride;
    for (int s0 = 0; s0 < p.split; s0 += 4)
#pragma unroll
      for (int k = 0; k < MAXC; ++k) {
        const int c = (threadIdx.x + k * 256) * VEC;
        if (c >= p.width) continue;
        float t[4][VEC];
#pragma unroll
        for (int u = 0; u < 4; ++u) Io<float>::ldv<VEC>(yp + c + (int64_t)min(s0 + u, p.split - 1) * p.rows * p.y_stride, t[u]);
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
          for (int j = 0; j < VEC; ++j) x[k][j] += s0 + u < p.split ? t[u][j] : 0.f;
      }
  } else if (p.y) {
#pragma unroll
    for (int k = 0; k < MAXC; ++k) {
      const int c = (threadIdx.x + k * 256) * VEC;
      if (c < p.width) Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.y) + row * p.y_stride + c, x[k]);
    }
  }
  for (int j0 = 0; j0 < p.top; j0 += 4) {
    const T* src[4];
    float w[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int64_t pair = row * p.top + min(j0 + u, p.top - 1);
      src[u] = reinterpret_cast<const T*>(p.part) + (p.row_of_pair ? p.row_of_pair[pair] : pair) * p.part_stride;
      w[u] = j0 + u >= p.top ? 0.f : p.weights ? p.weights[pair] : 1.f;
    }
#pragma unroll
    for (int k = 0; k < MAXC; ++k) {
      const int c = (threadIdx.x + k * 256) * VEC;
      if (c >= p.width) continue;
      float t[4][VEC];
#pragma unroll
      for (int u = 0; u < 4; ++u) Io<T>::template ldv<VEC>(src[u] + c, t[u]);
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int j = 0; j < VEC; ++j) x[k][j] += w[u] != 0.f ? w[u] * t[u][j] : 0.f;
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= p.width) continue;
    float t[VEC];
    if (p.y) {
      Io<float>::ldv<VEC>(xr + c, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[k][j] = t[j] + p.mult * x[k][j];
    }
    if (p.table) {
      Io<T>::template ldv<VEC>(er + c, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[k][j] += known ? t[j] : 0.f;
    }
    if (p.add_row) {
      Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.add_row) + c, t);
#pragma unroll
      for (int j = 0; j < VEC; ++j) x[k][j] += t[j];
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss += x[k][j] * x[k][j];
    Io<float>::stv<VEC>(xr + c, x[k]);
  }
  const float inv = inv_rms(wg_sum(ss, smem), p.width, p.eps);
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= p.width) continue;
    float w[VEC], v[VEC];
    Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.w1) + c, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) v[j] = x[k][j] * inv * (w[j] + p.w_shift);
    Io<T>::template stv<VEC>(reinterpret_cast<T*>(p.h1) + row * p.h1_stride + c, v);
    if (p.w2) {
      Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.w2) + c, w);
#pragma unroll
      for (int j = 0; j < VEC; ++j) v[j] = x[k][j] * inv * (w[j] + p.w_shift);
      Io<T>::template stv<VEC>(reinterpret_cast<T*>(p.h2) + row * p.h2_stride + c, v);
    }
  }
}

struct PairEmbedParams {
  float* x;
  void* h;
  const void* table;       // [vocab, width]
  const void* pairs;       // [buckets + 1, width]
  const void* w_pre;
  const int64_t* ids;
  const int64_t* prev_ids;   // nullptr: every row takes the previous token from last_token[slot]
  const int32_t* slots;      // per row: slot whose last_token this row leaves behind (< 0: none)
  int64_t* last_token;
  const int64_t* positions;
  int64_t x_stride, h_stride, mul_prev, mul_cur, buckets;
  int width, vocab;
  float scale, eps;
};

template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void pair_embed_norm_kernel(const PairEmbedParams p) {
  scalar_cache_acquire();
  __shared__ float smem[16];
  __shared__ int64_t s_prev;
  const int64_t row = blockIdx.x;
  const int64_t id = p.ids[row];
  const int slot = p.slots[row];
  if (threadIdx.x == 0) {
    int64_t prev = p.prev_ids ? p.prev_ids[row] : -1;
    if (prev < 0 && slot >= 0) prev = p.last_token[slot];
    if (slot >= 0) p.last_token[slot] = id;
    s_prev = prev < 0 ? 0 : prev;
  }
  __syncthreads();
  const bool known = id >= 0 && id < p.vocab;   // an id outside the table reads as a zero row
  const int64_t cur = known ? id : 0;
  const int64_t pr = p.positions[row] <= 0 ? p.buckets : (s_prev * p.mul_prev + cur * p.mul_cur) % p.buckets;
  const T* er = reinterpret_cast<const T*>(p.table) + cur * p.width;
  const T* br = reinterpret_cast<const T*>(p.pairs) + pr * p.width;
  float x[MAXC][VEC];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= p.width) continue;
    float b[VEC];
    Io<T>::template ldv<VEC>(er + c, x[k]);
    Io<T>::template ldv<VEC>(br + c, b);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      x[k][j] = known ? x[k][j] * p.scale + b[j] : 0.f;
      ss += x[k][j] * x[k][j];
    }
    Io<float>::stv<VEC>(p.x + row * p.x_stride + c, x[k]);
  }
  const float inv = inv_rms(wg_sum(ss, smem), p.width, p.eps);
  T* hr = reinterpret_cast<T*>(p.h) + row * p.h_stride;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * 256) * VEC;
    if (c >= p.width) continue;
    float w[VEC];
    Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(p.w_pre) + c, w);
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[k][j] *= inv * w[j];
    Io<T>::template stv<VEC>(hr + c, x[k]);
  }
}

__device__ __forceinline__ float gelu_tanh_f(float z) {
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void gelu_lookup_mul_kernel(T* out, const T* z, const T* table, const int64_t* ids, int rows,
                                                              int dim, int64_t z_stride, int64_t table_stride, int64_t offset,
                                                              int vocab) {
  scalar_cache_acquire();
  const int per = dim / VEC;
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= (int64_t)rows * per) return;
  const int64_t row = i / per;
  const int c = (int)(i % per) * VEC;
  const int64_t id = ids[row];
  float v[VEC], e[VEC];
  Io<T>::template ldv<VEC>(z + row * z_stride + c, v);
  const bool known = id >= 0 && id < vocab;
  Io<T>::template ldv<VEC>(table + (known ? id : 0) * table_stride + offset + c, e);
#pragma unroll
  for (int j = 0; j < VEC; ++j) v[j] = known ? gelu_tanh_f(v[j]) * e[j] : 0.f;
  Io<T>::template stv<VEC>(out + row * dim + c, v);
}

template <typename T, int VEC>
__global__ __launch_bounds__(256) void clamped_glu_kernel(T* out, const T* gu, int rows, int ff, int64_t gu_stride,
                                                          int64_t out_stride, float alpha, float limit) {
  scalar_cache_acquire();
  const int per = ff / VEC;
  const int64_t n = (int64_t)rows * per;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
    const int64_t row = i / per;
    const int c = (int)(i % per) * VEC;
    float g[VEC], u[VEC];
    Io<T>::template ldv<VEC>(gu + row * gu_stride + c, g);
    Io<T>::template ldv<VEC>(gu + row * gu_stride + ff + c, u);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      const float a = fminf(g[j], limit);
      g[j] = a * sigmoid_f(alpha * a) * (fminf(fmaxf(u[j], -limit), limit) + 1.0f);
    }
    Io<T>::template stv<VEC>(out + row * out_stride + c, g);
  }
}

template <typename T, int VEC, int ACT>
__global__ __launch_bounds__(256) void glu_kernel(T* out, const T* gate, const T* up, int rows, int ff, int64_t gu_stride,
                                                  int64_t out_stride) {
  scalar_cache_acquire();
  const int per = ff / VEC;
  const int64_t n = (int64_t)rows * per;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
    const int64_t row = i / per;
    const int c = (int)(i % per) * VEC;
    float g[VEC], u[VEC];
    Io<T>::template ldv<VEC>(gate + row * gu_stride + c, g);
    Io<T>::template ldv<VEC>(up + row * gu_stride + c, u);
#pragma unroll
    for (int j = 0; j < VEC; ++j) g[j] = (ACT == MI_ACT_SILU ? silu_f(g[j]) : gelu_tanh_f(g[j])) * u[j];
    Io<T>::template stv<VEC>(out + row * out_stride + c, g);
  }
}

// relu(z)^2 of T rows (split == 0) or of the sum of fp32 slabs [split][rows][z_stride]
template <typename T, int VEC>
__global__ __launch_bounds__(256) void relu_squared_kernel(T* out, const void* z, int split, int rows, int ff, int64_t z_stride,
                                                           int64_t out_stride) {
  scalar_cache_acquire();
  const int per = ff / VEC;
  const int64_t n = (int64_t)rows * per;
  for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) {
    const int64_t row = i / per;
    const int c = (int)(i % per) * VEC;
    float v[VEC], t[VEC];
    if (split) {
      const float* zp = reinterpret_cast<const float*>(z) + row * z_stride + c;
      Io<float>::ldv<VEC>(zp, v);
      for (int s = 1; s < split; ++s) {
        Io<float>::ldv<VEC>(zp + (int64_t)s * rows * z_stride, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) v[j] += t[j];
      }
    } else {
      Io<T>::template ldv<VEC>(reinterpret_cast<const T*>(z) + row * z_stride + c, v);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      const float a = fmaxf(v[j], 0.f);
      v[j] = a * a;
    }
    Io<T>::template stv<VEC>(out + row * out_stride + c, v);
  }
}

#define MI_ROW_DISPATCH(KERN, T, width, vec_ok, ...)                                         \
  do {                                                                                       \
    if (vec_ok) {                                                                            \
      if ((width) <= 2048) hipLaunchKernelGGL((KERN<T, 8, 1>), grid, block, 0, s, __VA_ARGS__);      \
      else if ((width) <= 4096) hipLaunchKernelGGL((KERN<T, 8, 2>), grid, block, 0, s, __VA_ARGS__); \
      else if ((width) <= 8192) hipLaunchKernelGGL((KERN<T, 8, 4>), grid, block, 0, s, __VA_ARGS__); \
      else if ((width) <= 16384) hipLaunchKernelGGL((KERN<T, 8, 8>), grid, block, 0, s, __VA_ARGS__); \
      else return MI_ERR_UNSUPPORTED;                                                        \
    } else {                                                                                 \
      if ((width) <= 1024) hipLaunchKernelGGL((KERN<T, 1, 4>), grid, block, 0, s, __VA_ARGS__);      \
      else if ((width) <= 8192) hipLaunchKernelGGL((KERN<T, 1, 32>), grid, block, 0, s, __VA_ARGS__); \
      else return MI_ERR_UNSUPPORTED;                                                        \
    }                                                                                        \
  } while (0)

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int mi_residual_norm(void* x, const void* y, int32_t split, const void* w_post, const void* w_pre, void* h, float eps,
                                int32_t rows, int32_t width, int64_t x_stride, int64_t y_stride, int64_t h_stride, int dtype,
                                void* stream) {
  if (rows == 0) return MI_OK;
  if (!x || !y || !w_post || rows < 0 || width <= 0 || split < 0) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  ResidualNormParams p{(float*)x, y, w_post, w_pre, h, x_stride, y_stride, h_stride, rows, width, split, eps};
  const bool vec = width % 8 == 0 && x_stride % 8 == 0 && (split || y_stride % 8 == 0) && (!h || h_stride % 8 == 0) &&
                   aligned16(x) && aligned16(y) && aligned16(w_post) && aligned16(w_pre) && aligned16(h);
  const dim3 grid(rows), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MI_DTYPE_BF16) MI_ROW_DISPATCH(residual_norm_kernel, uint16_t, width, vec, p);
  else MI_ROW_DISPATCH(residual_norm_kernel, float, width, vec, p);
  return launch_status();
}

extern "C" int mi_pair_embed_norm(void* x, void* h, const void* table, const void* pairs, const void* w_pre, const int64_t* ids,
                                  const int64_t* prev_ids, const int32_t* slots, int64_t* last_token, const int64_t* positions,
                                  float scale, int64_t mul_prev, int64_t mul_cur, int64_t buckets, float eps, int32_t rows,
                                  int32_t width, int32_t vocab, int64_t x_stride, int64_t h_stride, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!x || !h || !table || !pairs || !w_pre || !ids || !slots || !last_token || !positions) return MI_ERR_INVALID_ARG;
  if (rows < 0 || width <= 0 || vocab <= 0 || buckets <= 0 || mul_prev < 0 || mul_cur < 0) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  PairEmbedParams p{(float*)x, h, table, pairs, w_pre, ids, prev_ids, slots, last_token, positions, x_stride, h_stride,
                    mul_prev, mul_cur, buckets, width, vocab, scale, eps};
  const bool vec = width % 8 == 0 && x_stride % 8 == 0 && h_stride % 8 == 0 && aligned16(x) && aligned16(h) &&
                   aligned16(table) && aligned16(pairs) && aligned16(w_pre);
  const dim3 grid(rows), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MI_DTYPE_BF16) MI_ROW_DISPATCH(pair_embed_norm_kernel, uint16_t, width, vec, p);
  else MI_ROW_DISPATCH(pair_embed_norm_kernel, float, width, vec, p);
  return launch_status();
}

extern "C" int mi_gelu_lookup_mul(void* out, const void* z, const void* table, const int64_t* ids, int32_t rows, int32_t dim,
                                  int64_t z_stride, int64_t table_stride, int64_t offset, int32_t vocab, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!out || !z || !table || !ids || rows < 0 || dim <= 0 || vocab <= 0 || offset < 0) return MI_ERR_INVALID_ARG;
  const bool vec = dim % 8 == 0 && z_stride % 8 == 0 && table_stride % 8 == 0 && offset % 8 == 0 && aligned16(out) &&
                   aligned16(z) && aligned16(table);
  const int64_t n = (int64_t)rows * (vec ? dim / 8 : dim);
  const dim3 grid((unsigned)((n + 255) / 256)), block(256);
  hipStream_t s = (hipStream_t)stream;
#define MI_GL(T, V)                                                                                                     \
  hipLaunchKernelGGL((gelu_lookup_mul_kernel<T, V>), grid, block, 0, s, (T*)out, (const T*)z, (const T*)table, ids, rows, dim, \
                     z_stride, table_stride, offset, vocab)
  if (dtype == MI_DTYPE_BF16) { if (vec) MI_GL(uint16_t, 8); else MI_GL(uint16_t, 1); }
  else if (dtype == MI_DTYPE_F32) { if (vec) MI_GL(float, 8); else MI_GL(float, 1); }
  else return MI_ERR_UNSUPPORTED;
#undef MI_GL
  return launch_status();
}

extern "C" int mi_clamped_glu(void* out, const void* gate_up, int32_t rows, int32_t ff, int64_t gu_stride, int64_t out_stride,
                              float alpha, float limit, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!out || !gate_up || rows < 0 || ff <= 0) return MI_ERR_INVALID_ARG;
  const bool vec = ff % 8 == 0 && gu_stride % 8 == 0 && out_stride % 8 == 0 && aligned16(out) && aligned16(gate_up);
  const int64_t n = (int64_t)rows * (vec ? ff / 8 : ff);
  const int64_t want = (n + 255) / 256;
  const dim3 grid((unsigned)(want < 65536 ? want : 65536)), block(256);
  hipStream_t s = (hipStream_t)stream;
#define MI_CG(T, V) \
  hipLaunchKernelGGL((clamped_glu_kernel<T, V>), grid, block, 0, s, (T*)out, (const T*)gate_up, rows, ff, gu_stride, out_stride, alpha, limit)
  if (dtype == MI_DTYPE_BF16) { if (vec) MI_CG(uint16_t, 8); else MI_CG(uint16_t, 1); }
  else if (dtype == MI_DTYPE_F32) { if (vec) MI_CG(float, 8); else MI_CG(float, 1); }
  else return MI_ERR_UNSUPPORTED;
#undef MI_CG
  return launch_status();
}

extern "C" int mi_residual_add_norm(void* x, const void* y, int32_t split, const void* part, const int32_t* row_of_pair,
                                    const float* weights, int32_t top, const void* w_pre, float w_shift, void* h, int32_t start,
                                    float eps, int32_t rows, int32_t width, int64_t x_stride, int64_t y_stride, int64_t h_stride,
                                    int64_t part_stride, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!x || !y || !h || rows < 0 || width <= 0 || split < 0 || y_stride < width || h_stride < width || x_stride < width)
    return MI_ERR_INVALID_ARG;
  if (part && (!weights || top <= 0 || part_stride < width)) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  const ResidualAddParams p{(float*)x, y, part, row_of_pair, weights, w_pre, h, x_stride, y_stride, h_stride, part_stride,
                            rows, width, split, part ? top : 0, start, w_shift, eps, nullptr, {}};
  const bool vec = width % 8 == 0 && x_stride % 8 == 0 && y_stride % 8 == 0 && h_stride % 8 == 0 && (!part || part_stride % 8 == 0) &&
                   aligned16(x) && aligned16(y) && aligned16(w_pre) && aligned16(h) && aligned16(part);
  const dim3 grid(rows), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MI_DTYPE_BF16) MI_ROW_DISPATCH(residual_add_norm_kernel, uint16_t, width, vec, p);
  else MI_ROW_DISPATCH(residual_add_norm_kernel, float, width, vec, p);
  return launch_status();
}

extern "C" int mi_residual_add_norm_conv(void* x, const void* y, int32_t split, const void* add_row, const void* w_pre, float w_shift,
                                         void* h, const void* conv_w, void* ring, const int32_t* slots, const int64_t* positions,
                                         int32_t taps, float eps, int32_t rows, int32_t width, int64_t x_stride, int64_t y_stride,
                                         int64_t h_stride, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!x || !y || !h || rows < 0 || width <= 0 || split < 0 || y_stride < width || h_stride < width || x_stride < width)
    return MI_ERR_INVALID_ARG;
  if (conv_w && (taps < 1 || (taps > 1 && (!ring || !slots || !positions)))) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  ResidualAddParams p{(float*)x, y, nullptr, nullptr, nullptr, w_pre, h, x_stride, y_stride, h_stride, 0,
                      rows, width, split, 0, 0, w_shift, eps, add_row, {conv_w, ring, slots, positions, taps}};
  const bool vec = width % 8 == 0 && x_stride % 8 == 0 && y_stride % 8 == 0 && h_stride % 8 == 0 && aligned16(x) && aligned16(y) &&
                   aligned16(w_pre) && aligned16(h) && aligned16(add_row) && aligned16(conv_w) && aligned16(ring);
  const dim3 grid(rows), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MI_DTYPE_BF16) MI_ROW_DISPATCH(residual_add_norm_conv_kernel, uint16_t, width, vec, p);
  else MI_ROW_DISPATCH(residual_add_norm_conv_kernel, float, width, vec, p);
  return launch_status();
}

extern "C" int mi_input_conv(void* out, const void* h, const void* conv_w, void* ring, const int32_t* slots,
                             const int32_t* query_start_loc, const int32_t* seq_lens, int32_t req0, int32_t num_reqs,
                             int32_t max_query_len, int32_t taps, int32_t width, int64_t h_stride, int64_t out_stride, int dtype,
                             void* stream) {
  if (num_reqs == 0 || max_query_len == 0) return MI_OK;
  if (!out || !h || out == h || !conv_w || !query_start_loc || !seq_lens || req0 < 0 || num_reqs < 0 || max_query_len < 0 || taps < 1 ||
      width <= 0 || h_stride < width || out_stride < width || !slots || (taps > 1 && !ring))
    return MI_ERR_INVALID_ARG;
  if (taps - 1 > kConvRows || num_reqs > 65535) return MI_ERR_UNSUPPORTED;
  const InputConvParams p{h, out, {conv_w, ring, slots, nullptr, taps}, query_start_loc, seq_lens, h_stride, out_stride, req0, width};
  const bool vec = width % 8 == 0 && h_stride % 8 == 0 && out_stride % 8 == 0 && aligned16(out) && aligned16(h) && aligned16(conv_w) &&
                   aligned16(ring);
  const int per = 256 * (vec ? 8 : 1);
  const dim3 grid((max_query_len + kConvRows - 1) / kConvRows, num_reqs, (width + per - 1) / per), block(256);
  hipStream_t s = (hipStream_t)stream;
#define MI_IC(T, V) hipLaunchKernelGGL((input_conv_kernel<T, V>), grid, block, 0, s, p)
  if (dtype == MI_DTYPE_BF16) { if (vec) MI_IC(uint16_t, 8); else MI_IC(uint16_t, 1); }
  else if (dtype == MI_DTYPE_F32) { if (vec) MI_IC(float, 8); else MI_IC(float, 1); }
  else return MI_ERR_UNSUPPORTED;
#undef MI_IC
  return launch_status();
}

extern "C" int mi_relu_squared(void* out, const void* z, int32_t split, int32_t rows, int32_t ff, int64_t z_stride, int64_t out_stride,
                               int dtype, void* stream) {
  if (rows == 0 || ff == 0) return MI_OK;
  if (!out || !z || split < 0 || rows < 0 || ff < 0 || z_stride < ff || out_stride < ff) return MI_ERR_INVALID_ARG;
  const bool vec = ff % 8 == 0 && z_stride % 8 == 0 && out_stride % 8 == 0 && aligned16(out) && aligned16(z);
  const int64_t n = (int64_t)rows * (vec ? ff / 8 : ff);
  const int64_t want = (n + 255) / 256;
  const dim3 grid((unsigned)(want < 65536 ? want : 65536)), block(256);
  hipStream_t s = (hipStream_t)stream;
#define MI_RS(T, V) hipLaunchKernelGGL((relu_squared_kernel<T, V>), grid, block, 0, s, (T*)out, z, split, rows, ff, z_stride, out_stride)
  if (dtype == MI_DTYPE_BF16) { if (vec) MI_RS(uint16_t, 8); else MI_RS(uint16_t, 1); }
  else if (dtype == MI_DTYPE_F32) { if (vec) MI_RS(float, 8); else MI_RS(float, 1); }
  else return MI_ERR_UNSUPPORTED;
#undef MI_RS
  return launch_status();
}

extern "C" int mi_embed_pos_norm(void* x, void* h, const void* table, float scale, const void* pos_table, const int64_t* positions,
                                 int32_t max_positions, const void* add_row, const void* w_pre, float w_shift, const int64_t* ids,
                                 const void* conv_w, void* ring, const int32_t* slots, int32_t taps, float eps, int32_t rows, int32_t width, int32_t vocab, int64_t x_stride, int64_t h_stride, int dtype,
                                 void* stream) {
  if (rows == 0) return MI_OK;
  if (!x || !h || !table || !ids || rows < 0 || width <= 0 || vocab <= 0 || x_stride < width || h_stride < width)
    return MI_ERR_INVALID_ARG;
  if (pos_table && (!positions || max_positions <= 0)) return MI_ERR_INVALID_ARG;
  if (conv_w && (taps < 1 || (taps > 1 && (!ring || !slots || !positions)))) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  const EmbedNormParams p{(float*)x, h, nullptr, table, w_pre, ids, x_stride, h_stride, 0, width, vocab, w_shift, eps,
                          pos_table, positions, add_row, max_positions, scale, {conv_w, ring, slots, positions, taps}};
  const bool vec = width % 8 == 0 && x_stride % 8 == 0 && h_stride % 8 == 0 && aligned16(x) && aligned16(h) && aligned16(table) &&
                   aligned16(w_pre) && aligned16(pos_table) && aligned16(add_row) && aligned16(conv_w) && aligned16(ring);
  const dim3 grid(rows), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MI_DTYPE_BF16) MI_ROW_DISPATCH(embed_pos_norm_kernel, uint16_t, width, vec, p);
  else MI_ROW_DISPATCH(embed_pos_norm_kernel, float, width, vec, p);
  return launch_status();
}

extern "C" int mi_embed_norm(void* x, void* h, void* copy, const void* table, const void* w_pre, float w_shift, const int64_t* ids,
                             float eps, int32_t rows, int32_t width, int32_t vocab, int64_t x_stride, int64_t h_stride,
                             int64_t copy_stride, int dtype, void* stream) {
  if (rows == 0) return MI_OK;
  if (!x || !h || !table || !ids || rows < 0 || width <= 0 || vocab <= 0 || x_stride < width || h_stride < width)
    return MI_ERR_INVALID_ARG;
  if (copy && copy_stride < width) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  const EmbedNormParams p{(float*)x, h, copy, table, w_pre, ids, x_stride, h_stride, copy_stride, width, vocab, w_shift, eps,
                          nullptr, nullptr, nullptr, 0, 1.f, {}};
  const bool vec = width % 8 == 0 && x_stride % 8 == 0 && h_stride % 8 == 0 && (!copy || copy_stride % 8 == 0) && aligned16(x) &&
                   aligned16(h) && aligned16(copy) && aligned16(table) && aligned16(w_pre);
  const dim3 grid(rows), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MI_DTYPE_BF16) MI_ROW_DISPATCH(embed_norm_kernel, uint16_t, width, vec, p);
  else MI_ROW_DISPATCH(embed_norm_kernel, float, width, vec, p);
  return launch_status();
}

extern "C" int mi_stream_norm2(void* x, const void* y, int32_t split, const void* part, const int32_t* row_of_pair, const float* weights,
                               int32_t top, float mult, const void* table, const int64_t* ids, int32_t vocab, const void* add_row,
                               const void* w1, const void* w2, float w_shift, void* h1, void* h2, float eps, int32_t rows, int32_t width,
                               int64_t x_stride, int64_t y_stride, int64_t part_stride, int64_t h1_stride, int64_t h2_stride, int dtype,
                               void* stream) {
  if (rows == 0) return MI_OK;
  if (!x || !w1 || !h1 || rows < 0 || width <= 0 || split < 0 || x_stride < width || h1_stride < width) return MI_ERR_INVALID_ARG;
  if (!y && !table) return MI_ERR_INVALID_ARG;
  if ((y && y_stride < width) || (part && (!y || top <= 0 || part_stride < width)) || (table && (!ids || vocab <= 0)) ||
      (w2 && (!h2 || h2_stride < width)))
    return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  const StreamParams p{(float*)x, y, part, row_of_pair, weights, table, ids, add_row, w1, w2, h1, h2, x_stride, y_stride, part_stride,
                       h1_stride, h2_stride, rows, width, split, part ? top : 0, vocab, mult, w_shift, eps};
  const bool vec = width % 8 == 0 && x_stride % 8 == 0 && (!y || y_stride % 8 == 0) && (!part || part_stride % 8 == 0) &&
                   h1_stride % 8 == 0 && (!w2 || h2_stride % 8 == 0) && aligned16(x) && aligned16(y) && aligned16(part) &&
                   aligned16(table) && aligned16(add_row) && aligned16(w1) && aligned16(w2) && aligned16(h1) && aligned16(h2);
  const dim3 grid(rows), block(256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == MI_DTYPE_BF16) MI_ROW_DISPATCH(stream_norm2_kernel, uint16_t, width, vec, p);
  else MI_ROW_DISPATCH(stream_norm2_kernel, float, width, vec, p);
  return launch_status();
}

extern "C" int mi_glu(void* out, const void* gate, const void* up, int32_t rows, int32_t ff, int64_t gu_stride, int64_t out_stride,
                      int32_t act, int dtype, void* stream) {
  if (rows == 0 || ff == 0) return MI_OK;
  if (!out || !gate || !up || rows < 0 || ff < 0 || gu_stride < ff || out_stride < ff) return MI_ERR_INVALID_ARG;
  if (act != MI_ACT_SILU && act != MI_ACT_GELU_TANH) return MI_ERR_INVALID_ARG;
  const bool vec = ff % 8 == 0 && gu_stride % 8 == 0 && out_stride % 8 == 0 && aligned16(out) && aligned16(gate) && aligned16(up);
  const int64_t n = (int64_t)rows * (vec ? ff / 8 : ff);
  const int64_t want = (n + 255) / 256;
  const dim3 grid((unsigned)(want < 65536 ? want : 65536)), block(256);
  hipStream_t s = (hipStream_t)stream;
#define MI_GLU(T, V, A) \
  hipLaunchKernelGGL((glu_kernel<T, V, A>), grid, block, 0, s, (T*)out, (const T*)gate, (const T*)up, rows, ff, gu_stride, out_stride)
#define MI_GLU_A(T, V) \
  do { if (act == MI_ACT_SILU) MI_GLU(T, V, MI_ACT_SILU); else MI_GLU(T, V, MI_ACT_GELU_TANH); } while (0)
  if (dtype == MI_DTYPE_BF16) { if (vec) MI_GLU_A(uint16_t, 8); else MI_GLU_A(uint16_t, 1); }
  else if (dtype == MI_DTYPE_F32) { if (vec) MI_GLU_A(float, 8); else MI_GLU_A(float, 1); }
  else return MI_ERR_UNSUPPORTED;
#undef MI_GLU_A
#undef MI_GLU
  return launch_status();
}
