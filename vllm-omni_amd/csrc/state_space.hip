// State-space recurrence with one decay per head and token (the dual form of a gated linear attention): the mixer of a decoder
// layer.  Per row, x (H x V), B and C (G x N) pass a causal filter per channel and silu;  dt = softplus(raw + bias);  per head h
// of group g
//   S_t = a_t S_(t-1) + dt_t B_t x_t^T,   ln a_t = -exp(A_log) dt_t,     y_t = S_t^T C_t + D x_t        S: [N][V] fp32
// and the row's y, all heads side by side, is gated by silu(z) and RMS-normed in equal parts.  A request's state is S per head
// and a ring of the filter's last inputs; one whose first token is position 0 starts from zeros.
//   * state_step: a workgroup per (head, 64 columns of S, request), S in registers, token after token: decode (HBM bound: S is
//     read and written once), 32-bit models and sizes the chunked form is not built for;
//   * prompt portions, 64 tokens (a chunk) at a time on the bf16 matrix cores: prep (filters; step sizes and sums of log decays),
//     then the chain of chunks, each wave with 16 columns of a head's S in registers:
//       Y = e^(G_i) C S0 + P X,   P_ij = e^(G_i - G_j) dt_j C_i . B_j (j < i; D more on the diagonal),
//       S1 = e^(G_C) S0 + sum_j e^(G_C - G_j) dt_j B_j x_j^T
//     x, B and C are bf16 (the filters' outputs); every fp32 operand (S0, P, the weighted x) enters as three bf16 terms, which
//     hold all 24 bits of it, so that the products are 32-bit products at a fifth of the fp32 matrix cores' time.  Few heads and
//     requests: a request's chunks in segments side by side, their end states first;
//   * finish: gate and norm, a workgroup per (token, part).
#include "mfma_attn_common.h"
#include "short_conv.h"

namespace mi {
namespace {

struct SsmParams {
  ConvInputs in;            // x | B | C
  const void* conv_b;
  const void* dt;           // [rows][ld of in]: H
  const float* dt_bias;
  const float* a_log;
  const float* d;
  float* state;             // [slots][H][N][V]
  float* y;                 // read-outs [rows of the requests][H V]
  int row0, H, G, N, V;
};

constexpr int kCols = 64;       // columns of S a step workgroup holds
constexpr int kC = 64;          // tokens per chunk
constexpr int kMaxSegments = 8;

// ------------------------------------------------------------------------------------------------ token by token
// thread: VEC columns x R rows of S; the filters' outputs of a token are staged for everybody.  Everything a token needs is asked
// for before the first use, S with it; loads are unconditional on clamped addresses.
template <typename T, int VEC, int R, int TAPS>
__global__ __launch_bounds__(256) void state_step_kernel(const SsmParams p) {
  scalar_cache_acquire();
  constexpr int LV = kCols / VEC, GR = 256 / LV;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int N = p.N, V = p.V, per = p.H / p.G;
  float* sx = lds;                 // [kCols]
  float* sb = sx + kCols;          // [N]
  float* sc = sb + N;              // [N]
  float* red = sc + N;             // [GR][kCols]
  const int h = blockIdx.x, r = p.in.req0 + blockIdx.z, c0 = blockIdx.y * kCols, grp = h / per;
  const int s0 = p.in.qsl[r], L = p.in.qsl[r + 1] - s0, start = p.in.seq_lens[r] - L;   // start < 0: a padded row of a graph replay
  if (L <= 0) return;
  const int tid = threadIdx.x, g = tid / LV, c = c0 + (tid % LV) * VEC;
  const int64_t slot = p.in.slots[r];
  float* S = p.state + (slot * p.H + h) * N * (int64_t)V;
  T* ring = reinterpret_cast<T*>(p.in.ring) + slot * p.in.taps * (int64_t)p.in.channels;
  const T* w = reinterpret_cast<const T*>(p.in.w);
  const bool cols = c < V;         // VEC divides V
  float st[R][VEC];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const float* src = S + (int64_t)min(g + i * GR, N - 1) * V + (cols ? c : 0);
    if constexpr (VEC == 4) {
      const f32x4_t a = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t*>(src));
      st[i][0] = a[0], st[i][1] = a[1], st[i][2] = a[2], st[i][3] = a[3];
    } else {
      st[i][0] = *src;
    }
  }
  const float rate = -expf(p.a_log[h]), bias = p.dt_bias[h], skip = p.d[h];
  const int nx = min(kCols, V - c0), nch = nx + 2 * N, inner = p.H * V, taps = TAPS ? TAPS : p.in.taps;
  const bool first_of_group = h % per == 0 && blockIdx.y == 0;
  for (int i = 0; i < L; ++i) {
    const int64_t row = s0 + i;
    const int pos = start + i;
    const T* x = reinterpret_cast<const T*>(p.in.x) + row * p.in.ld;
    const float raw = Io<T>::ld(reinterpret_cast<const T*>(p.dt) + row * p.in.ld + h);
    for (int n0 = 0; n0 < nch; n0 += 256) {
      const int n = min(n0 + tid, nch - 1), m = n - nx;
      const int ch = m < 0 ? h * V + c0 + n : m < N ? inner + grp * N + m : inner + (p.G + grp) * N + m - N;
      const T cur = x[ch];
      float acc = Io<T>::ld(reinterpret_cast<const T*>(p.conv_b) + ch);
      if constexpr (TAPS > 0) {
        float v[TAPS], wt[TAPS];
        v[0] = Io<T>::ld(&cur);
#pragma unroll
        for (int b = 1; b < TAPS; ++b) v[b] = Io<T>::ld(conv_input(p.in, x, (const T*)ring, i, pos, b) + ch);
#pragma unroll
        for (int b = 0; b < TAPS; ++b) wt[b] = Io<T>::ld(w + (int64_t)ch * TAPS + TAPS - 1 - b);
#pragma unroll
        for (int b = 0; b < TAPS; ++b) acc += (b == 0 || pos >= b ? v[b] : 0.f) * wt[b];
      } else {
        acc += Io<T>::ld(&cur) * Io<T>::ld(w + (int64_t)ch * taps + taps - 1);
        for (int b = 1; b < taps && b <= pos; ++b)
          acc += Io<T>::ld(conv_input(p.in, x, (const T*)ring, i, pos, b) + ch) * Io<T>::ld(w + (int64_t)ch * taps + taps - 1 - b);
      }
      if (n0 + tid < nch) {
        T out;                      // the filters leave the storage type, here as in the chunked form
        Io<T>::st(&out, silu_f(acc));
        (m < 0 ? sx[n] : sb[m]) = Io<T>::ld(&out);      // sc follows sb
        // one token: its row of the ring is nobody's to read this step
        if (L == 1 && pos >= 0 && (m < 0 || first_of_group)) ring[(int64_t)(pos % p.in.taps) * p.in.channels + ch] = cur;
      }
    }
    if (i == 0) {
#pragma unroll
      for (int n = 0; n < R; ++n)
#pragma unroll
        for (int j = 0; j < VEC; ++j) st[n][j] = start > 0 && g + n * GR < N ? st[n][j] : 0.f;
    }
    const float dt = softplus_f(raw + bias), keep = expf(rate * dt);
    __syncthreads();
    float xv[VEC], acc[VEC] = {};
#pragma unroll
    for (int j = 0; j < VEC; ++j) xv[j] = cols ? sx[c - c0 + j] * dt : 0.f;
#pragma unroll
    for (int n = 0; n < R; ++n) {
      const int d = min(g + n * GR, N - 1);
      const bool in = g + n * GR < N;
      const float bb = in ? sb[d] : 0.f, cc = in ? sc[d] : 0.f;
#pragma unroll
      for (int j = 0; j < VEC; ++j) st[n][j] = st[n][j] * keep + bb * xv[j], acc[j] += st[n][j] * cc;
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) red[g * kCols + (tid % LV) * VEC + j] = acc[j];
    const float own = tid < nx ? sx[tid] : 0.f;
    __syncthreads();      // (also: every reader of sx, sb, sc is done)
    if (tid < nx) {
      float t = 0.f;
#pragma unroll
      for (int n = 0; n < GR; ++n) t += red[n * kCols + tid];
      p.y[(row - p.row0) * inner + (int64_t)h * V + c0 + tid] = t + skip * own;
    }
  }
  if (!cols) return;
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int d = g + i * GR;
    if (d >= N) continue;
    if constexpr (VEC == 4) {
      const f32x4_t a = {st[i][0], st[i][1], st[i][2], st[i][3]};
      __builtin_nontemporal_store(a, reinterpret_cast<f32x4_t*>(S + (int64_t)d * V + c));
    } else {
      S[(int64_t)d * V + c] = st[i][0];
    }
  }
}

// ------------------------------------------------------------------------------------------------ chunks
// Workspace of one chunk (bf16): C [G][64][Np], B [G][64][Np], Bt [G][Np][64], Xt [H][Vp][64], then fp32 [H][5][64] (ChunkVec below).
// Rows past the portion's end are zeros.  A matrix lies in fragments of 16 rows x 32 columns as the matrix cores take them, a lane's
// eight values after the other's: one contiguous KB a load (a lane per row would be 64 cache accesses).  Lane 16 q + row, value 4 t +
// r holds column 16 t + 4 q + r: the order of an accumulator pair, which so IS an operand.
struct SsmLayout {
  int G, H, Np, Vp;
  __host__ __device__ int64_t c() const { return 0; }
  __host__ __device__ int64_t b() const { return (int64_t)G * kC * Np; }
  __host__ __device__ int64_t bt() const { return 2 * (int64_t)G * kC * Np; }
  __host__ __device__ int64_t xt() const { return 3 * (int64_t)G * kC * Np; }
  __host__ __device__ int64_t vec() const { return xt() + (int64_t)H * Vp * kC; }                    // (in bf16 units)
  __host__ __device__ int64_t size() const { return vec() + (int64_t)H * 5 * kC * 2; }
};

// numbers of a token of a chunk, per head.  ln a summed over the token's own 16 tokens up to it is `lead`; no sum that runs over more
// is ever taken off another, so that decays of any strength may stand beside each other.
enum ChunkVec {
  kDt,       // dt
  kTail,     // dt e^(ln a summed over the rest of its 16 tokens)
  kLead,
  kFrom0,    // e^(ln a summed from the chunk's start up to it)
  kToEnd,    // dt e^(ln a summed from behind it to the chunk's end)
};

struct SsmChunks {
  uint16_t* ws;
  float* y;              // read-outs [chunks][64][H][Vp]
  float* seg_state;      // [requests][nseg][H][N][V]: end state of each segment but the last; the last place: what the request started from
  float* seg_log;        // [requests][nseg][H]: ln of a segment's decay
  SsmLayout lay;
  int nseg, seg_chunks;
  int vec;               // the step's rows may be read 16 bytes at a time
};

template <typename P>
__device__ __forceinline__ int64_t chunk_base(const P& p, int r) {
  return (p.qsl[r] - p.qsl[p.req0]) / kC + (r - p.req0);
}

constexpr int kPrepCh = 64;     // channels of a prep workgroup: two waves, a thread has 8 channels of four neighbouring tokens

// blockIdx.y: first the filters' (kind, head or group, 64 channels) blocks, then two heads' token numbers each
__global__ __launch_bounds__(128) void ssm_prep_kernel(const SsmParams p, const SsmChunks k) {
  scalar_cache_acquire();
  // fragments [token tile][channel half] of the rows, then [channel tile][token half] of the columns, in units of 16 bytes
  __shared__ uint4 frag[2][8 * 64];
  using E = Elem<bf16_tag>;
  const int r = p.in.req0 + blockIdx.z, ck = blockIdx.x, tid = threadIdx.x;
  const int s0 = p.in.qsl[r], L = p.in.qsl[r + 1] - s0, i0 = ck * kC;
  if (i0 >= L) return;
  const int start = p.in.seq_lens[r] - L, len = min(kC, L - i0);
  uint16_t* ws = k.ws + (chunk_base(p.in, r) + ck) * k.lay.size();
  const int Np = k.lay.Np, Vp = k.lay.Vp;
  const int bx = (Vp + kPrepCh - 1) / kPrepCh, bn = (Np + kPrepCh - 1) / kPrepCh;
  int y = blockIdx.y;
  if (y >= p.H * bx + 2 * p.G * bn) {                       // a wave per head, a lane per token
    const int h = (y - p.H * bx - 2 * p.G * bn) * 2 + (tid >> 6), lane = tid & 63;
    if (h >= p.H) return;
    float* out = reinterpret_cast<float*>(ws + k.lay.vec()) + (int64_t)h * 5 * kC + lane;
    const int64_t row = s0 + i0 + min(lane, len - 1);
    const float raw = E::from_bits(reinterpret_cast<const uint16_t*>(p.dt)[row * p.in.ld + h]);
    const float dt = lane < len ? softplus_f(raw + p.dt_bias[h]) : 0.f, lg = -expf(p.a_log[h]) * dt;
    float lead = lg, tail = lg;       // sums over the token's 16 up to it, and from it on
#pragma unroll
    for (int o = 1; o < 16; o <<= 1) {
      const float a = __shfl_up(lead, o, 64), b = __shfl_down(tail, o, 64);
      lead += (lane & 15) >= o ? a : 0.f;
      tail += (lane & 15) + o < 16 ? b : 0.f;
    }
    const float next = __shfl_down(tail, 1, 64);
    const float t0 = __shfl(lead, 15, 64), t1 = __shfl(lead, 31, 64), t2 = __shfl(lead, 47, 64), t3 = __shfl(lead, 63, 64);
    const int t = lane >> 4;
    const float behind = (lane & 15) == 15 ? 0.f : next;
    const float before = t == 0 ? 0.f : t == 1 ? t0 : t == 2 ? t0 + t1 : t0 + t1 + t2;
    const float after = t == 3 ? 0.f : t == 2 ? t3 : t == 1 ? t2 + t3 : t1 + t2 + t3;
    out[kDt * kC] = dt;
    out[kTail * kC] = dt * expf(behind);
    out[kLead * kC] = lead;
    out[kFrom0 * kC] = expf(before + lead);
    out[kToEnd * kC] = dt * expf(behind + after);
    return;
  }
  int unit, blk, kind, width, real, ch0;
  if (y < p.H * bx) {
    kind = 0, unit = y / bx, blk = y % bx, width = Vp, real = p.V, ch0 = unit * p.V;
  } else {
    y -= p.H * bx;
    kind = 1 + y / (p.G * bn), y %= p.G * bn;
    unit = y / bn, blk = y % bn, width = Np, real = p.N, ch0 = p.H * p.V + ((kind - 1) * p.G + unit) * p.N;
  }
  const int c = blk * kPrepCh + (tid & 7) * 8, t = (tid >> 3) * 4;
  const int taps = p.in.taps, CH = p.in.channels;
  const uint16_t* X = reinterpret_cast<const uint16_t*>(p.in.x);
  const uint16_t* W = reinterpret_cast<const uint16_t*>(p.in.w);
  const uint16_t* ring = reinterpret_cast<const uint16_t*>(p.in.ring) + (int64_t)p.in.slots[r] * taps * CH;
  const int live = min(8, real - c);                        // <= 0: padding channels only
  float acc[4][8];
  auto source = [&](int i) {                                // token i of the portion (negative: before it)
    return (i >= 0 ? X + (int64_t)(s0 + min(i, L - 1)) * p.in.ld : ring + (int64_t)(max(start + i, 0) % taps) * CH) + ch0 + c;
  };
  if (live > 0) {
    if (k.vec && taps == 4) {
      uint4 raw[7];
      float wt[4][8], bias[8], v[8];
#pragma unroll
      for (int b = 0; b < 7; ++b) raw[b] = *reinterpret_cast<const uint4*>(source(i0 + t + 3 - b));
      conv_taps4<uint16_t>(W + (int64_t)(ch0 + c) * 4, wt);
      Io<uint16_t>::ldv<8>(reinterpret_cast<const uint16_t*>(p.conv_b) + ch0 + c, bias);
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[u][j] = bias[j];
#pragma unroll
      for (int b = 0; b < 7; ++b) {                         // the input of token t + 3 - b: tap u - (3 - b) of token t + u
        Io<uint16_t>::ldv<8>(reinterpret_cast<const uint16_t*>(&raw[b]), v);
        const bool there = start + i0 + t + 3 - b >= 0;
#pragma unroll
        for (int u = 0; u < 4; ++u)
          if (u - (3 - b) >= 0 && u - (3 - b) < 4)
#pragma unroll
            for (int j = 0; j < 8; ++j) acc[u][j] += wt[u - (3 - b)][j] * (there ? v[j] : 0.f);
      }
    } else {
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[u][j] = Io<uint16_t>::ld(reinterpret_cast<const uint16_t*>(p.conv_b) + ch0 + c + min(j, live - 1));
      for (int b = 0; b < taps; ++b)
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const int i = i0 + t + u - b;
          if (start + i < 0) continue;
          const uint16_t* src = source(i);
#pragma unroll
          for (int j = 0; j < 8; ++j) {
            const int jj = min(j, live - 1);
            acc[u][j] += Io<uint16_t>::ld(W + (int64_t)(ch0 + c + jj) * taps + taps - 1 - b) * Io<uint16_t>::ld(src + jj);
          }
        }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[u][j] = j < live && t + u < len ? silu_f(acc[u][j]) : 0.f;
  } else {
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[u][j] = 0.f;
  }
  // units are spread over the banks: the low bits of a place take in the bits that the writing threads differ in
  auto place = [](int u) { return u ^ ((u >> 3) & 1) ^ (((u >> 5) & 1) << 1) ^ (((u >> 4) & 1) << 2); };
  const int a = tid & 7, q = tid >> 3;
  if (kind != 0) {                                          // rows: 8 neighbours fall into two pieces of 4
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int unit0 = ((t >> 4) * 2 + (a >> 2)) * 64 + 2 * (a & 1) * 16 + (t & 15) + u;
      uint2* d0 = reinterpret_cast<uint2*>(&frag[0][place(unit0)]) + ((a >> 1) & 1);
      uint2* d1 = reinterpret_cast<uint2*>(&frag[0][place(unit0 + 16)]) + ((a >> 1) & 1);
      *d0 = make_uint2(E::pack(acc[u][0], acc[u][1]), E::pack(acc[u][2], acc[u][3]));
      *d1 = make_uint2(E::pack(acc[u][4], acc[u][5]), E::pack(acc[u][6], acc[u][7]));
    }
  }
  if (kind != 2) {
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int u = ((a >> 1) * 2 + (q >> 3)) * 64 + (q & 3) * 16 + 8 * (a & 1) + j;
      *(reinterpret_cast<uint2*>(&frag[1][place(u)]) + ((q >> 2) & 1)) =
          make_uint2(E::pack(acc[0][j], acc[1][j]), E::pack(acc[2][j], acc[3][j]));
    }
  }
  __syncthreads();
  if (kind != 0) {
    uint4* dst = reinterpret_cast<uint4*>(ws + (kind == 1 ? k.lay.b() : k.lay.c()) + (int64_t)unit * kC * Np);
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      const int u = tid + 128 * m, f = u >> 6;              // fragment (token tile f / 2, half f % 2)
      if (blk * kPrepCh + 32 * (f & 1) < Np) dst[((f >> 1) * (Np / 32) + blk * 2 + (f & 1)) * 64 + (u & 63)] = frag[0][place(u)];
    }
  }
  if (kind != 2) {
    uint4* dst = reinterpret_cast<uint4*>(ws + (kind == 0 ? k.lay.xt() : k.lay.bt()) + ((int64_t)unit * width + blk * kPrepCh) * kC);
#pragma unroll
    for (int m = 0; m < 4; ++m) {
      const int u = tid + 128 * m;                          // fragment (channel tile f / 2, token half f % 2)
      if (blk * kPrepCh + 16 * (u >> 7) < width) dst[u] = frag[1][place(u)];
    }
  }
}

// an fp32 octet as three bf16 terms: hi + mid + lo holds its 24 bits
struct Terms {
  uint4 hi, mid, lo;
};
// (cut off, not rounded: 8 + 8 + 8 bits, and a pair of upper halves is one instruction)
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& mid, uint32_t& lo) {
  auto bits = [](float x) { return __builtin_bit_cast(uint32_t, x); };
  auto cut = [&](float x) { return __builtin_bit_cast(float, bits(x) & 0xffff0000u); };
  auto upper = [&](float x, float y) { return __builtin_amdgcn_perm(bits(y), bits(x), 0x07060302); };
  hi = upper(a, b);
  a -= cut(a), b -= cut(b);
  mid = upper(a, b);
  a -= cut(a), b -= cut(b);
  lo = upper(a, b);
}
__device__ __forceinline__ Terms split8(const f32x4_t& a, const f32x4_t& b) {
  Terms t;
  split2(a[0], a[1], t.hi.x, t.mid.x, t.lo.x);
  split2(a[2], a[3], t.hi.y, t.mid.y, t.lo.y);
  split2(b[0], b[1], t.hi.z, t.mid.z, t.lo.z);
  split2(b[2], b[3], t.hi.w, t.mid.w, t.lo.w);
  return t;
}
// NT: 32-wide tiles of the state's rows.  A wave has 16 columns of a head's S; the four waves of a workgroup form a quarter of P
// each and share it through LDS (two buffers, formed a chunk ahead: one barrier a chunk that nobody waits long at).  ENDS: only the
// end state of a segment.  The chain of chunks is the critical path and its loads must not be: registers are loaded for the next
// chunk as soon as this one's products have read them, every load and store unconditional, so that the number in flight is known at
// every wait (waves past the last column do the last tile's work once more; past the last chunk the loads fetch it again).
template <int NT, bool ENDS>
__global__ __launch_bounds__(256, 1) void ssm_scan_kernel(const SsmParams p, const SsmChunks k, int vgroups) {
  scalar_cache_acquire();
  constexpr int Np = 32 * NT;
  constexpr bool AHEAD = NT <= 4;          // (a state of 256 rows leaves no registers for the operands of P)
  __shared__ uint4 sP[ENDS ? 1 : 2][ENDS ? 1 : 4 * 2 * 3 * 64];      // fragments (row tile, 32 columns), three terms each
  // the heads of a group, and the column groups of a head, on one XCD (workgroups go to the 8 XCDs in turn)
  const int work = p.H * vgroups, each = (work + 7) / 8;
  const int item = (blockIdx.x & 7) * each + (blockIdx.x >> 3);
  if ((int)(blockIdx.x >> 3) >= each || item >= work) return;
  const int h = item / vgroups, vg = item % vgroups, r = p.in.req0 + blockIdx.y, seg = blockIdx.z;
  // (scalars, so that the operands' addresses are)
  const int s0 = __builtin_amdgcn_readfirstlane(p.in.qsl[r]), L = __builtin_amdgcn_readfirstlane(p.in.qsl[r + 1]) - s0;
  if (L <= 0) return;
  const int start = __builtin_amdgcn_readfirstlane(p.in.seq_lens[r]) - L, all = (L + kC - 1) / kC, segs = (all + k.seg_chunks - 1) / k.seg_chunks;
  if (ENDS ? seg >= segs - 1 : seg >= segs) return;
  const int first = seg * k.seg_chunks, nck = min(k.seg_chunks, all - first);
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, lr = lane & 15, kg = lane >> 4;
  const SsmLayout& lay = k.lay;
  const int grp = h / (p.H / p.G), vt = min(vg * 4 + wave, lay.Vp / 16 - 1), v = vt * 16 + lr;
  float* S = p.state + ((int64_t)p.in.slots[r] * p.H + h) * p.N * p.V;
  auto seg_at = [&](int n) { return k.seg_state + (((int64_t)(r - p.in.req0) * k.nseg + n) * p.H + h) * p.N * p.V; };
  auto log_at = [&](int n) { return k.seg_log + ((int64_t)(r - p.in.req0) * k.nseg + n) * p.H + h; };
  f32x4_t st[2 * NT] = {};                                  // tile n: rows 16 n + 4 kg + i, column v
  auto add_state = [&](const float* src, float keep) {      // st <- keep st + src
#pragma unroll
    for (int n = 0; n < 2 * NT; ++n)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = 16 * n + 4 * kg + i;
        const bool in = d < p.N && v < p.V;
        const float a = src[in ? (int64_t)d * p.V + v : 0];
        st[n][i] = st[n][i] * keep + (in ? a : 0.f);
      }
  };
  auto put_state = [&](float* dst) {
#pragma unroll
    for (int n = 0; n < 2 * NT; ++n)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int d = 16 * n + 4 * kg + i;
        if (d < p.N && v < p.V) dst[(int64_t)d * p.V + v] = st[n][i];
      }
  };
  if (segs == 1) {
    if (start > 0) add_state(S, 0.f);
  } else if constexpr (ENDS) {
    // the first segment starts from the request's state and leaves a copy of it: the pass behind this one overwrites it
    if (seg == 0) {
      if (start > 0) add_state(S, 0.f);
      put_state(seg_at(k.nseg - 1));
    }
  } else if (seg == 0) {
    add_state(seg_at(k.nseg - 1), 0.f);
  } else {
    for (int n = 0; n < seg; ++n) add_state(seg_at(n), n ? fast_exp2(*log_at(n) * kLog2e) : 0.f);
  }
  const int64_t chunk0 = (s0 - __builtin_amdgcn_readfirstlane(p.in.qsl[p.in.req0])) / kC + (r - p.in.req0) + first;
  const uint16_t* base = k.ws + chunk0 * lay.size();
  const int64_t gofs = (int64_t)grp * kC * Np;
  auto chunk = [&](int c) { return base + min(c, nck - 1) * lay.size(); };
  auto numbers = [&](const uint16_t* b, int which) { return reinterpret_cast<const float*>(b + lay.vec()) + ((int64_t)h * 5 + which) * kC; };
  const uint32_t lofs = lane * 16, kofs = kg * 16;
  auto ld4 = [&](const uint16_t* a) { return *reinterpret_cast<const uint4*>(reinterpret_cast<const char*>(a) + lofs); };      // a fragment
  auto ldf4 = [&](const float* a) { return *reinterpret_cast<const f32x4_t*>(reinterpret_cast<const char*>(a) + kofs); };      // values 4 kg ..

  // ---- S <- e^(G_C) S + sum_j B_j (weight_j x_j)^T
  uint4 tf[2 * NT][2], xf[2];
  f32x4_t wx[4];
  float decay;
  auto load_t = [&](int c) {
    const uint16_t* b = chunk(c);
#pragma unroll
    for (int t = 0; t < 2; ++t) xf[t] = ld4(b + lay.xt() + ((int64_t)h * lay.Vp + vt * 16) * kC + t * 512);
    const float* w = numbers(b, kToEnd);
#pragma unroll
    for (int t = 0; t < 4; ++t) wx[t] = ldf4(w + 16 * t);
    decay = numbers(b, kFrom0)[kC - 1];
    const uint16_t* bt = b + lay.bt() + gofs;
#pragma unroll
    for (int n = 0; n < 2 * NT; ++n)
#pragma unroll
      for (int t = 0; t < 2; ++t) tf[n][t] = ld4(bt + (2 * n + t) * 512);
  };
  auto update = [&]() {
    using E = Elem<bf16_tag>;
    Terms xw[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      f32x4_t a = wx[2 * t], b = wx[2 * t + 1];
      a[0] *= E::lo(xf[t].x), a[1] *= E::hi(xf[t].x), a[2] *= E::lo(xf[t].y), a[3] *= E::hi(xf[t].y);
      b[0] *= E::lo(xf[t].z), b[1] *= E::hi(xf[t].z), b[2] *= E::lo(xf[t].w), b[3] *= E::hi(xf[t].w);
      xw[t] = split8(a, b);
    }
#pragma unroll
    for (int n = 0; n < 2 * NT; ++n) st[n] *= decay;
#pragma unroll
    for (int t = 0; t < 2; ++t) {
#pragma unroll
      for (int n = 0; n < 2 * NT; ++n) st[n] = mfma16<bf16_tag>(tf[n][t], xw[t].lo, st[n]);
#pragma unroll
      for (int n = 0; n < 2 * NT; ++n) st[n] = mfma16<bf16_tag>(tf[n][t], xw[t].mid, st[n]);
#pragma unroll
      for (int n = 0; n < 2 * NT; ++n) st[n] = mfma16<bf16_tag>(tf[n][t], xw[t].hi, st[n]);
    }
  };
  if constexpr (ENDS) {
    float seg_sum = 0.f;
    load_t(0);
    for (int ck = 0; ck < nck; ++ck) {
      const float* lead = numbers(chunk(ck), kLead);
      seg_sum += (lead[15] + lead[31]) + (lead[47] + lead[63]);
      update();
      load_t(ck + 1);
      __builtin_amdgcn_sched_barrier(0);
    }
    put_state(seg_at(seg));
    if (tid == 0 && vg == 0) *log_at(seg) = seg_sum;
  } else {
    // ---- P of row tile `wave`, as P^T (rows j, columns i): an accumulator pair is an operand of P X
    uint4 bf[4][NT], cw[NT];
    f32x4_t pw[4], pl;
    float li, m1, m2;
    auto load_p = [&](int c) {
      const uint16_t* b = chunk(c);
      const float* lead = numbers(b, kLead);
      li = lead[16 * wave + lr], m1 = lead[31], m2 = lead[47];
      pl = ldf4(lead + 16 * wave);
#pragma unroll
      for (int t = 0; t < 4; ++t) pw[t] = ldf4(numbers(b, t < wave ? kTail : kDt) + 16 * t);
#pragma unroll
      for (int n = 0; n < NT; ++n) cw[n] = ld4(b + lay.c() + gofs + (wave * NT + n) * 512);
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int n = 0; n < NT; ++n) bf[t][n] = ld4(b + lay.b() + gofs + (t * NT + n) * 512);
    };
    const float skip = p.d[h];
    auto form_p = [&](int c) {
      f32x4_t a[4] = {};
#pragma unroll
      for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int t = 0; t < 4; ++t) a[t] = mfma16<bf16_tag>(bf[t][n], cw[n], a[t]);
      // no branches: what lies behind the diagonal is dropped by selects
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        const float mid = wave - t <= 1 ? 0.f : wave - t == 3 ? m1 + m2 : t == 0 ? m1 : m2;      // the tiles between
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int below = 16 * (wave - t) + lr - (4 * kg + i);      // row - column
          const float e = a[t][i] * pw[t][i] * fast_exp2((t == wave ? li - pl[i] : li + mid) * kLog2e);
          a[t][i] = below > 0 ? e : 0.f;
          if (below == 0) a[t][i] = e + skip;
        }
      }
      uint4* dst = sP[c & 1] + wave * 6 * 64 + lane;
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        const Terms f = split8(a[2 * t], a[2 * t + 1]);
        dst[(3 * t + 0) * 64] = f.hi;
        dst[(3 * t + 1) * 64] = f.mid;
        dst[(3 * t + 2) * 64] = f.lo;
      }
    };
    uint4 cf[4][NT];
    f32x4_t eq[4];
    auto load_c = [&](int c) {
      const uint16_t* b = chunk(c);
#pragma unroll
      for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int t = 0; t < 4; ++t) cf[t][n] = ld4(b + lay.c() + gofs + (t * NT + n) * 512);
#pragma unroll
      for (int t = 0; t < 4; ++t) eq[t] = ldf4(numbers(b, kFrom0) + 16 * t);
    };
    load_p(0);
    load_c(0);
    load_t(0);
    __builtin_amdgcn_sched_barrier(0);
    form_p(0);
    if constexpr (AHEAD) load_p(1);
    __builtin_amdgcn_sched_barrier(0);
    const int64_t ys = (int64_t)p.H * lay.Vp;
    float* yr = k.y + chunk0 * kC * ys + (int64_t)h * lay.Vp + vt * 16;
    const uint32_t yofs = (uint32_t)(4 * kg * ys + lr) * 4;
    for (int ck = 0; ck < nck; ++ck, yr += kC * ys) {
      // every part of this chunk's P is there; nobody still reads the other buffer's
      asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
      const uint4* src = sP[ck & 1] + lane;
      uint4 pf[6][3];                     // row tiles 0..3 of the first 32 columns, 2 and 3 of the others
#pragma unroll
      for (int q = 0; q < 4; ++q)
#pragma unroll
        for (int z = 0; z < 3; ++z) pf[q][z] = src[(q * 6 + z) * 64];
      __builtin_amdgcn_sched_barrier(0);
      // ---- e^(G_i) C S0
      f32x4_t acc[4] = {};
#pragma unroll
      for (int n = 0; n < NT; ++n) {
        const Terms t = split8(st[2 * n], st[2 * n + 1]);
#pragma unroll
        for (int it = 0; it < 4; ++it) acc[it] = mfma16<bf16_tag>(cf[it][n], t.lo, acc[it]);
#pragma unroll
        for (int it = 0; it < 4; ++it) acc[it] = mfma16<bf16_tag>(cf[it][n], t.mid, acc[it]);
#pragma unroll
        for (int it = 0; it < 4; ++it) acc[it] = mfma16<bf16_tag>(cf[it][n], t.hi, acc[it]);
      }
#pragma unroll
      for (int it = 0; it < 4; ++it) acc[it] *= eq[it];
      load_c(ck + 1);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int q = 4; q < 6; ++q)
#pragma unroll
        for (int z = 0; z < 3; ++z) pf[q][z] = src[((q - 2) * 6 + 3 + z) * 64];
#pragma unroll
      for (int z = 2; z >= 0; --z)
#pragma unroll
        for (int it = 0; it < 4; ++it) acc[it] = mfma16<bf16_tag>(pf[it][z], xf[0], acc[it]);
#pragma unroll
      for (int z = 2; z >= 0; --z)
#pragma unroll
        for (int it = 2; it < 4; ++it) acc[it] = mfma16<bf16_tag>(pf[it + 2][z], xf[1], acc[it]);
#pragma unroll
      for (int it = 0; it < 4; ++it)
#pragma unroll
        for (int i = 0; i < 4; ++i) *reinterpret_cast<float*>(reinterpret_cast<char*>(yr + (16 * it + i) * ys) + yofs) = acc[it][i];
      update();
      load_t(ck + 1);
      __builtin_amdgcn_sched_barrier(0);
      if constexpr (!AHEAD) load_p(ck + 1);
      form_p(ck + 1);
      if constexpr (AHEAD) load_p(ck + 2);
      __builtin_amdgcn_sched_barrier(0);
    }
    if (seg == segs - 1) put_state(S);
  }
}

// ------------------------------------------------------------------------------------------------ gate and norm
struct SsmFinish {
  void* out;                // [rows][ld_out]
  const void* z;            // [rows][ld]
  const void* norm_w;       // [H V]
  const float* y;           // the step's [rows - row0][H V], or (chunked) [chunks][64][H][Vp]
  const int32_t* qsl;
  int64_t ld_out, ld;
  int req0, nreq, row0, H, V, pitch;      // pitch: a head's columns in y
  int part, chunked;        // part: columns normed together
  float eps;
};

template <typename T, int VEC, int MAXC>
__global__ __launch_bounds__(256) void ssm_finish_kernel(const SsmFinish p) {
  scalar_cache_acquire();
  __shared__ float smem[16];
  const int64_t row = p.row0 + blockIdx.x;
  const int c0 = blockIdx.y * p.part;
  int64_t at = blockIdx.x;
  if (p.chunked) {
    const int r = p.req0 + row_request(p.qsl + p.req0, p.nreq, (int)row), i = (int)row - p.qsl[r];
    at = chunk_base(p, r) * kC + i;       // (a request's chunks follow each other)
  }
  const float* y = p.y + at * p.H * p.pitch;
  const T* z = reinterpret_cast<const T*>(p.z) + row * p.ld + c0;
  float x[MAXC][VEC];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * blockDim.x) * VEC;
    if (c >= p.part) continue;
    float g[VEC];
    Io<float>::ldv<VEC>(y + (int64_t)((c0 + c) / p.V) * p.pitch + (c0 + c) % p.V, x[k]);
    Io<T>::template ldv<VEC>(z + c, g);
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      x[k][j] *= silu_f(g[j]);
      ss += x[k][j] * x[k][j];
    }
  }
  const float inv = inv_rms(wg_sum(ss, smem), p.part, p.eps);
  const T* w = reinterpret_cast<const T*>(p.norm_w) + c0;
  T* out = reinterpret_cast<T*>(p.out) + row * p.ld_out + c0;
#pragma unroll
  for (int k = 0; k < MAXC; ++k) {
    const int c = (threadIdx.x + k * blockDim.x) * VEC;
    if (c >= p.part) continue;
    float wv[VEC];
    Io<T>::template ldv<VEC>(w + c, wv);
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[k][j] *= inv * wv[j];
    Io<T>::template stv<VEC>(out + c, x[k]);
  }
}

template <typename T>
int finish(const SsmFinish& f, int rows, int parts, hipStream_t s) {
  const int al = 16 / sizeof(T), n = f.part;
  const bool vec = n % 8 == 0 && f.V % 8 == 0 && f.ld_out % al == 0 && f.ld % al == 0 && aligned16(f.out) && aligned16(f.z) && aligned16(f.norm_w);
  const int per = vec ? 8 : 1;
  const dim3 grid(rows, parts), block(n <= 64 * per ? 64 : n <= 128 * per ? 128 : 256);
#define MI_SF(VEC, MAXC) hipLaunchKernelGGL((ssm_finish_kernel<T, VEC, MAXC>), grid, block, 0, s, f)
  if (vec) {
    if (n <= 2048) MI_SF(8, 1);
    else if (n <= 4096) MI_SF(8, 2);
    else if (n <= 16384) MI_SF(8, 8);
    else return MI_ERR_UNSUPPORTED;
  } else {
    if (n <= 1024) MI_SF(1, 4);
    else if (n <= 8192) MI_SF(1, 32);
    else return MI_ERR_UNSUPPORTED;
  }
#undef MI_SF
  return launch_status();
}

template <typename T>
int step(const SsmParams& p, int nreq, hipStream_t s) {
  const bool v4 = p.V % 4 == 0;
  const int gr = v4 ? 16 : 4, need = (p.N + gr - 1) / gr;
  const dim3 grid(p.H, (p.V + kCols - 1) / kCols, nreq), block(256);
  const size_t lds = (size_t)(kCols + 2 * p.N + gr * kCols) * sizeof(float);
#define MI_SS(VEC, R)                                                                                     \
  do {                                                                                                    \
    if (p.in.taps == 4) hipLaunchKernelGGL((state_step_kernel<T, VEC, R, 4>), grid, block, lds, s, p);    \
    else hipLaunchKernelGGL((state_step_kernel<T, VEC, R, 0>), grid, block, lds, s, p);                   \
  } while (0)
  if (v4) {
    if (need <= 2) MI_SS(4, 2);
    else if (need <= 4) MI_SS(4, 4);
    else if (need <= 8) MI_SS(4, 8);
    else if (need <= 16) MI_SS(4, 16);
    else if (need <= 32) MI_SS(4, 32);
    else return MI_ERR_UNSUPPORTED;
  } else {
    if (need <= 16) MI_SS(1, 16);
    else if (need <= 64) MI_SS(1, 64);
    else if (need <= 128) MI_SS(1, 128);
    else return MI_ERR_UNSUPPORTED;
  }
#undef MI_SS
  return launch_status();
}

bool ssm_layout(int G, int H, int N, int V, SsmLayout* lay) {
  if (N > 256 || V > 256) return false;
  *lay = SsmLayout{G, H, N <= 32 ? 32 : N <= 64 ? 64 : N <= 128 ? 128 : 256, (V + 15) / 16 * 16};
  return true;
}

template <bool ENDS>
int launch_scan(const SsmParams& p, const SsmChunks& k, int nreq, hipStream_t s) {
  const int vgroups = (p.V + 63) / 64;
  const dim3 grid((p.H * vgroups + 7) / 8 * 8, nreq, ENDS ? k.nseg - 1 : k.nseg), block(256);
#define MI_SC(NT) hipLaunchKernelGGL((ssm_scan_kernel<NT, ENDS>), grid, block, 0, s, p, k, vgroups)
  switch (k.lay.Np / 32) {
    case 1: MI_SC(1); break;
    case 2: MI_SC(2); break;
    case 4: MI_SC(4); break;
    default: MI_SC(8); break;
  }
#undef MI_SC
  return launch_status();
}

int64_t align256(int64_t n) { return (n + 255) / 256 * 256; }

}  // namespace
}  // namespace mi

using namespace mi;

extern "C" int64_t mi_state_space_workspace_bytes(int32_t rows, int32_t num_reqs, int32_t heads, int32_t groups, int32_t state_dim,
                                                  int32_t vdim, int32_t chunked, int dtype) {
  if (rows < 0 || num_reqs < 0 || heads <= 0 || groups <= 0 || state_dim <= 0 || vdim <= 0) return 0;
  if (!chunked) return align256((int64_t)rows * heads * vdim * 4);
  SsmLayout lay;
  if (dtype != MI_DTYPE_BF16 || !ssm_layout(groups, heads, state_dim, vdim, &lay)) return 0;
  const int64_t chunks = (int64_t)rows / kC + num_reqs;
  return align256(chunks * kC * heads * lay.Vp * 4) + align256(chunks * lay.size() * 2) +
         (int64_t)num_reqs * kMaxSegments * heads * ((int64_t)state_dim * vdim + 1) * 4;
}

extern "C" int mi_state_space(const mi_state_space_args* a, int32_t row0, int32_t rows, int32_t max_query_len, int32_t chunked,
                              void* workspace, int64_t workspace_bytes, int dtype, void* stream) {
  if (a && (a->num_reqs == 0 || rows == 0)) return MI_OK;
  if (!a || !a->xbc || !a->z || !a->dt || !a->conv_w || !a->conv_b || !a->norm_w || !a->dt_bias || !a->a_log || !a->d || !a->state ||
      !a->ring || !a->slots || !a->query_start_loc || !a->seq_lens || !a->out || !workspace)
    return MI_ERR_INVALID_ARG;
  const int H = a->heads, G = a->groups, N = a->state_dim, V = a->vdim, nreq = a->num_reqs;
  if (a->req0 < 0 || nreq < 0 || row0 < 0 || rows < 0 || max_query_len <= 0 || H <= 0 || G <= 0 || H % G || N <= 0 || V <= 0 ||
      a->taps <= 0 || a->norm_groups <= 0 || H * V % a->norm_groups)
    return MI_ERR_INVALID_ARG;
  const int inner = H * V, ch = inner + 2 * G * N;
  if (a->stride < ch || a->out_stride < inner) return MI_ERR_INVALID_ARG;
  if (dtype != MI_DTYPE_BF16 && dtype != MI_DTYPE_F32) return MI_ERR_UNSUPPORTED;
  const int64_t need = mi_state_space_workspace_bytes(rows, nreq, H, G, N, V, chunked, dtype);
  if (need == 0 || nreq > 65535) return MI_ERR_UNSUPPORTED;
  if (workspace_bytes < need) return MI_ERR_WORKSPACE;
  hipStream_t s = (hipStream_t)stream;
  float* y = (float*)workspace;
  const SsmParams p{{a->xbc, a->conv_w, a->ring, a->slots, a->query_start_loc, a->seq_lens, a->stride, a->req0, a->taps, ch},
                    a->conv_b, a->dt, a->dt_bias, a->a_log, a->d, a->state, y, row0, H, G, N, V};
  int rc;
  SsmChunks k{};
  if (!chunked) {
    rc = dtype == MI_DTYPE_BF16 ? step<uint16_t>(p, nreq, s) : step<float>(p, nreq, s);
  } else {
    const int64_t held = (int64_t)rows / kC + nreq;
    ssm_layout(G, H, N, V, &k.lay);
    k.y = y;
    k.ws = (uint16_t*)((char*)workspace + align256(held * kC * H * k.lay.Vp * 4));
    k.seg_state = (float*)((char*)k.ws + align256(held * k.lay.size() * 2));
    k.seg_log = k.seg_state + (int64_t)nreq * kMaxSegments * H * N * V;
    k.vec = N % 8 == 0 && V % 8 == 0 && a->stride % 8 == 0 && aligned16(a->xbc) && aligned16(a->ring) && aligned16(a->conv_b) &&
            aligned16(a->conv_w);
    const int chunks = (max_query_len + kC - 1) / kC;
    const int64_t groups = (int64_t)nreq * H * ((V + 63) / 64);
    int n = (int)(256 / groups);                           // segments: a workgroup a CU
    if (n > chunks / 4) n = chunks / 4;
    if (n > kMaxSegments) n = kMaxSegments;
    if (n < 1) n = 1;
    k.seg_chunks = (chunks + n - 1) / n;
    k.nseg = (chunks + k.seg_chunks - 1) / k.seg_chunks;
    const int blocks = H * ((k.lay.Vp + kPrepCh - 1) / kPrepCh) + 2 * G * ((k.lay.Np + kPrepCh - 1) / kPrepCh) + (H + 1) / 2;
    if (blocks > 65535) return MI_ERR_UNSUPPORTED;
    hipLaunchKernelGGL(ssm_prep_kernel, dim3(chunks, blocks, nreq), dim3(128), 0, s, p, k);
    rc = launch_status();
    if (rc == MI_OK && k.nseg > 1) rc = launch_scan<true>(p, k, nreq, s);
    if (rc == MI_OK) rc = launch_scan<false>(p, k, nreq, s);
  }
  if (rc != MI_OK) return rc;
  if (chunked || max_query_len > 1) {      // (a step of one row has left it there itself)
    rc = dtype == MI_DTYPE_BF16 ? launch_conv_update<uint16_t>(p.in, nreq, s) : launch_conv_update<float>(p.in, nreq, s);
    if (rc != MI_OK) return rc;
  }
  const SsmFinish f{a->out, a->z, a->norm_w, y, a->query_start_loc, a->out_stride, a->stride, a->req0, nreq, row0, H, V,
                    chunked ? k.lay.Vp : V, inner / a->norm_groups, chunked, a->eps};
  return dtype == MI_DTYPE_BF16 ? finish<uint16_t>(f, rows, a->norm_groups, s) : finish<float>(f, rows, a->norm_groups, s);
}
