// Linear recurrences with ONE decay per head and token (state-space duality, decayed linear attention):
//     S_t = a_t S_(t-1) + k_t (c_t v_t)^T,      o_t = S_t^T q_t + D v_t
// with S [dim, vdim] per request and head, q and k shared by the heads of a group, a_t a number per token and head or
// a constant of the head, and the factor c_t and the skip D options.  Around it: the step that prepares a
// state-space mixer's operands (a short causal convolution with bias and SiLU per channel, step sizes through
// softplus, decays from them).
//
// Everything is float32 in both precisions.  Per request the state row holds S of every head as [heads][dim][vdim]
// from column 0 (a convolution's saved inputs lie behind it).
#include "common.h"

namespace {

constexpr int kThreads = 256;

__device__ __forceinline__ float silu(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// Row t of p: the convolutions' inputs from column conv_off (`channels` of them), step sizes' pre-activations from
// dt_off (one per head).  Row t of x: [silu(conv + bias): channels | c = softplus(dt + dt_bias): heads, from column
// dt_col | ln a = -exp(A_log) c: heads, from a_col].  A thread takes one channel (or head) of a run of up to RUN tokens
// of a request.
template <int RUN, int TAPS>
__global__ __launch_bounds__(kThreads) void ssd_prepare_kernel(
    const float* __restrict__ p, int64_t p_stride, int conv_off, int dt_off, const float* __restrict__ conv_b,
    const float* __restrict__ a_log, const float* __restrict__ dt_bias, const ShortConv conv, float* __restrict__ x,
    int64_t x_stride, int dt_col, int a_col, int channels, int heads, const int32_t* __restrict__ tile_req,
    const int32_t* __restrict__ tile_tok0, const int32_t* __restrict__ tile_ntok) {
  const int tile = blockIdx.x;
  const int c = blockIdx.y * kThreads + threadIdx.x;
  if (c >= channels + heads) return;
  const int req = RUN == 1 ? tile : tile_req[tile], tok0 = RUN == 1 ? tile : tile_tok0[tile];
  const int n_tok = RUN == 1 ? 1 : tile_ntok[tile];
  if (n_tok <= 0) return;                    // a padding tile
  if (c >= channels) {
    const int h = c - channels;
    const float rate = -expf(a_log[h]), bias = dt_bias[h];
    for (int tt = 0; tt < n_tok; ++tt) {
      const int64_t t = tok0 + tt;
      const float dt = softplus(p[t * p_stride + dt_off + h] + bias);
      x[t * x_stride + dt_col + h] = dt;
      x[t * x_stride + a_col + h] = rate * dt;
    }
    return;
  }
  const int t0 = RUN == 1 ? tok0 : conv.cu[req];
  float* saved = conv.taps > 1 ? conv.state + (int64_t)conv.slots[req] * conv.state_stride + conv.saved_off +
                                     (int64_t)c * (conv.taps - 1)
                               : nullptr;
  ConvRun<RUN, TAPS> cv;
  cv.load(conv, p + conv_off + c, p_stride, t0, tok0 - t0, n_tok, c, 0.f, saved);
  const float b = conv_b ? conv_b[c] : 0.f;
#pragma unroll
  for (int tt = 0; tt < RUN; ++tt)
    if (tt < n_tok) x[(int64_t)(tok0 + tt) * x_stride + c] = silu(cv.value(tt) + b);
  if (RUN == 1 && conv.taps > 1) cv.save_first(conv, saved);
}

// What a recurrence reads: rows x[t] with q and k (groups x dim numbers, from q_off and k_off), v (heads x vdim, from
// v_off); c and the decay's logarithm ln a per head from c_off and a_off, or, where these are negative, 1 and decay[h]
// (the decay itself); silu: q, k and v are pre-activations.
struct Operands {
  const float* x;
  int64_t x_stride;
  int q_off, k_off, v_off, c_off, a_off;
  const float* decay;
  const float* skip;      // D per head, or null
  int heads, groups, dim, vdim, silu;
  int vec;                // every size, column and row is a multiple of four floats, the rows begin at 16 bytes
};

// Any number of tokens.  A workgroup owns EC value columns of one (request, head) and walks the request's tokens of
// this step in order.  The rows of S are cut into P slices of 8 (P a power of two, 8 P >= dim); thread (e, p) keeps
// S[8 p .. 8 p + 7, e] in registers, and the P lanes of a column are neighbours, so the sum over the rows ends with
// log2 P lane exchanges.  q, k and v of 16 tokens at a time are staged in LDS, the next 16 requested before these are
// worked on.  The order of additions is the same whatever the step holds.
constexpr int kSlice = 8;
constexpr int kChunk = 16;

template <int P>
__device__ __forceinline__ float sum_over_slices(float v) {
  if constexpr (P >= 2) v += dpp_f32<TL_DPP_XOR1>(v);
  if constexpr (P >= 4) v += dpp_f32<TL_DPP_XOR2>(v);
  if constexpr (P >= 8) v += dpp_f32<TL_DPP_HALF_MIRROR>(v);      // the quads of a half row hold one value each by now
  if constexpr (P >= 16) v += dpp_f32<TL_DPP_MIRROR>(v);
  if constexpr (P >= 32) {
    float a, b;
    pair16(v, a, b);
    v = a + b;
  }
  return v;
}

template <int P>
__global__ __launch_bounds__(kThreads) void linear_recurrence_kernel(const Operands op, float* __restrict__ state,
                                                                     int64_t state_stride, const int32_t* __restrict__ cu,
                                                                     const int32_t* __restrict__ slots,
                                                                     float* __restrict__ o) {
  constexpr int EC = kThreads / P, Dp = kSlice * P;
  constexpr int NST = (kChunk * Dp + kThreads - 1) / kThreads, NV = (kChunk * EC + kThreads - 1) / kThreads;
  __shared__ __align__(16) float q_s[kChunk * Dp];
  __shared__ __align__(16) float k_s[kChunk * Dp];
  __shared__ float v_s[kChunk * EC], a_s[kChunk], c_s[kChunk];
  const int req = blockIdx.z, head = blockIdx.y;
  const int t0 = cu[req], n = cu[req + 1] - t0;
  if (n <= 0) return;                     // a request without tokens touches no state
  const int dim = op.dim, vdim = op.vdim, group = head / (op.heads / op.groups);
  const int tid = threadIdx.x, p = tid % P, el = tid / P;
  const int e = blockIdx.x * EC + el;
  const bool col = e < vdim;
  float* Sg = state + (int64_t)slots[req] * state_stride + ((int64_t)head * dim + p * kSlice) * vdim + (col ? e : 0);
  float S[kSlice];
#pragma unroll
  for (int s = 0; s < kSlice; ++s) S[s] = (col && p * kSlice + s < dim) ? Sg[(int64_t)s * vdim] : 0.f;
  const float skip = op.skip ? op.skip[head] : 0.f;
  const float decay = op.a_off < 0 ? op.decay[head] : 0.f;
  // what this thread stages of a chunk: element i = tid + j * kThreads of [token][channel], token i / Dp
  float pq[NST], pk[NST], pv[NV], pa = 0.f, pc = 0.f;
  auto fetch = [&](int c0) {
    const int m = min(kChunk, n - c0);
#pragma unroll
    for (int j = 0; j < NST; ++j) {
      const int i = tid + j * kThreads, tt = i / Dp, d = i % Dp;
      pq[j] = pk[j] = 0.f;
      if (i < kChunk * Dp && tt < m && d < dim) {
        const float* row = op.x + (int64_t)(t0 + c0 + tt) * op.x_stride + group * dim + d;
        pq[j] = row[op.q_off];
        pk[j] = row[op.k_off];
      }
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = tid + j * kThreads, tt = i / EC, ee = blockIdx.x * EC + i % EC;
      pv[j] = (i < kChunk * EC && tt < m && ee < vdim) ? op.x[(int64_t)(t0 + c0 + tt) * op.x_stride + op.v_off + head * vdim + ee] : 0.f;
    }
    if (tid < kChunk && tid < m) {
      const float* row = op.x + (int64_t)(t0 + c0 + tid) * op.x_stride + head;
      pa = op.a_off < 0 ? decay : expf(row[op.a_off]);
      pc = op.c_off < 0 ? 1.f : row[op.c_off];
    }
  };
  fetch(0);
  for (int c0 = 0; c0 < n; c0 += kChunk) {
    const int m = min(kChunk, n - c0);
    __syncthreads();                       // the chunk before is done with
#pragma unroll
    for (int j = 0; j < NST; ++j) {
      const int i = tid + j * kThreads;
      if (i < kChunk * Dp) {
        q_s[i] = op.silu ? silu(pq[j]) : pq[j];
        k_s[i] = op.silu ? silu(pk[j]) : pk[j];
      }
    }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
      const int i = tid + j * kThreads;
      if (i < kChunk * EC) v_s[i] = op.silu ? silu(pv[j]) : pv[j];
    }
    if (tid < kChunk) {
      a_s[tid] = pa;
      c_s[tid] = pc;
    }
    __syncthreads();
    if (c0 + kChunk < n) fetch(c0 + kChunk);      // on its way while this chunk is worked on
    const int64_t o_step = (int64_t)op.heads * vdim;
    float* orow = o + (int64_t)(t0 + c0) * o_step + head * vdim + e;
    auto token = [&](int tt) {
      const float v = v_s[tt * EC + el], a = a_s[tt], cv = c_s[tt] * v;
      float acc[2] = {0.f, 0.f};
#pragma unroll
      for (int i = 0; i < kSlice; i += 4) {
        const f32x4 q4 = *(const f32x4*)(q_s + tt * Dp + p * kSlice + i), k4 = *(const f32x4*)(k_s + tt * Dp + p * kSlice + i);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          S[i + j] = fmaf(a, S[i + j], k4[j] * cv);
          acc[j & 1] = fmaf(q4[j], S[i + j], acc[j & 1]);
        }
      }
      const float sum = sum_over_slices<P>(acc[0] + acc[1]);
      if (p == 0 && col) orow[(int64_t)tt * o_step] = fmaf(skip, v, sum);
    };
    if (m == kChunk) {
#pragma unroll 4
      for (int tt = 0; tt < kChunk; ++tt) token(tt);
    } else {
      for (int tt = 0; tt < m; ++tt) token(tt);
    }
  }
#pragma unroll
  for (int s = 0; s < kSlice; ++s)
    if (col && p * kSlice + s < dim) Sg[(int64_t)s * vdim] = S[s];
}

// A decode step: every request brings one token.  One workgroup per (request, head): thread (cq, sl) holds the value
// columns 4 cq .. 4 cq + 3 of rows sl, sl + NS, sl + 2 NS, ... of S, so that a wave's 16-byte loads and stores cover
// consecutive rows; the NS slices' partial sums meet in LDS and are added in a fixed order.
template <int ROWS>
__global__ __launch_bounds__(kThreads) void linear_recurrence_decode_kernel(const Operands op, float* __restrict__ state,
                                                                            int64_t state_stride,
                                                                            const int32_t* __restrict__ cu,
                                                                            const int32_t* __restrict__ slots,
                                                                            float* __restrict__ o) {
  __shared__ float q_s[kThreads], k_s[kThreads];
  __shared__ f32x4 part[kThreads];
  const int r = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
  const int t = cu[r];
  if (cu[r + 1] - t != 1) return;         // a padding request owns no state (the whole workgroup)
  const int dim = op.dim, vdim = op.vdim, group = head / (op.heads / op.groups);
  const int quads = vdim / 4, NS = kThreads / quads;
  const int cq = tid % quads, sl = tid / quads;
  const bool live = sl < NS;
  const float* row = op.x + (int64_t)t * op.x_stride;
  float* S_mem = state + (int64_t)slots[r] * state_stride + (int64_t)head * dim * vdim + cq * 4;
  // everything the token needs is requested before the first value is used
  const float q = tid < dim ? row[op.q_off + group * dim + tid] : 0.f, k = tid < dim ? row[op.k_off + group * dim + tid] : 0.f;
  float v[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) v[e] = row[op.v_off + head * vdim + cq * 4 + e];
  const float a = op.a_off < 0 ? op.decay[head] : expf(row[op.a_off + head]);
  const float c = op.c_off < 0 ? 1.f : row[op.c_off + head];
  const float skip = op.skip ? op.skip[head] : 0.f;
  f32x4 S[ROWS];
#pragma unroll
  for (int j = 0; j < ROWS; ++j) {
    const int i = sl + j * NS;
    S[j] = (live && i < dim) ? *(const f32x4*)(S_mem + (int64_t)i * vdim) : f32x4{0.f, 0.f, 0.f, 0.f};
  }
  if (tid < dim) {
    q_s[tid] = op.silu ? silu(q) : q;
    k_s[tid] = op.silu ? silu(k) : k;
  }
  if (op.silu) {
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = silu(v[e]);
  }
  __syncthreads();
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < ROWS; ++j) {
    const int i = sl + j * NS;
    if (live && i < dim) {
      const float ki = k_s[i], qi = q_s[i];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[j][e] = fmaf(a, S[j][e], ki * (c * v[e]));
        acc[e] = fmaf(qi, S[j][e], acc[e]);
      }
      *(f32x4*)(S_mem + (int64_t)i * vdim) = S[j];
    }
  }
  part[tid] = acc;
  __syncthreads();
  if (tid < vdim) {                       // one column a thread (vdim <= 256)
    const float* pf = (const float*)part;
    float sum = 0.f;
    for (int s = 0; s < NS; ++s) sum += pf[(s * quads + tid / 4) * 4 + tid % 4];
    const float pre = row[op.v_off + head * vdim + tid];
    o[((int64_t)t * op.heads + head) * vdim + tid] = fmaf(skip, op.silu ? silu(pre) : pre, sum);
  }
}

// ------------------------------------------------------------------------------ many tokens, in chunks
// The same recurrence over chunks of 64 tokens, so that a prompt fills the chip and its arithmetic runs on the matrix
// cores (v_mfma_f32_16x16x4_f32: true float32).  With L_i = sum of ln a over the chunk's tokens up to i, and S the state
// ahead of the chunk,
//     o_i = exp(L_i) S^T q_i + sum_(j <= i) exp(L_i - L_j) (q_i . k_j) c_j v_j + D v_i
//     S'  = exp(L_63) S + U,      U = sum_j exp(L_63 - L_j) k_j (c_j v_j)^T
// Three launches: U and exp(L_63) of every chunk (chunk_update), the states ahead of every chunk from them, in place of
// U (chunk_scan: the only step that walks a request's chunks in order, two operations an element), and the outputs
// (chunk_output).  Chunks are cut inside a request from the step's first token of it on; the last one is filled up with
// tokens that add nothing and do not decay.  Every exponent is a difference of two prefix sums; these are formed in
// float64, so that a strong decay early in a chunk costs later differences nothing.
constexpr int kC = 64;            // tokens of a chunk
constexpr int kVB = 64;           // value columns a workgroup takes

struct ChunkTiles {
  const int32_t* tok0;            // first token row and number of tokens of every chunk (0: padding)
  const int32_t* ntok;
};

// Wave 0: lam[i] = sum of ln a over the chunk's tokens 0 .. i.
__device__ __forceinline__ void chunk_log_decays(const Operands& op, int head, int tok0, int n, double* lam) {
  const int lane = threadIdx.x;
  if (lane >= TL_WAVE) return;
  double v = 0.0;
  if (lane < n) {
    if (op.a_off < 0) v = fmax(log((double)op.decay[head]), -800.0);      // a decay of zero: exp(-800) is zero
    else v = fmax((double)op.x[(int64_t)(tok0 + lane) * op.x_stride + op.a_off + head], -1e6);
  }
#pragma unroll
  for (int d = 1; d < TL_WAVE; d *= 2) {
    const double o = __shfl_up(v, d, TL_WAVE);
    if (lane >= d) v += o;
  }
  lam[lane] = v;
}

// Four neighbouring numbers of a chunk's token t, from channel i on, as they are; zero beyond the chunk's n tokens and
// the `width` channels there are.
__device__ __forceinline__ f32x4 chunk_load(const Operands& op, const float* __restrict__ base, int t, int n, int i, int width) {
  f32x4 r = {0.f, 0.f, 0.f, 0.f};
  if (t < n) {
    const float* p = base + (int64_t)t * op.x_stride + i;
    if (op.vec) {                     // uniform: whole vectors only (sizes and columns are multiples of four)
      if (i < width) r = *(const f32x4*)p;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (i + e < width) r[e] = p[e];
    }
  }
  return r;
}
__device__ __forceinline__ f32x4 chunk_act(const Operands& op, f32x4 r) {
  if (op.silu) {
#pragma unroll
    for (int e = 0; e < 4; ++e) r[e] = silu(r[e]);      // silu(0) = 0
  }
  return r;
}
// A chunk's kC rows of W channels, a share of every thread: vector j is row chunk_row<W>(j), channels from chunk_col<W>(j).
template <int W>
struct ChunkRows {
  static constexpr int G = kC * W / 4 / kThreads;
  f32x4 r[G];
  __device__ __forceinline__ static int row(int j) { return (threadIdx.x + j * kThreads) / (W / 4); }
  __device__ __forceinline__ static int col(int j) { return (threadIdx.x + j * kThreads) % (W / 4) * 4; }
  __device__ __forceinline__ void load(const Operands& op, const float* __restrict__ base, int n, int width) {
#pragma unroll
    for (int j = 0; j < G; ++j) r[j] = chunk_load(op, base, row(j), n, col(j), width);
  }
  __device__ __forceinline__ void store(const Operands& op, float* __restrict__ dst, int stride) {
#pragma unroll
    for (int j = 0; j < G; ++j) *(f32x4*)(dst + row(j) * stride + col(j)) = chunk_act(op, r[j]);
  }
};

// U[tile][head][n][v] and decay[tile][head] = exp(L_63).  A wave owns 16 x 16 blocks of U in turn.
template <int NB>
__global__ __launch_bounds__(kThreads) void chunk_update_kernel(const Operands op, const ChunkTiles tiles, float* __restrict__ U,
                                                                float* __restrict__ decay) {
  constexpr int KS = NB * 16 + 16, VS = kVB + 16;      // row strides: four neighbouring rows begin 16 banks apart
  extern __shared__ __attribute__((aligned(16))) float smem[];
  float* K = smem;                  // [kC][KS]
  float* V = smem + kC * KS;        // [kC][VS], times c_t exp(L_63 - L_t)
  __shared__ double lam[kC];
  const int tile = blockIdx.x, head = blockIdx.y, v0 = blockIdx.z * kVB, tid = threadIdx.x;
  const int n = tiles.ntok[tile];
  if (n <= 0) return;               // a padding tile (the whole workgroup)
  const int tok0 = tiles.tok0[tile], dim = op.dim, vdim = op.vdim, group = head / (op.heads / op.groups);
  const int VT = min(kVB, vdim - v0 + 15) / 16;
  ChunkRows<NB * 16> k;
  ChunkRows<kVB> v;
  float c[ChunkRows<kVB>::G];
  k.load(op, op.x + (int64_t)tok0 * op.x_stride + op.k_off + group * dim, n, dim);
  v.load(op, op.x + (int64_t)tok0 * op.x_stride + op.v_off + head * vdim + v0, n, vdim - v0);
#pragma unroll
  for (int j = 0; j < v.G; ++j)
    c[j] = op.c_off >= 0 ? op.x[(int64_t)(tok0 + min(v.row(j), n - 1)) * op.x_stride + op.c_off + head] : 1.f;
  chunk_log_decays(op, head, tok0, n, lam);
  k.store(op, K, KS);
  __syncthreads();
#pragma unroll
  for (int j = 0; j < v.G; ++j) {
    const float f = c[j] * expf((float)(lam[kC - 1] - lam[v.row(j)]));
    f32x4 x = chunk_act(op, v.r[j]);
#pragma unroll
    for (int e = 0; e < 4; ++e) x[e] *= f;
    *(f32x4*)(V + v.row(j) * VS + v.col(j)) = x;
  }
  if (blockIdx.z == 0 && tid == 0) decay[(int64_t)tile * op.heads + head] = expf((float)lam[kC - 1]);
  __syncthreads();
  const int wave = tid / TL_WAVE, lane = tid % TL_WAVE, l16 = lane % 16, kk = lane / 16;
  float* out = U + ((int64_t)tile * op.heads + head) * dim * vdim;
  for (int b = wave; b < NB * VT; b += kThreads / TL_WAVE) {
    const int nb = b / VT, vt = b % VT;
    if (nb * 16 >= dim) break;      // (only blocks beyond the head's channels follow)
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int st = 0; st < kC / 4; ++st)
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(K[(st * 4 + kk) * KS + nb * 16 + l16], V[(st * 4 + kk) * VS + vt * 16 + l16],
                                                 acc, 0, 0, 0);
    const int v = v0 + vt * 16 + l16;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int row = nb * 16 + kk * 4 + r;
      if (row < dim && v < vdim) out[(int64_t)row * vdim + v] = acc[r];
    }
  }
}

// In place of every chunk's U the state ahead of the chunk; the state behind a request's last chunk becomes its state.
template <int VEC>
__global__ __launch_bounds__(kThreads) void chunk_scan_kernel(float* __restrict__ U, const float* __restrict__ decay,
                                                              float* __restrict__ state, int64_t state_stride,
                                                              const int32_t* __restrict__ cu, const int32_t* __restrict__ slots,
                                                              int heads, int size) {
  typedef float vec __attribute__((ext_vector_type(VEC)));
  const int head = blockIdx.y, req = blockIdx.z;
  const int n = cu[req + 1] - cu[req];
  const int at = (blockIdx.x * kThreads + threadIdx.x) * VEC;
  if (n <= 0) return;               // (the whole workgroup)
  // the request's first chunk: those of the requests in front of it come first
  __shared__ float red[kThreads / TL_WAVE];
  int before = 0;
  for (int r = threadIdx.x; r < req; r += kThreads) before += (cu[r + 1] - cu[r] + kC - 1) / kC;
  const int first = (int)block_sum<kThreads / TL_WAVE>((float)before, red);      // exact: far below 2^24
  if (at >= size) return;
  const int chunks = (n + kC - 1) / kC;
  float* sp = state + (int64_t)slots[req] * state_stride + (int64_t)head * size + at;
  vec S = *(const vec*)sp;
  constexpr int kAhead = 8;
  for (int c0 = 0; c0 < chunks; c0 += kAhead) {
    const int m = min(kAhead, chunks - c0);
    vec u[kAhead];
    float d[kAhead];
#pragma unroll
    for (int j = 0; j < kAhead; ++j)
      if (j < m) {
        const int64_t row = (int64_t)(first + c0 + j) * heads + head;
        u[j] = *(const vec*)(U + row * size + at);
        d[j] = decay[row];
      }
#pragma unroll
    for (int j = 0; j < kAhead; ++j)
      if (j < m) {
        *(vec*)(U + ((int64_t)(first + c0 + j) * heads + head) * size + at) = S;
#pragma unroll
        for (int e = 0; e < VEC; ++e) S[e] = fmaf(d[j], S[e], u[j][e]);
      }
  }
  *(vec*)sp = S;
}

// The outputs of a chunk.  Wave w owns the chunk's tokens 16 w .. 16 w + 15.  It forms the scores transposed, K Q^T, so
// that a lane holds four scores of ONE token (lane l16), which are the second operand of V^T P^T as they are.
template <int NB>
__global__ __launch_bounds__(kThreads, NB <= 8 ? 3 : 2) void chunk_output_kernel(const Operands op, const ChunkTiles tiles,
                                                                const float* __restrict__ S_in, float* __restrict__ o) {
  constexpr int KS = NB * 16 + 4, VS = kVB + 4;        // row strides: neighbouring rows begin four banks apart
  constexpr int AREA = kC * KS > NB * 16 * VS ? kC * KS : NB * 16 * VS;
  constexpr int PER = NB * 16 * kVB / 4 / kThreads;    // vectors of S a thread moves
  extern __shared__ __attribute__((aligned(16))) float smem[];
  float* K = smem;                  // [kC][KS], later S [NB * 16][VS]
  float* V = smem + AREA;           // [kC][VS], times c_t
  __shared__ double lam[kC];
  const int tile = blockIdx.x, head = blockIdx.y, v0 = blockIdx.z * kVB, tid = threadIdx.x;
  const int n = tiles.ntok[tile];
  if (n <= 0) return;               // a padding tile (the whole workgroup)
  const int tok0 = tiles.tok0[tile], dim = op.dim, vdim = op.vdim, group = head / (op.heads / op.groups);
  const int VT = min(kVB, vdim - v0 + 15) / 16;
  const int wave = tid / TL_WAVE, lane = tid % TL_WAVE, l16 = lane % 16, kk = lane / 16;
  const float* qb = op.x + (int64_t)tok0 * op.x_stride + op.q_off + group * dim;
  const float* vb = op.x + (int64_t)tok0 * op.x_stride + op.v_off + head * vdim + v0;
  const int i = wave * 16 + l16;    // this lane's token
  ChunkRows<NB * 16> k;
  ChunkRows<kVB> v;
  float c[ChunkRows<kVB>::G];
  f32x4 q[NB], sreg[PER];
  k.load(op, op.x + (int64_t)tok0 * op.x_stride + op.k_off + group * dim, n, dim);
#pragma unroll
  for (int s = 0; s < NB; ++s) q[s] = chunk_load(op, qb, i, n, s * 16 + kk * 4, dim);
  v.load(op, vb, n, vdim - v0);
#pragma unroll
  for (int j = 0; j < v.G; ++j)
    c[j] = op.c_off >= 0 ? op.x[(int64_t)(tok0 + min(v.row(j), n - 1)) * op.x_stride + op.c_off + head] : 1.f;
  chunk_log_decays(op, head, tok0, n, lam);
  k.store(op, K, KS);
#pragma unroll
  for (int j = 0; j < v.G; ++j) {
    f32x4 x = chunk_act(op, v.r[j]);
#pragma unroll
    for (int e = 0; e < 4; ++e) x[e] *= c[j];
    *(f32x4*)(V + v.row(j) * VS + v.col(j)) = x;
  }
#pragma unroll
  for (int s = 0; s < NB; ++s) q[s] = chunk_act(op, q[s]);
  // S on its way while the scores are formed
  const float* sp = S_in + ((int64_t)tile * op.heads + head) * dim * vdim + v0;
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int e = tid + j * kThreads, row = e / (kVB / 4), col = e % (kVB / 4) * 4;
    sreg[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (row < dim) {
      if (op.vec) {
        if (v0 + col < vdim) sreg[j] = *(const f32x4*)(sp + (int64_t)row * vdim + col);
      } else {
#pragma unroll
        for (int e4 = 0; e4 < 4; ++e4)
          if (v0 + col + e4 < vdim) sreg[j][e4] = sp[(int64_t)row * vdim + col + e4];
      }
    }
  }
  __syncthreads();
  const double lam_i = lam[i];
  f32x4 p[kC / 16];
#pragma unroll
  for (int J = 0; J < kC / 16; ++J) {
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    if (J <= wave) {                // (the whole wave)
#pragma unroll
      for (int s = 0; s < NB; ++s) {
        const f32x4 kf = *(const f32x4*)(K + (J * 16 + l16) * KS + s * 16 + kk * 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[e], q[s][e], acc, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = J * 16 + kk * 4 + r;
        acc[r] = j <= i ? acc[r] * expf((float)(lam_i - lam[j])) : 0.f;
      }
    }
    p[J] = acc;
  }
  __syncthreads();                  // the keys have been read
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int e = tid + j * kThreads;
    *(f32x4*)(K + e / (kVB / 4) * VS + e % (kVB / 4) * 4) = sreg[j];
  }
  __syncthreads();
  const float from_state = expf((float)lam_i);
  const float skip = op.skip ? op.skip[head] : 0.f;
#pragma unroll 1
  for (int vt = 0; vt < VT; ++vt) {
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < NB; ++s)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(K[(s * 16 + kk * 4 + e) * VS + vt * 16 + l16], q[s][e], acc, 0, 0, 0);
#pragma unroll
    for (int r = 0; r < 4; ++r) acc[r] *= from_state;
#pragma unroll
    for (int J = 0; J < kC / 16; ++J)
      if (J <= wave) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          acc = __builtin_amdgcn_mfma_f32_16x16x4f32(V[(J * 16 + kk * 4 + r) * VS + vt * 16 + l16], p[J][r], acc, 0, 0, 0);
      }
    // lane (l16, kk) holds token i, columns vt * 16 + 4 kk + r
    const int col = vt * 16 + kk * 4;
    if (i < n && v0 + col < vdim) {
      if (op.skip) {
        const f32x4 x = chunk_act(op, chunk_load(op, vb, i, n, col, vdim - v0));
#pragma unroll
        for (int r = 0; r < 4; ++r) acc[r] = fmaf(skip, x[r], acc[r]);
      }
      float* dst = o + ((int64_t)(tok0 + i) * op.heads + head) * vdim + v0 + col;
      if (op.vec) {
        *(f32x4*)dst = acc;
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (v0 + col + r < vdim) dst[r] = acc[r];
      }
    }
  }
}

// A row in `groups` equal parts (one workgroup a part), each divided by its own root mean square:
//   gate first:  u = o * act(g);  z = scale * w * u / sqrt(mean(u^2) + eps)
//   gate last:   z = scale * w * o / sqrt(mean(o^2) + eps) * act(g)
// act: the sigmoid (gate_kind 0) or g * sigmoid(g) (1).  Parts of up to KEEP * kThreads numbers stay in registers.
template <typename T, int KEEP>
__global__ __launch_bounds__(kThreads) void group_norm_gate_kernel(const float* __restrict__ o, const float* __restrict__ w,
                                                                   const float* __restrict__ gate, int64_t gate_stride,
                                                                   T* __restrict__ z, int64_t z_stride, int width, int part, float eps,
                                                                   int gate_kind, int gate_first, float scale) {
  __shared__ float red[kThreads / TL_WAVE];
  const int t = blockIdx.x, c0 = blockIdx.y * part;
  const float* src = o + (int64_t)t * width + c0;
  const float* gp = gate + (int64_t)t * gate_stride + c0;
  const float* wp = w + c0;
  T* dst = z + (int64_t)t * z_stride + c0;
  auto act = [&](float g) {
    const float s = 1.f / (1.f + expf(-g));
    return gate_kind ? g * s : s;
  };
  float ss = 0.f;
  if (part <= KEEP * kThreads) {
    float u[KEEP], f[KEEP], wv[KEEP];
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
      const int j = threadIdx.x + i * kThreads;
      const bool in = j < part;
      u[i] = in ? src[j] : 0.f;
      f[i] = in ? gp[j] : 0.f;
      wv[i] = in ? wp[j] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
      f[i] = act(f[i]);
      if (gate_first) {
        u[i] *= f[i];
        f[i] = 1.f;
      }
      ss += u[i] * u[i];
    }
    ss = block_sum<kThreads / TL_WAVE>(ss, red);
    const float r = scale / sqrtf(ss / (float)part + eps);
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
      const int j = threadIdx.x + i * kThreads;
      if (j < part) dst[j] = from_f32<T>(u[i] * r * wv[i] * f[i]);
    }
    return;
  }
  for (int j = threadIdx.x; j < part; j += kThreads) {
    const float u = gate_first ? src[j] * act(gp[j]) : src[j];
    ss += u * u;
  }
  ss = block_sum<kThreads / TL_WAVE>(ss, red);
  const float r = scale / sqrtf(ss / (float)part + eps);
  for (int j = threadIdx.x; j < part; j += kThreads) dst[j] = from_f32<T>(src[j] * act(gp[j]) * r * wp[j]);
}

}  // namespace

extern "C" {

constexpr int kConvRun = 8;       // tokens of a run (tl_conv_run)

// single: every request brings one token (row i is request i's), no tile lists; else the lists cut every request's tokens
// into runs of at most tl_conv_run() and conv_state_update has to follow.
int tl_ssd_prepare(const float* p, int64_t p_stride, int conv_off, int dt_off, const float* conv_w, const float* conv_b,
                   const float* a_log, const float* dt_bias, float* state, int64_t state_stride, int64_t saved_off,
                   const int32_t* cu, const int32_t* slots, float* x, int64_t x_stride, int dt_col, int a_col, int channels,
                   int heads, int taps, int single, const int32_t* tile_req, const int32_t* tile_tok0,
                   const int32_t* tile_ntok, int n_tiles, hipStream_t stream) {
  if (n_tiles <= 0) return TL_OK;
  if (channels <= 0 || heads <= 0 || taps < 1 || taps > kConvMaxTaps || !p || !conv_w || !a_log || !dt_bias ||
      (taps > 1 && !state) || !slots || !x || dt_col < channels || a_col < dt_col + heads || x_stride < a_col + heads ||
      (!single && (!tile_req || !tile_tok0 || !tile_ntok || !cu)))
    return TL_ERR_ARG;
  const ShortConv conv{conv_w, taps, single, state, state_stride, saved_off, cu, slots};
  dim3 g(n_tiles, (channels + heads + kThreads - 1) / kThreads), b(kThreads);
#define TL_SSD(RUN, TAPS)                                                                                                \
  hipLaunchKernelGGL((ssd_prepare_kernel<RUN, TAPS>), g, b, 0, stream, p, p_stride, conv_off, dt_off, conv_b, a_log,      \
                     dt_bias, conv, x, x_stride, dt_col, a_col, channels, heads, tile_req, tile_tok0, tile_ntok)
  if (single && taps <= 4) TL_SSD(1, 4);
  else if (single) TL_SSD(1, kConvMaxTaps);
  else if (taps <= 4) TL_SSD(kConvRun, 4);
  else TL_SSD(kConvRun, kConvMaxTaps);
#undef TL_SSD
  return tl_launch_status();
}

// decode != 0: every request brings at most one token (vdim a multiple of 4 up to 256, 16-byte aligned state rows).
// c_off negative: a factor of 1; a_off: columns of ln a, negative: the decay is decay[head].
int tl_linear_recurrence(const float* x, int64_t x_stride, int q_off, int k_off, int v_off, int c_off, int a_off,
                         const float* decay, const float* skip, float* state, int64_t state_stride, const int32_t* cu,
                         const int32_t* slots, float* o, int n_requests, int heads, int groups, int dim, int vdim,
                         int act_silu, int decode, hipStream_t stream) {
  if (n_requests <= 0) return TL_OK;
  if (heads <= 0 || heads > 65535 || n_requests > 65535 || groups <= 0 || heads % groups || dim <= 0 || dim > 256 ||
      vdim <= 0 || !x || !state || !cu || !slots || !o || q_off < 0 || k_off < 0 || v_off < 0 || (a_off < 0 && !decay) ||
      state_stride < (int64_t)heads * dim * vdim)
    return TL_ERR_ARG;
  const Operands op{x, x_stride, q_off, k_off, v_off, c_off, a_off, decay, skip, heads, groups, dim, vdim, act_silu, 0};
  if (decode) {
    if (vdim % 4 || vdim > kThreads || state_stride % 4 || ((uintptr_t)state & 15)) return TL_ERR_ARG;
    const int NS = kThreads / (vdim / 4), rows = (dim + NS - 1) / NS;
    dim3 g(n_requests, heads), b(kThreads);
#define TL_LR_DEC(R) \
  hipLaunchKernelGGL(linear_recurrence_decode_kernel<R>, g, b, 0, stream, op, state, state_stride, cu, slots, o)
    if (rows <= 1) TL_LR_DEC(1);
    else if (rows <= 2) TL_LR_DEC(2);
    else if (rows <= 4) TL_LR_DEC(4);
    else if (rows <= 8) TL_LR_DEC(8);
    else if (rows <= 16) TL_LR_DEC(16);
    else if (rows <= 32) TL_LR_DEC(32);
    else TL_LR_DEC(64);
#undef TL_LR_DEC
    return tl_launch_status();
  }
  int P = 1;
  while (P * kSlice < dim) P *= 2;
  const int EC = kThreads / P;
  dim3 g((vdim + EC - 1) / EC, heads, n_requests), b(kThreads);
#define TL_LR(PP)                                                                                                   \
  case PP:                                                                                                          \
    hipLaunchKernelGGL(linear_recurrence_kernel<PP>, g, b, 0, stream, op, state, state_stride, cu, slots, o);       \
    break;
  switch (P) {
    TL_LR(1) TL_LR(2) TL_LR(4) TL_LR(8) TL_LR(16) TL_LR(32)
    default: return TL_ERR_ARG;
  }
#undef TL_LR
  return tl_launch_status();
}

// The same for steps that bring many tokens of a request: tile_tok0 / tile_ntok [n_tiles] list every request's tokens of
// the step in chunks of up to 64, request after request (0 tokens: padding); U [n_tiles, heads, dim, vdim] and decays
// [n_tiles, heads] are scratch.
int tl_linear_recurrence_chunks(const float* x, int64_t x_stride, int q_off, int k_off, int v_off, int c_off, int a_off,
                                const float* decay, const float* skip, float* state, int64_t state_stride,
                                const int32_t* cu, const int32_t* slots, const int32_t* tile_tok0, const int32_t* tile_ntok,
                                float* U, float* decays, float* o, int n_tiles, int n_requests, int heads, int groups, int dim,
                                int vdim, int act_silu, hipStream_t stream) {
  if (n_requests <= 0 || n_tiles <= 0) return TL_OK;
  if (heads <= 0 || heads > 65535 || n_requests > 65535 || groups <= 0 || heads % groups || dim <= 0 || dim > 256 ||
      vdim <= 0 || (vdim + kVB - 1) / kVB > 65535 || !x || !state || !cu || !slots || !o || q_off < 0 || k_off < 0 ||
      v_off < 0 || (a_off < 0 && !decay) || state_stride < (int64_t)heads * dim * vdim || !tile_tok0 || !tile_ntok || !U || !decays)
    return TL_ERR_ARG;
  const int vec4 = !((dim | vdim | q_off | k_off | v_off | (int)(x_stride & 3)) & 3) &&
                   !(((uintptr_t)x | (uintptr_t)U | (uintptr_t)o) & 15);
  const Operands op{x, x_stride, q_off, k_off, v_off, c_off, a_off, decay, skip, heads, groups, dim, vdim, act_silu, vec4};
  const ChunkTiles tiles{tile_tok0, tile_ntok};
  dim3 g(n_tiles, heads, (vdim + kVB - 1) / kVB), b(kThreads);
  const int size = dim * vdim;
  const bool vec = size % 4 == 0 && state_stride % 4 == 0 && !(((uintptr_t)state | (uintptr_t)U) & 15);
  dim3 gs((size / (vec ? 4 : 1) + kThreads - 1) / kThreads, heads, n_requests);
#define TL_CHUNKS(NB)                                                                                                     \
  {                                                                                                                       \
    constexpr int lds_u = (kC * (NB * 16 + 16) + kC * (kVB + 16)) * (int)sizeof(float);                                   \
    constexpr int area = kC * (NB * 16 + 4) > NB * 16 * (kVB + 4) ? kC * (NB * 16 + 4) : NB * 16 * (kVB + 4);             \
    constexpr int lds_o = (area + kC * (kVB + 4)) * (int)sizeof(float);                                                   \
    static bool configured = false;                                                                                       \
    if (!configured) {                                                                                                    \
      if (hipFuncSetAttribute((const void*)chunk_update_kernel<NB>, hipFuncAttributeMaxDynamicSharedMemorySize, lds_u) !=  \
              hipSuccess ||                                                                                               \
          hipFuncSetAttribute((const void*)chunk_output_kernel<NB>, hipFuncAttributeMaxDynamicSharedMemorySize, lds_o) !=  \
              hipSuccess)                                                                                                 \
        return TL_ERR_LAUNCH;                                                                                             \
      configured = true;                                                                                                  \
    }                                                                                                                     \
    hipLaunchKernelGGL(chunk_update_kernel<NB>, g, b, lds_u, stream, op, tiles, U, decays);                               \
    if (vec)                                                                                                              \
      hipLaunchKernelGGL(chunk_scan_kernel<4>, gs, b, 0, stream, U, decays, state, state_stride, cu, slots, heads, size); \
    else                                                                                                                  \
      hipLaunchKernelGGL(chunk_scan_kernel<1>, gs, b, 0, stream, U, decays, state, state_stride, cu, slots, heads, size); \
    hipLaunchKernelGGL(chunk_output_kernel<NB>, g, b, lds_o, stream, op, tiles, U, o);                                    \
  }
  if (dim <= 16) TL_CHUNKS(1)
  else if (dim <= 32) TL_CHUNKS(2)
  else if (dim <= 64) TL_CHUNKS(4)
  else if (dim <= 128) TL_CHUNKS(8)
  else TL_CHUNKS(16)
#undef TL_CHUNKS
  return tl_launch_status();
}

// o: float32 [n_tokens, width]; w: float32 [width]; gate: float32, rows gate_stride apart; z: [n_tokens, width] in dtype, rows z_stride apart.
int tl_group_norm_gate(const float* o, const float* w, const float* gate, int64_t gate_stride, void* z,
                       int64_t z_stride, int n_tokens, int width, int groups, float eps, int gate_kind, int gate_first, float scale, int dtype,
                       hipStream_t stream) {
  if (n_tokens <= 0) return TL_OK;
  if (width <= 0 || groups <= 0 || groups > 65535 || width % groups || gate_kind < 0 || gate_kind > 1 || !o || !w || !gate || !z)
    return TL_ERR_ARG;
  const int part = width / groups;
  dim3 g(n_tokens, groups), b(kThreads);
#define TL_GNG(T, K)                                                                                                     \
  hipLaunchKernelGGL((group_norm_gate_kernel<T, K>), g, b, 0, stream, o, w, gate, gate_stride, (T*)z, z_stride, width, part, eps, \
                     gate_kind, gate_first, scale)
#define TL_GNG_K(T)                         \
  if (part <= 2 * kThreads) TL_GNG(T, 2);   \
  else if (part <= 8 * kThreads) TL_GNG(T, 8); \
  else TL_GNG(T, 24);
  if (dtype == 0) { TL_GNG_K(float) }
  else if (dtype == 1) { TL_GNG_K(bf16_t) }
  else return TL_ERR_ARG;
#undef TL_GNG_K
#undef TL_GNG
  return tl_launch_status();
}

}  // extern "C"
