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
constexpr int kMaxTaps = 16;

__device__ __forceinline__ float silu(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float softplus(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// Row t of p: the convolutions' inputs from column conv_off (`channels` of them), step sizes' pre-activations from
// dt_off (one per head).  Row t of x: [silu(conv + bias): channels | c = softplus(dt + dt_bias): heads, from column
// dt_col | a = exp(-exp(A_log) c): heads, from a_col].  A request's inputs ahead of its first token of the step come
// from its state row at saved_off, [channel][taps - 1], oldest first.  save_single: no request brings more than one
// token, and the thread that has read a channel's saved inputs leaves the next token's in their place.
__global__ __launch_bounds__(kThreads) void ssd_prepare_kernel(
    const float* __restrict__ p, int64_t p_stride, int conv_off, int dt_off, const float* __restrict__ conv_w,
    const float* __restrict__ conv_b, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
    float* __restrict__ state, int64_t state_stride, int64_t saved_off, const int32_t* __restrict__ req_of_token,
    const int32_t* __restrict__ cu, const int32_t* __restrict__ slots, float* __restrict__ x, int64_t x_stride, int dt_col,
    int a_col, int channels, int heads, int taps, int save_single) {
  const int t = blockIdx.x;
  const int c = blockIdx.y * kThreads + threadIdx.x;
  if (c >= channels) {
    const int h = c - channels;
    if (h < heads) {
      const float dt = softplus(p[(int64_t)t * p_stride + dt_off + h] + dt_bias[h]);
      x[(int64_t)t * x_stride + dt_col + h] = dt;
      x[(int64_t)t * x_stride + a_col + h] = expf(-expf(a_log[h]) * dt);
    }
    return;
  }
  const int r = req_of_token[t];
  const int t0 = cu[r], n = t - t0;          // (a padding row of a captured step: n beyond the request's tokens)
  float* saved = state + (int64_t)slots[r] * state_stride + saved_off + (int64_t)c * (taps - 1);
  const float* w = conv_w + (int64_t)c * taps;
  const float* col = p + conv_off + c;
  float acc = conv_b ? conv_b[c] : 0.f;
  const bool keep = save_single && t == t0 && cu[r + 1] == t + 1;
  auto input = [&](int j) {                  // tap j meets input n - (taps - 1) + j
    const int m = n - (taps - 1) + j;
    return m >= 0 ? col[(int64_t)(t0 + m) * p_stride] : saved[(taps - 1) + m];
  };
  if (taps <= 4) {
    float in[4], wt[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      in[j] = j < taps ? input(j) : 0.f;
      wt[j] = j < taps ? w[j] : 0.f;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) acc = fmaf(wt[j], in[j], acc);
    if (keep) {
#pragma unroll
      for (int j = 1; j < 4; ++j)
        if (j < taps) saved[j - 1] = in[j];
    }
  } else {
    float in[kMaxTaps];
#pragma unroll
    for (int j = 0; j < kMaxTaps; ++j) {
      in[j] = j < taps ? input(j) : 0.f;
      if (j < taps) acc = fmaf(w[j], in[j], acc);
    }
    if (keep) {
#pragma unroll
      for (int j = 1; j < kMaxTaps; ++j)
        if (j < taps) saved[j - 1] = in[j];
    }
  }
  x[(int64_t)t * x_stride + c] = silu(acc);
}

// What a recurrence reads: rows x[t] with q and k (groups x dim numbers, from q_off and k_off), v (heads x vdim, from
// v_off); c and a per head from c_off and a_off, or, where these are negative, 1 and decay[h]; silu: q, k and v are
// pre-activations.
struct Operands {
  const float* x;
  int64_t x_stride;
  int q_off, k_off, v_off, c_off, a_off;
  const float* decay;
  const float* skip;      // D per head, or null
  int heads, groups, dim, vdim, silu;
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
      pa = op.a_off < 0 ? decay : row[op.a_off];
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
  const float a = op.a_off < 0 ? op.decay[head] : row[op.a_off + head];
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

// A row in `groups` equal parts (one workgroup a part), each divided by its own root mean square:
//   gate first:  u = o * act(g);  z = scale * w * u / sqrt(mean(u^2) + eps)
//   gate last:   z = scale * w * o / sqrt(mean(o^2) + eps) * act(g)
// act: the sigmoid (gate_kind 0) or g * sigmoid(g) (1).  Parts of up to KEEP * kThreads numbers stay in registers.
template <typename T, int KEEP>
__global__ __launch_bounds__(kThreads) void group_norm_gate_kernel(const float* __restrict__ o, const float* __restrict__ w,
                                                                   const float* __restrict__ gate, int64_t gate_stride,
                                                                   T* __restrict__ z, int width, int part, float eps,
                                                                   int gate_kind, int gate_first, float scale) {
  __shared__ float red[kThreads / TL_WAVE];
  const int t = blockIdx.x, c0 = blockIdx.y * part;
  const float* src = o + (int64_t)t * width + c0;
  const float* gp = gate + (int64_t)t * gate_stride + c0;
  const float* wp = w + c0;
  T* dst = z + (int64_t)t * width + c0;
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

int tl_ssd_prepare(const float* p, int64_t p_stride, int conv_off, int dt_off, const float* conv_w, const float* conv_b,
                   const float* a_log, const float* dt_bias, float* state, int64_t state_stride, int64_t saved_off,
                   const int32_t* req_of_token, const int32_t* cu, const int32_t* slots, float* x, int64_t x_stride,
                   int dt_col, int a_col, int n_tokens, int channels, int heads, int taps, int save_single,
                   hipStream_t stream) {
  if (n_tokens <= 0) return TL_OK;
  if (channels <= 0 || heads <= 0 || taps < 1 || taps > kMaxTaps || !p || !conv_w || !a_log || !dt_bias || !state ||
      !req_of_token || !cu || !slots || !x || dt_col < channels || a_col < dt_col + heads || x_stride < a_col + heads)
    return TL_ERR_ARG;
  dim3 g(n_tokens, (channels + heads + kThreads - 1) / kThreads), b(kThreads);
  hipLaunchKernelGGL(ssd_prepare_kernel, g, b, 0, stream, p, p_stride, conv_off, dt_off, conv_w, conv_b, a_log, dt_bias,
                     state, state_stride, saved_off, req_of_token, cu, slots, x, x_stride, dt_col, a_col, channels, heads,
                     taps, save_single);
  return tl_launch_status();
}

// decode != 0: every request brings at most one token (vdim a multiple of 4 up to 256, 16-byte aligned state rows).
// c_off / a_off negative: factor 1 / decay[head].
int tl_linear_recurrence(const float* x, int64_t x_stride, int q_off, int k_off, int v_off, int c_off, int a_off,
                         const float* decay, const float* skip, float* state, int64_t state_stride, const int32_t* cu,
                         const int32_t* slots, float* o, int n_requests, int heads, int groups, int dim, int vdim,
                         int act_silu, int decode, hipStream_t stream) {
  if (n_requests <= 0) return TL_OK;
  if (heads <= 0 || heads > 65535 || n_requests > 65535 || groups <= 0 || heads % groups || dim <= 0 || dim > 256 ||
      vdim <= 0 || !x || !state || !cu || !slots || !o || q_off < 0 || k_off < 0 || v_off < 0 || (a_off < 0 && !decay) ||
      state_stride < (int64_t)heads * dim * vdim)
    return TL_ERR_ARG;
  const Operands op{x, x_stride, q_off, k_off, v_off, c_off, a_off, decay, skip, heads, groups, dim, vdim, act_silu};
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

// o: float32 [n_tokens, width]; w: float32 [width]; gate: float32, rows gate_stride apart; z: [n_tokens, width] in dtype.
int tl_group_norm_gate(const float* o, const float* w, const float* gate, int64_t gate_stride, void* z, int n_tokens,
                       int width, int groups, float eps, int gate_kind, int gate_first, float scale, int dtype,
                       hipStream_t stream) {
  if (n_tokens <= 0) return TL_OK;
  if (width <= 0 || groups <= 0 || groups > 65535 || width % groups || gate_kind < 0 || gate_kind > 1 || !o || !w || !gate || !z)
    return TL_ERR_ARG;
  const int part = width / groups;
  dim3 g(n_tokens, groups), b(kThreads);
#define TL_GNG(T, K)                                                                                                     \
  hipLaunchKernelGGL((group_norm_gate_kernel<T, K>), g, b, 0, stream, o, w, gate, gate_stride, (T*)z, width, part, eps,   \
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
