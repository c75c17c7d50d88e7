// Between the query/key product and the attention kernel, for attention whose queries and keys carry a
// bias, are rotated on part of their dims and then scaled to unit root mean square, and whose values
// may be the keys themselves as projected; and behind the attention kernel, a sigmoid gate per head.
//
// Everything here is float32 arithmetic on the float32 result of the product; what leaves is rounded
// once to the engine's element type (queries, cached keys and values).
#include "common.h"

namespace {

// One wave per (token, head); heads 0 .. nq - 1 are queries, nq .. nq + nkv - 1 keys.
//   a = p[t, head, :] + bias[head, :]
//   keys with values_are_keys: v_cache[slot] = a           (before rotation and norm)
//   values otherwise (v_off >= 0): v_cache[slot] = p[t, v_off + kv head, :]
//   a <- rotate(a) on the first `rot` dims, pair i = (2i, 2i + 1) or (i, i + rot / 2), angle table row of the position
//   a <- a / sqrt(mean(a^2) + eps)   if unit_norm
//   queries -> q_out[t, head, :], keys -> k_cache[slot]    (a negative slot stores nothing)
template <typename T>
__global__ __launch_bounds__(TL_WAVE) void qk_prepare_kernel(
    const float* __restrict__ p, int64_t p_stride, const float* __restrict__ bias, const int32_t* __restrict__ positions,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, const int32_t* __restrict__ slot_mapping,
    T* __restrict__ q_out, int64_t q_stride, T* __restrict__ k_cache, T* __restrict__ v_cache, int nq, int nkv, int hd,
    int rot, int interleaved, int unit_norm, float eps, int values_are_keys, int v_off, int block_size) {
  const int t = blockIdx.x, head = blockIdx.y, lane = threadIdx.x;
  const bool is_key = head >= nq;
  const int slot = slot_mapping ? slot_mapping[t] : -1;
  if (is_key && slot < 0) return;
  const float* src = p + (int64_t)t * p_stride + (int64_t)head * hd;
  const float* bs = bias ? bias + (int64_t)head * hd : nullptr;
  const int half = rot / 2, pairs = hd / 2;       // hd is even
  const int pos = positions[t];
  const float* cs = cos_t ? cos_t + (int64_t)pos * half : nullptr;
  const float* sn = sin_t ? sin_t + (int64_t)pos * half : nullptr;
  int64_t cache_row = 0;
  if (is_key) cache_row = (((int64_t)(slot / block_size) * nkv + (head - nq)) * block_size + slot % block_size) * hd;
  constexpr int kPairs = 2;                        // head sizes up to 256: at most 128 pairs, two a lane
  float ra[kPairs], rb[kPairs];
  int ia[kPairs], ib[kPairs];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < kPairs; ++i) {
    const int j = lane + i * TL_WAVE;
    ra[i] = rb[i] = 0.f;
    ia[i] = ib[i] = 0;
    if (j < pairs) {
      if (j < half) {
        ia[i] = interleaved ? 2 * j : j;
        ib[i] = interleaved ? 2 * j + 1 : j + half;
      } else {
        ia[i] = rot + 2 * (j - half);
        ib[i] = ia[i] + 1;
      }
      float a = src[ia[i]], b = src[ib[i]];
      if (bs) {
        a += bs[ia[i]];
        b += bs[ib[i]];
      }
      if (is_key && values_are_keys) {
        v_cache[cache_row + ia[i]] = from_f32<T>(a);
        v_cache[cache_row + ib[i]] = from_f32<T>(b);
      }
      if (j < half) {
        const float c = cs[j], s = sn[j];
        ra[i] = c * a - s * b;
        rb[i] = s * a + c * b;
      } else {
        ra[i] = a;
        rb[i] = b;
      }
      ss += ra[i] * ra[i] + rb[i] * rb[i];
    }
  }
  float r = 1.f;
  if (unit_norm) r = 1.f / sqrtf(wave_sum(ss) / (float)hd + eps);
  T* dst = is_key ? k_cache + cache_row : q_out + (int64_t)t * q_stride + (int64_t)head * hd;
#pragma unroll
  for (int i = 0; i < kPairs; ++i) {
    const int j = lane + i * TL_WAVE;
    if (j < pairs) {
      dst[ia[i]] = from_f32<T>(ra[i] * r);
      dst[ib[i]] = from_f32<T>(rb[i] * r);
    }
  }
  if (is_key && !values_are_keys && v_off >= 0) {
    const float* vs = p + (int64_t)t * p_stride + v_off + (int64_t)(head - nq) * hd;
    for (int d = lane; d < hd; d += TL_WAVE) v_cache[cache_row + d] = from_f32<T>(vs[d]);
  }
}

// z[t, h, :] = a[t, h, :] * sigmoid(g[t, h]) * scale; one thread an element.
template <typename T>
__global__ void head_gate_kernel(const T* __restrict__ a, int64_t a_stride, const float* __restrict__ g, int64_t g_stride,
                                 T* __restrict__ z, int64_t z_stride, int64_t total, int heads, int hd, float scale) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  const int width = heads * hd;
  const int64_t t = i / width;
  const int c = (int)(i - t * width);
  const float gate = 1.f / (1.f + expf(-g[t * g_stride + c / hd]));
  z[t * z_stride + c] = from_f32<T>(to_f32(a[t * a_stride + c]) * gate * scale);
}

// The general form of the step between the product that reads the mixer's input and the attention kernel: the
// workgroups (t, 0 .. gridDim.y - 1) share a token's units and values out, a wave a unit at a time (steps of few
// tokens get many workgroups a token; each forms the sums of the whole-projection norm for itself).  Row t of p (float32) holds q as `q_units` units of `dim` numbers, then k as
// `k_units` units, then v as `nkv` heads of `vdim` numbers (from column v_off); a unit is one score map of one
// head, unit u = head * maps + map.  In this order, each step an option:
//   a = p + bias                                      (bias over [q | k | v], or null)
//   a <- a / sqrt(mean over ALL of the token's q (or k) numbers of a^2 + eps) * norm_w    (whole_norm; norm_w over [q | k])
//   a <- rotate(a) on the first `rot` dims of every unit, pair (i, i + rot/2) or (2i, 2i + 1)
//   a <- a / sqrt(mean over the unit of a^2 + eps)     (unit_norm)
//   q <- q * (1 + temp_coef * ln(floor((pos + 1) / temp_every) + 1))                       (temp_every > 0)
// Queries of map m leave as q_out[m][t][head][0 .. D), keys go to k_cache[m] and values to v_cache at the
// token's slot, pages [blocks, nkv, block_size, D]; D >= dim, vdim, and what lies beyond dim (vdim) is written as
// zeros, so that an attention kernel over heads of D computes the same scores and leaves the values' columns first.
// A negative slot (padding) stores nothing.
constexpr int kPrepThreads = 256, kPrepWaves = kPrepThreads / TL_WAVE, kPrepPerLane = 4;     // units of up to 256
template <typename T>
__global__ __launch_bounds__(kPrepThreads) void attn_prepare_kernel(
    const float* __restrict__ p, int64_t p_stride, const float* __restrict__ bias, const float* __restrict__ norm_w,
    const int32_t* __restrict__ positions, const float* __restrict__ cos_t, const float* __restrict__ sin_t,
    const int32_t* __restrict__ slot_mapping, T* __restrict__ q_out, int64_t q_stride, int64_t q_map_stride,
    T* __restrict__ k_cache0, T* __restrict__ k_cache1, T* __restrict__ v_cache, int heads, int nkv, int maps, int dim,
    int vdim, int D, int v_off, int rot, int interleaved, int whole_norm, int unit_norm, float eps, float temp_coef,
    int temp_every, int block_size) {
  __shared__ float red[kPrepWaves];
  const int t = blockIdx.x, tid = threadIdx.x, wave = tid / TL_WAVE, lane = tid % TL_WAVE;
  const float* row = p + (int64_t)t * p_stride;
  const int q_units = heads * maps, k_units = nkv * maps;
  const int q_size = q_units * dim, k_size = k_units * dim;
  const int pos = positions[t];
  const int slot = slot_mapping ? slot_mapping[t] : -1;
  float rq = 1.f, rk = 1.f;
  if (whole_norm) {
    float sq = 0.f, sk = 0.f;
    for (int c = tid; c < q_size; c += kPrepThreads) {
      const float a = row[c] + (bias ? bias[c] : 0.f);
      sq += a * a;
    }
    for (int c = q_size + tid; c < q_size + k_size; c += kPrepThreads) {
      const float a = row[c] + (bias ? bias[c] : 0.f);
      sk += a * a;
    }
    rq = 1.f / sqrtf(block_sum<kPrepWaves>(sq, red) / (float)q_size + eps);
    rk = 1.f / sqrtf(block_sum<kPrepWaves>(sk, red) / (float)k_size + eps);
  }
  float temp = 1.f;
  if (temp_every > 0) temp = 1.f + temp_coef * logf((float)((pos + 1) / temp_every) + 1.f);
  const int half = rot / 2;
  const float* cs = rot ? cos_t + (int64_t)pos * half : nullptr;
  const float* sn = rot ? sin_t + (int64_t)pos * half : nullptr;
  const int64_t page_row = slot >= 0 ? (int64_t)(slot / block_size) * nkv * block_size + slot % block_size : 0;
  for (int u = blockIdx.y * kPrepWaves + wave; u < q_units + k_units; u += gridDim.y * kPrepWaves) {
    const bool is_key = u >= q_units;
    if (is_key && slot < 0) continue;
    const int uu = is_key ? u - q_units : u;
    const int head = uu / maps, map = uu % maps;
    const int c0 = (is_key ? q_size : 0) + uu * dim;        // the unit's first column in p, bias and norm_w
    const float r = is_key ? rk : rq;
    auto value = [&](int d) {
      float a = row[c0 + d] + (bias ? bias[c0 + d] : 0.f);
      if (whole_norm) a = a * r * norm_w[c0 + d];
      return a;
    };
    float out[kPrepPerLane];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < kPrepPerLane; ++i) {
      const int d = lane + i * TL_WAVE;
      out[i] = 0.f;
      if (d < dim) {
        float a = value(d);
        if (d < rot) {
          int j, partner;
          bool first;
          if (interleaved) {
            j = d / 2;
            first = (d & 1) == 0;
            partner = first ? d + 1 : d - 1;
          } else {
            first = d < half;
            j = first ? d : d - half;
            partner = first ? d + half : d - half;
          }
          const float b = value(partner);
          a = first ? a * cs[j] - b * sn[j] : a * cs[j] + b * sn[j];
        }
        out[i] = a;
        ss += a * a;
      }
    }
    float f = is_key ? 1.f : temp;
    if (unit_norm) f *= 1.f / sqrtf(wave_sum(ss) / (float)dim + eps);
    T* dst;
    if (is_key)
      dst = (map == 0 ? k_cache0 : k_cache1) + (page_row + (int64_t)head * block_size) * D;
    else
      dst = q_out + (int64_t)map * q_map_stride + (int64_t)t * q_stride + (int64_t)head * D;
#pragma unroll
    for (int i = 0; i < kPrepPerLane; ++i) {
      const int d = lane + i * TL_WAVE;
      if (d < D) dst[d] = from_f32<T>(d < dim ? out[i] * f : 0.f);
    }
  }
  if (slot < 0) return;
  for (int c = blockIdx.y * kPrepThreads + tid; c < nkv * D; c += gridDim.y * kPrepThreads) {
    const int g = c / D, d = c - g * D;
    float a = 0.f;
    if (d < vdim) {
      const int col = v_off + g * vdim + d;
      a = row[col] + (bias ? bias[q_size + k_size + g * vdim + d] : 0.f);
    }
    v_cache[(page_row + (int64_t)g * block_size) * D + d] = from_f32<T>(a);
  }
}

// The same step for attention whose q, k and v run through a short causal convolution over time behind their biases, and
// whose queries and keys are normed per head ahead of the rotation:
//   a <- conv(p + bias) per channel;   q, k: a <- a / sqrt(mean over the head of a^2 + eps) * head_w (or no norm);
//   q, k: a <- rotate(a) on the first `rot` dims
// A wave takes one head of q, k or v for a run of up to RUN consecutive tokens of a request (its inputs are requested once,
// and the run's sums and rotations have each other's latencies to hide behind).  head_w: `dim` weights for queries, then
// `dim` for keys.  Channels count [q | k | v], as the columns of p do.
template <typename T, int RUN, int PER, int TAPS>
__global__ __launch_bounds__(kPrepThreads) void conv_attn_prepare_kernel(
    const float* __restrict__ p, int64_t p_stride, const float* __restrict__ bias, const float* __restrict__ head_w,
    const int32_t* __restrict__ positions, const float* __restrict__ cos_t, const float* __restrict__ sin_t,
    const int32_t* __restrict__ slot_mapping, T* __restrict__ q_out, int64_t q_stride, T* __restrict__ k_cache,
    T* __restrict__ v_cache, int heads, int nkv, int dim, int vdim, int D, int rot, int interleaved, float eps,
    int block_size, const ShortConv conv, const int32_t* __restrict__ tile_req, const int32_t* __restrict__ tile_tok0,
    const int32_t* __restrict__ tile_ntok) {
  __shared__ float stage[kPrepWaves][RUN][PER * TL_WAVE];
  const int tile = blockIdx.x, wave = threadIdx.x / TL_WAVE, lane = threadIdx.x % TL_WAVE;
  const int u = blockIdx.y * kPrepWaves + wave;
  if (u >= heads + 2 * nkv) return;                // whole waves; the kernel has no workgroup barrier
  const int req = RUN == 1 ? tile : tile_req[tile], tok0 = RUN == 1 ? tile : tile_tok0[tile];
  const int n_tok = RUN == 1 ? 1 : tile_ntok[tile];
  if (n_tok <= 0) return;                          // a padding tile
  const int t0 = RUN == 1 ? tok0 : conv.cu[req];
  const bool is_q = u < heads, is_v = u >= heads + nkv;
  const int head = is_q ? u : is_v ? u - heads - nkv : u - heads;
  const int width = is_v ? vdim : dim;
  const int c0 = is_q ? head * dim : is_v ? (heads + nkv) * dim + head * vdim : (heads + head) * dim;
  float* saved_row = conv.taps > 1 ? conv.state + (int64_t)conv.slots[req] * conv.state_stride + conv.saved_off : nullptr;
  const int pos0 = positions[tok0];                // the tokens of a run are consecutive
  ConvRun<RUN, TAPS> cv[PER];
  float hw[PER], cs[RUN][PER], sn[RUN][PER];
  int partner[PER];
  bool first[PER];
  const int half = rot / 2;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int d = lane + i * TL_WAVE, ch = c0 + min(d, width - 1);
    cv[i].load(conv, p + ch, p_stride, t0, tok0 - t0, n_tok, ch, bias ? bias[ch] : 0.f,
               saved_row + (int64_t)ch * (conv.taps - 1));
    hw[i] = (head_w && !is_v) ? head_w[(is_q ? 0 : dim) + min(d, dim - 1)] : 1.f;
    partner[i] = d;
    first[i] = true;
    if (!is_v && d < rot) {
      int j;
      if (interleaved) {
        j = d / 2;
        first[i] = (d & 1) == 0;
        partner[i] = first[i] ? d + 1 : d - 1;
      } else {
        first[i] = d < half;
        j = first[i] ? d : d - half;
        partner[i] = first[i] ? d + half : d - half;
      }
#pragma unroll
      for (int tt = 0; tt < RUN; ++tt) {
        const int64_t row = (int64_t)(pos0 + min(tt, n_tok - 1)) * half;
        cs[tt][i] = cos_t[row + j];
        sn[tt][i] = sin_t[row + j];
      }
    }
  }
  float a[RUN][PER];
#pragma unroll
  for (int tt = 0; tt < RUN; ++tt)
#pragma unroll
    for (int i = 0; i < PER; ++i) a[tt][i] = lane + i * TL_WAVE < width ? cv[i].value(tt) : 0.f;
  if (RUN == 1 && conv.taps > 1) {
#pragma unroll
    for (int i = 0; i < PER; ++i)
      if (lane + i * TL_WAVE < width) cv[i].save_first(conv, saved_row + (int64_t)(c0 + lane + i * TL_WAVE) * (conv.taps - 1));
  }
  if (!is_v) {
    if (head_w) {
#pragma unroll
      for (int tt = 0; tt < RUN; ++tt) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < PER; ++i) ss += a[tt][i] * a[tt][i];
        const float r = 1.f / sqrtf(wave_sum(ss) / (float)dim + eps);
#pragma unroll
        for (int i = 0; i < PER; ++i) a[tt][i] *= r * hw[i];
      }
    }
    if (rot) {
#pragma unroll
      for (int tt = 0; tt < RUN; ++tt)
#pragma unroll
        for (int i = 0; i < PER; ++i) stage[wave][tt][lane + i * TL_WAVE] = a[tt][i];
      // one wave's LDS operations are carried out in order; the fences keep the compiler to it
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
      for (int tt = 0; tt < RUN; ++tt)
#pragma unroll
        for (int i = 0; i < PER; ++i)
          if (lane + i * TL_WAVE < rot) {
            const float b = stage[wave][tt][partner[i]];
            a[tt][i] = first[i] ? a[tt][i] * cs[tt][i] - b * sn[tt][i] : a[tt][i] * cs[tt][i] + b * sn[tt][i];
          }
    }
  }
#pragma unroll
  for (int tt = 0; tt < RUN; ++tt) {
    if (tt >= n_tok) break;
    T* dst;
    if (is_q) {
      dst = q_out + (int64_t)(tok0 + tt) * q_stride + (int64_t)head * D;
    } else {
      const int slot = slot_mapping ? slot_mapping[tok0 + tt] : -1;
      if (slot < 0) continue;
      dst = (is_v ? v_cache : k_cache) + (((int64_t)(slot / block_size) * nkv + head) * block_size + slot % block_size) * D;
    }
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int d = lane + i * TL_WAVE;
      if (d < D) dst[d] = from_f32<T>(a[tt][i]);      // zero beyond the head's numbers
    }
  }
}

// Behind the attention kernel, one wave per (token, head): the head's `vdim` values out of rows of D,
//   o = a0 - lambda * a1      (two maps; one map: o = a0)
//   o <- o / sqrt(mean(o^2) + eps)                (sub_norm)
//   o <- o * scale * gate,  gate = 1, sigmoid(g[t, head]) (gate_kind 1) or sigmoid(g[t, head * vdim + j]) (2)
// written side by side as z[t, head * vdim + j]; columns heads * vdim .. heads * vdim + tail - 1 of z become
// 1, 0, 0, ...: the one meets a bias stored as one more column of the output product's weight.
template <typename TA, typename T>
__global__ __launch_bounds__(TL_WAVE) void attn_finish_kernel(const TA* __restrict__ a0, const TA* __restrict__ a1,
                                                              int64_t a_stride, const float* __restrict__ g,
                                                              int64_t g_stride, T* __restrict__ z, int64_t z_stride,
                                                              int heads, int vdim, int D, float lambda, int sub_norm,
                                                              float eps, float scale, int gate_kind, int tail) {
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const TA* s0 = a0 + (int64_t)t * a_stride + (int64_t)h * D;
  const TA* s1 = a1 ? a1 + (int64_t)t * a_stride + (int64_t)h * D : nullptr;
  constexpr int kPer = 4;       // heads of up to 256 values
  float o[kPer];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < kPer; ++i) {
    const int j = lane + i * TL_WAVE;
    o[i] = 0.f;
    if (j < vdim) {
      o[i] = to_f32(s0[j]);
      if (s1) o[i] -= lambda * to_f32(s1[j]);
      ss += o[i] * o[i];
    }
  }
  float f = scale;
  if (sub_norm) f *= 1.f / sqrtf(wave_sum(ss) / (float)vdim + eps);
  if (gate_kind == 1) f *= 1.f / (1.f + expf(-g[(int64_t)t * g_stride + h]));
  T* dst = z + (int64_t)t * z_stride + (int64_t)h * vdim;
#pragma unroll
  for (int i = 0; i < kPer; ++i) {
    const int j = lane + i * TL_WAVE;
    if (j < vdim) {
      float v = o[i] * f;
      if (gate_kind == 2) v *= 1.f / (1.f + expf(-g[(int64_t)t * g_stride + (int64_t)h * vdim + j]));
      dst[j] = from_f32<T>(v);
    }
  }
  if (h == 0 && lane < tail) z[(int64_t)t * z_stride + (int64_t)heads * vdim + lane] = from_f32<T>(lane == 0 ? 1.f : 0.f);
}

}  // namespace

extern "C" {

// p: float32 [n_tokens, >= (nq + nkv) * hd] (row stride p_stride): query heads, then key heads; with
// values_are_keys == 0 and v_off >= 0 the value heads start at column v_off.  bias: [(nq + nkv) * hd] or null.
// cos_t / sin_t: [positions, rot / 2] (null when rot == 0).  Caches: [blocks, nkv, block_size, hd].
int tl_qk_prepare(const float* p, int64_t p_stride, const float* bias, const int32_t* positions, const float* cos_t,
                  const float* sin_t, const int32_t* slot_mapping, void* q_out, int64_t q_stride, void* k_cache,
                  void* v_cache, int n_tokens, int nq, int nkv, int hd, int rot, int interleaved, int unit_norm, float eps,
                  int values_are_keys, int v_off, int block_size, int dtype, hipStream_t stream) {
  if (n_tokens <= 0) return TL_OK;
  if (nq <= 0 || nkv < 0 || nq + nkv > 65535 || hd <= 0 || hd > 256 || (hd & 1) || rot < 0 || rot > hd || (rot & 1) ||
      block_size <= 0 || !p || !positions || !q_out)
    return TL_ERR_ARG;
  if (rot > 0 && (!cos_t || !sin_t)) return TL_ERR_ARG;
  if (slot_mapping && (!k_cache || !v_cache)) return TL_ERR_ARG;
  if (interleaved != 0 && interleaved != 1) return TL_ERR_ARG;
  dim3 g(n_tokens, nq + nkv), b(TL_WAVE);
  if (dtype == 0)
    hipLaunchKernelGGL(qk_prepare_kernel<float>, g, b, 0, stream, p, p_stride, bias, positions, cos_t, sin_t, slot_mapping,
                       (float*)q_out, q_stride, (float*)k_cache, (float*)v_cache, nq, nkv, hd, rot, interleaved, unit_norm,
                       eps, values_are_keys, v_off, block_size);
  else if (dtype == 1)
    hipLaunchKernelGGL(qk_prepare_kernel<bf16_t>, g, b, 0, stream, p, p_stride, bias, positions, cos_t, sin_t,
                       slot_mapping, (bf16_t*)q_out, q_stride, (bf16_t*)k_cache, (bf16_t*)v_cache, nq, nkv, hd, rot,
                       interleaved, unit_norm, eps, values_are_keys, v_off, block_size);
  else
    return TL_ERR_ARG;
  return tl_launch_status();
}

// a, z: [n_tokens, heads * hd] of the engine's type (z may be a); g: float32, one number per token and head.
int tl_head_gate(const void* a, int64_t a_stride, const float* g, int64_t g_stride, void* z, int64_t z_stride,
                 int n_tokens, int heads, int hd, float scale, int dtype, hipStream_t stream) {
  if (n_tokens <= 0) return TL_OK;
  if (heads <= 0 || hd <= 0 || !a || !g || !z) return TL_ERR_ARG;
  const int64_t total = (int64_t)n_tokens * heads * hd;
  dim3 grid((unsigned)ceil_div64(total, 256)), b(256);
  if (dtype == 0)
    hipLaunchKernelGGL(head_gate_kernel<float>, grid, b, 0, stream, (const float*)a, a_stride, g, g_stride, (float*)z,
                       z_stride, total, heads, hd, scale);
  else if (dtype == 1)
    hipLaunchKernelGGL(head_gate_kernel<bf16_t>, grid, b, 0, stream, (const bf16_t*)a, a_stride, g, g_stride,
                       (bf16_t*)z, z_stride, total, heads, hd, scale);
  else
    return TL_ERR_ARG;
  return tl_launch_status();
}

// p: float32 [n_tokens, p_stride]; bias [q | k | v] and norm_w [q | k] float32 or null; cos_t / sin_t [positions,
// rot / 2] (null when rot == 0); q_out: `maps` arrays of [n_tokens, q_stride], q_map_stride elements apart; caches
// [blocks, nkv, block_size, D], k_cache1 for the second map.
int tl_attn_prepare(const float* p, int64_t p_stride, const float* bias, const float* norm_w, const int32_t* positions,
                    const float* cos_t, const float* sin_t, const int32_t* slot_mapping, void* q_out, int64_t q_stride,
                    int64_t q_map_stride, void* k_cache0, void* k_cache1, void* v_cache, int n_tokens, int heads, int nkv,
                    int maps, int dim, int vdim, int D, int v_off, int rot, int interleaved, int whole_norm, int unit_norm,
                    float eps, float temp_coef, int temp_every, int block_size, int dtype, hipStream_t stream) {
  if (n_tokens <= 0) return TL_OK;
  if (heads <= 0 || nkv <= 0 || maps < 1 || maps > 2 || dim <= 0 || vdim <= 0 || D < dim || D < vdim ||
      D > kPrepPerLane * TL_WAVE || rot < 0 || rot > dim || (rot & 1) || block_size <= 0 || !p || !positions || !q_out ||
      v_off < (heads + nkv) * maps * dim || temp_every < 0)
    return TL_ERR_ARG;
  if (rot > 0 && (!cos_t || !sin_t)) return TL_ERR_ARG;
  if (whole_norm && !norm_w) return TL_ERR_ARG;
  if (slot_mapping && (!k_cache0 || !v_cache || (maps == 2 && !k_cache1))) return TL_ERR_ARG;
  if (interleaved != 0 && interleaved != 1) return TL_ERR_ARG;
  // about 256 workgroups in all where the units allow it, a wave with at least one unit
  const int units = (heads + nkv) * maps, most = (units + kPrepWaves - 1) / kPrepWaves;
  const int share = n_tokens >= 256 ? 1 : (256 / n_tokens < most ? 256 / n_tokens : most);
  dim3 g(n_tokens, share), b(kPrepThreads);
  if (dtype == 0)
    hipLaunchKernelGGL(attn_prepare_kernel<float>, g, b, 0, stream, p, p_stride, bias, norm_w, positions, cos_t, sin_t,
                       slot_mapping, (float*)q_out, q_stride, q_map_stride, (float*)k_cache0, (float*)k_cache1,
                       (float*)v_cache, heads, nkv, maps, dim, vdim, D, v_off, rot, interleaved, whole_norm, unit_norm, eps,
                       temp_coef, temp_every, block_size);
  else if (dtype == 1)
    hipLaunchKernelGGL(attn_prepare_kernel<bf16_t>, g, b, 0, stream, p, p_stride, bias, norm_w, positions, cos_t, sin_t,
                       slot_mapping, (bf16_t*)q_out, q_stride, q_map_stride, (bf16_t*)k_cache0, (bf16_t*)k_cache1,
                       (bf16_t*)v_cache, heads, nkv, maps, dim, vdim, D, v_off, rot, interleaved, whole_norm, unit_norm,
                       eps, temp_coef, temp_every, block_size);
  else
    return TL_ERR_ARG;
  return tl_launch_status();
}

// Tokens a wave of tl_conv_attn_prepare takes in a run (what its tile lists cut a request's tokens into).
constexpr int kConvRun = 8;
int tl_conv_run(void) { return kConvRun; }

// p: float32 [n_tokens, p_stride], columns [q | k | v]; bias (over them) and head_w [2 * dim] float32 or null; caches
// [blocks, nkv, block_size, D].  single: every request brings one token (row i is request i's), no tile lists; else the
// lists cut every request's tokens into runs of at most tl_conv_run() and conv_state_update has to follow.
int tl_conv_attn_prepare(const float* p, int64_t p_stride, const float* bias, const float* head_w, const int32_t* positions,
                         const float* cos_t, const float* sin_t, const int32_t* slot_mapping, void* q_out, int64_t q_stride,
                         void* k_cache, void* v_cache, int heads, int nkv, int dim, int vdim, int D, int rot, int interleaved,
                         float eps, int block_size, const float* conv_w, int taps, float* state, int64_t state_stride,
                         int64_t saved_off, const int32_t* cu, const int32_t* slots, int single, const int32_t* tile_req,
                         const int32_t* tile_tok0, const int32_t* tile_ntok, int n_tiles, int dtype, hipStream_t stream) {
  if (n_tiles <= 0) return TL_OK;
  if (heads <= 0 || nkv <= 0 || dim <= 0 || vdim <= 0 || D < dim || D < vdim || D > kPrepPerLane * TL_WAVE || rot < 0 ||
      rot > dim || (rot & 1) || block_size <= 0 || !p || !positions || !q_out || (rot > 0 && (!cos_t || !sin_t)) ||
      (slot_mapping && (!k_cache || !v_cache)) || (interleaved != 0 && interleaved != 1) || !conv_w || taps < 1 ||
      taps > kConvMaxTaps || (taps > 1 && !state) || !slots || (!single && (!tile_req || !tile_tok0 || !tile_ntok || !cu)) ||
      heads + 2 * nkv > 4 * 65535)
    return TL_ERR_ARG;
  const ShortConv conv{conv_w, taps, single, state, state_stride, saved_off, cu, slots};
  dim3 g(n_tiles, (heads + 2 * nkv + kPrepWaves - 1) / kPrepWaves), b(kPrepThreads);
#define TL_CAP(T, RUN, PER, TAPS)                                                                                        \
  hipLaunchKernelGGL((conv_attn_prepare_kernel<T, RUN, PER, TAPS>), g, b, 0, stream, p, p_stride, bias, head_w,           \
                     positions, cos_t, sin_t, slot_mapping, (T*)q_out, q_stride, (T*)k_cache, (T*)v_cache, heads, nkv,    \
                     dim, vdim, D, rot, interleaved, eps, block_size, conv, tile_req, tile_tok0, tile_ntok)
#define TL_CAP_TAPS(T, RUN, PER)                \
  if (taps <= 4) TL_CAP(T, RUN, PER, 4);        \
  else TL_CAP(T, RUN, PER, kConvMaxTaps);
#define TL_CAP_PER(T, RUN)                                \
  if (D <= TL_WAVE) { TL_CAP_TAPS(T, RUN, 1) }            \
  else if (D <= 2 * TL_WAVE) { TL_CAP_TAPS(T, RUN, 2) }   \
  else { TL_CAP_TAPS(T, RUN, 4) }
#define TL_CAP_RUN(T)                             \
  if (single) { TL_CAP_PER(T, 1) }                \
  else { TL_CAP_PER(T, kConvRun) }
  if (dtype == 0) { TL_CAP_RUN(float) }
  else if (dtype == 1) { TL_CAP_RUN(bf16_t) }
  else return TL_ERR_ARG;
#undef TL_CAP_RUN
#undef TL_CAP_PER
#undef TL_CAP_TAPS
#undef TL_CAP
  return tl_launch_status();
}

// a0, a1 (a1 null for one map): [n_tokens, heads * D] in a_dtype (float32, or z's type), rows a_stride apart; g:
// float32 gates or null; z: [n_tokens, >= heads * vdim + tail] in dtype, rows z_stride apart.
int tl_attn_finish(const void* a0, const void* a1, int64_t a_stride, const float* g, int64_t g_stride, void* z,
                   int64_t z_stride, int n_tokens, int heads, int vdim, int D, float lambda, int sub_norm, float eps,
                   float scale, int gate_kind, int tail, int a_dtype, int dtype, hipStream_t stream) {
  if (n_tokens <= 0) return TL_OK;
  if (heads <= 0 || heads > 65535 || vdim <= 0 || D < vdim || vdim > 4 * TL_WAVE || !a0 || !z || gate_kind < 0 ||
      gate_kind > 2 || (gate_kind && !g) || tail < 0 || tail > TL_WAVE)
    return TL_ERR_ARG;
  dim3 grid(n_tokens, heads), b(TL_WAVE);
#define TL_FINISH(TA, TZ)                                                                                             \
  hipLaunchKernelGGL((attn_finish_kernel<TA, TZ>), grid, b, 0, stream, (const TA*)a0, (const TA*)a1, a_stride, g,       \
                     g_stride, (TZ*)z, z_stride, heads, vdim, D, lambda, sub_norm, eps, scale, gate_kind, tail)
  if (a_dtype == 0 && dtype == 0) TL_FINISH(float, float);
  else if (a_dtype == 0 && dtype == 1) TL_FINISH(float, bf16_t);
  else if (a_dtype == 1 && dtype == 1) TL_FINISH(bf16_t, bf16_t);
  else return TL_ERR_ARG;
#undef TL_FINISH
  return tl_launch_status();
}

}  // extern "C"
