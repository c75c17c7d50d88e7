// Kernels around a sublayer whose norm sits on its OUTPUT: x += scale * w * y / rms(y), the copy
// of the residual stream in the engine's element type that the next sublayer's products read, a
// gated unit with clamped inputs, and the soft cap of the logits.
//
// The residual stream, the norm's statistics and its weight are float32 in both precisions.
#include "common.h"

namespace {

constexpr int kThreads = 256;
constexpr int kWaves = kThreads / TL_WAVE;

// x[t] += scale * w * y[t] / sqrt(mean(y[t]^2) + eps); copy[t] = x[t] in TC (optional).
// One workgroup per row.  `w` is the norm's effective weight, `scale` (optional) a factor per channel.
// Rows of up to KEEP * kThreads elements stay in registers between the two passes, and what the second
// pass needs (x, w, scale) is requested before the sum of squares is known (KEEP 8 for rows of up to
// 2,048 elements, 32 up to 8,192; longer rows are read twice).
template <typename TC, int KEEP>
__global__ __launch_bounds__(kThreads) void norm_scale_add_kernel(const float* __restrict__ y,
                                                                  const float* __restrict__ w,
                                                                  const float* __restrict__ scale,
                                                                  float* __restrict__ x, TC* __restrict__ copy,
                                                                  int hidden, float eps) {
  __shared__ float red[kWaves];
  const float* src = y + (int64_t)blockIdx.x * hidden;
  float* dst = x + (int64_t)blockIdx.x * hidden;
  float ss = 0.f;
  if (hidden <= KEEP * kThreads) {
    float yv[KEEP], xv[KEEP], wv[KEEP];
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
      const int j = threadIdx.x + i * kThreads;
      const bool in = j < hidden;
      yv[i] = in ? src[j] : 0.f;
      xv[i] = in ? dst[j] : 0.f;
      wv[i] = in ? (scale ? w[j] * scale[j] : w[j]) : 0.f;
      ss += yv[i] * yv[i];
    }
    ss = block_sum<kWaves>(ss, red);
    const float r = 1.f / sqrtf(ss / (float)hidden + eps);
#pragma unroll
    for (int i = 0; i < KEEP; ++i) {
      const int j = threadIdx.x + i * kThreads;
      if (j < hidden) {
        const float s = xv[i] + yv[i] * r * wv[i];
        dst[j] = s;
        if (copy) copy[(int64_t)blockIdx.x * hidden + j] = from_f32<TC>(s);
      }
    }
    return;
  }
  for (int j = threadIdx.x; j < hidden; j += kThreads) {
    const float v = src[j];
    ss += v * v;
  }
  ss = block_sum<kWaves>(ss, red);
  const float r = 1.f / sqrtf(ss / (float)hidden + eps);
  for (int j = threadIdx.x; j < hidden; j += kThreads) {
    float v = src[j] * r * w[j];
    if (scale) v *= scale[j];
    const float s = dst[j] + v;
    dst[j] = s;
    if (copy) copy[(int64_t)blockIdx.x * hidden + j] = from_f32<TC>(s);
  }
}

template <typename TO>
__global__ void cast_rows_kernel(const float* __restrict__ x, TO* __restrict__ out, int64_t total) {
  const int64_t i = (int64_t)blockIdx.x * kThreads + threadIdx.x;
  if (i < total) out[i] = from_f32<TO>(x[i]);
}

// z[t, j] = g * sigmoid(alpha * g) * (u + shift), g = min(gate_up[t, j], limit),
// u = clamp(gate_up[t, inter + j], -limit, limit).
template <typename T>
__global__ void clamped_glu_kernel(const T* __restrict__ gate_up, T* __restrict__ z, int64_t total, int inter,
                                   int64_t in_stride, float limit, float alpha, float shift) {
  const int64_t i = (int64_t)blockIdx.x * kThreads + threadIdx.x;
  if (i >= total) return;
  const int64_t t = i / inter;
  const int j = (int)(i - t * inter);
  const float g = fminf(to_f32(gate_up[t * in_stride + j]), limit);
  const float u = fminf(fmaxf(to_f32(gate_up[t * in_stride + inter + j]), -limit), limit);
  z[i] = from_f32<T>(g / (1.f + expf(-alpha * g)) * (u + shift));
}

// z[t, j] = gelu(gate_up[t, j]) * gate_up[t, inter + j], gelu in its tanh form:
// 0.5 g (1 + tanh(sqrt(2 / pi) (g + 0.044715 g^3))).
template <typename T>
__global__ void gelu_glu_kernel(const T* __restrict__ gate_up, T* __restrict__ z, int64_t total, int inter,
                                int64_t in_stride) {
  const int64_t i = (int64_t)blockIdx.x * kThreads + threadIdx.x;
  if (i >= total) return;
  const int64_t t = i / inter;
  const int j = (int)(i - t * inter);
  const float g = to_f32(gate_up[t * in_stride + j]);
  const float u = to_f32(gate_up[t * in_stride + inter + j]);
  const float act = 0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
  z[i] = from_f32<T>(act * u);
}

// z[t, j] = gelu(gate[t, j]) * table[tokens[t], off + j] for j < dim (gelu in its tanh form), zeros up to the row's `wide`.
template <typename T>
__global__ void gelu_table_rows_kernel(const float* __restrict__ gate, int64_t gate_stride, const int32_t* __restrict__ tokens,
                                       const T* __restrict__ table, int64_t table_stride, int off, T* __restrict__ z,
                                       int64_t total, int dim, int wide) {
  const int64_t i = (int64_t)blockIdx.x * kThreads + threadIdx.x;
  if (i >= total) return;
  const int64_t t = i / wide;
  const int j = (int)(i - t * wide);
  float v = 0.f;
  if (j < dim) {
    const float g = gate[t * gate_stride + j];
    const float act = 0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
    v = act * to_f32(table[(int64_t)tokens[t] * table_stride + off + j]);
  }
  z[i] = from_f32<T>(v);
}

// The product in front of it and gelu_table_rows_kernel in one, for few rows: a workgroup a column, eight rows at a time;
// its threads stride over the inner size in vectors (a row's sum is formed in one order whatever else the step holds).
constexpr int kGateRows = 8;
template <typename T>
__global__ __launch_bounds__(kThreads) void token_gate_kernel(const T* __restrict__ h, int64_t h_stride,
                                                              const T* __restrict__ w, const int32_t* __restrict__ tokens,
                                                              const T* __restrict__ table, int64_t table_stride, int off,
                                                              T* __restrict__ z, int n_rows, int K, int dim, int wide, int vec) {
  typedef T tvec __attribute__((ext_vector_type(8)));
  __shared__ float red[kWaves][kGateRows];
  const int j = blockIdx.x, tid = threadIdx.x, lane = tid % TL_WAVE, t0 = blockIdx.y * kGateRows;
  const int n = min(kGateRows, n_rows - t0);
  float acc[kGateRows], e = 0.f;
#pragma unroll
  for (int r = 0; r < kGateRows; ++r) acc[r] = 0.f;
  if (j < dim) {
    if (tid < n) e = to_f32(table[(int64_t)tokens[t0 + tid] * table_stride + off + j]);
    const T* wr = w + (int64_t)j * K;
    const T* hr[kGateRows];
#pragma unroll
    for (int r = 0; r < kGateRows; ++r) hr[r] = h + (int64_t)(t0 + min(r, n - 1)) * h_stride;
    if (vec) {
      for (int k = tid * 8; k < K; k += kThreads * 8) {
        const tvec wv = *(const tvec*)(wr + k);
        tvec hv[kGateRows];
#pragma unroll
        for (int r = 0; r < kGateRows; ++r) hv[r] = *(const tvec*)(hr[r] + k);
#pragma unroll
        for (int r = 0; r < kGateRows; ++r)
#pragma unroll
          for (int c = 0; c < 8; ++c) acc[r] = fmaf((float)hv[r][c], (float)wv[c], acc[r]);
      }
    } else {
      for (int k = tid; k < K; k += kThreads) {
        const float wv = to_f32(wr[k]);
#pragma unroll
        for (int r = 0; r < kGateRows; ++r) acc[r] = fmaf(to_f32(hr[r][k]), wv, acc[r]);
      }
    }
  }
#pragma unroll
  for (int r = 0; r < kGateRows; ++r) {
    const float s = wave_sum(acc[r]);
    if (lane == 0) red[tid / TL_WAVE][r] = s;
  }
  __syncthreads();
  if (tid < n) {
    float g = 0.f;
#pragma unroll
    for (int w4 = 0; w4 < kWaves; ++w4) g += red[w4][tid];
    const float act = 0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
    z[(int64_t)(t0 + tid) * wide + j] = from_f32<T>(j < dim ? act * e : 0.f);
  }
}

__global__ void softcap_kernel(float* __restrict__ x, int64_t total, float cap) {
  const int64_t i = (int64_t)blockIdx.x * kThreads + threadIdx.x;
  if (i < total) x[i] = cap * tanhf(x[i] / cap);
}

// Two streams side by side as the operand of one product: operand[t] = [a[t] | b[t]] rounded to T, and
// init[t] = vec (a row that the product then adds its result to, so a vector joins every row without a kernel of
// its own).  One thread an element of the wider of the two outputs.
template <typename T>
__global__ void stream_join_kernel(const float* __restrict__ a, const float* __restrict__ b, const float* __restrict__ vec,
                                   T* __restrict__ operand, float* __restrict__ init, int64_t total, int width) {
  const int64_t i = (int64_t)blockIdx.x * kThreads + threadIdx.x;
  if (i >= total) return;
  const int64_t t = i / (2 * width);
  const int c = (int)(i - t * 2 * width);
  operand[i] = from_f32<T>(c < width ? a[t * width + c] : b[t * width + c - width]);
  if (c < width) init[t * width + c] = vec ? vec[c] : 0.f;
}

}  // namespace

extern "C" {

// copy_dtype: 0 float32, 1 bfloat16; copy and scale may be null.
int tl_norm_scale_add(const float* y, const float* w, const float* scale, float* x, void* copy, int n_rows,
                      int hidden, float eps, int copy_dtype, hipStream_t stream) {
  if (n_rows <= 0) return TL_OK;
  if (hidden <= 0) return TL_ERR_ARG;
  dim3 g(n_rows), b(kThreads);
  const bool few = hidden <= 8 * kThreads;
  if (copy_dtype == 1 && few)
    hipLaunchKernelGGL((norm_scale_add_kernel<bf16_t, 8>), g, b, 0, stream, y, w, scale, x, (bf16_t*)copy, hidden, eps);
  else if (copy_dtype == 1)
    hipLaunchKernelGGL((norm_scale_add_kernel<bf16_t, 32>), g, b, 0, stream, y, w, scale, x, (bf16_t*)copy, hidden, eps);
  else if (copy_dtype == 0 && few)
    hipLaunchKernelGGL((norm_scale_add_kernel<float, 8>), g, b, 0, stream, y, w, scale, x, (float*)copy, hidden, eps);
  else if (copy_dtype == 0)
    hipLaunchKernelGGL((norm_scale_add_kernel<float, 32>), g, b, 0, stream, y, w, scale, x, (float*)copy, hidden, eps);
  else
    return TL_ERR_ARG;
  return tl_launch_status();
}

int tl_cast_rows(const float* x, void* out, int64_t total, int out_dtype, hipStream_t stream) {
  if (total <= 0) return TL_OK;
  dim3 g((unsigned)ceil_div64(total, kThreads)), b(kThreads);
  if (out_dtype == 1)
    hipLaunchKernelGGL(cast_rows_kernel<bf16_t>, g, b, 0, stream, x, (bf16_t*)out, total);
  else if (out_dtype == 0)
    hipLaunchKernelGGL(cast_rows_kernel<float>, g, b, 0, stream, x, (float*)out, total);
  else
    return TL_ERR_ARG;
  return tl_launch_status();
}

int tl_clamped_glu(const void* gate_up, void* z, int n_rows, int inter, int64_t in_stride, float limit, float alpha,
                   float shift, int dtype, hipStream_t stream) {
  if (n_rows <= 0) return TL_OK;
  if (inter <= 0 || in_stride < 2 * (int64_t)inter) return TL_ERR_ARG;
  const int64_t total = (int64_t)n_rows * inter;
  dim3 g((unsigned)ceil_div64(total, kThreads)), b(kThreads);
  if (dtype == 0)
    hipLaunchKernelGGL(clamped_glu_kernel<float>, g, b, 0, stream, (const float*)gate_up, (float*)z, total, inter,
                       in_stride, limit, alpha, shift);
  else if (dtype == 1)
    hipLaunchKernelGGL(clamped_glu_kernel<bf16_t>, g, b, 0, stream, (const bf16_t*)gate_up, (bf16_t*)z, total, inter,
                       in_stride, limit, alpha, shift);
  else
    return TL_ERR_ARG;
  return tl_launch_status();
}

int tl_gelu_glu(const void* gate_up, void* z, int n_rows, int inter, int64_t in_stride, int dtype, hipStream_t stream) {
  if (n_rows <= 0) return TL_OK;
  if (inter <= 0 || in_stride < 2 * (int64_t)inter) return TL_ERR_ARG;
  const int64_t total = (int64_t)n_rows * inter;
  dim3 g((unsigned)ceil_div64(total, kThreads)), b(kThreads);
  if (dtype == 0)
    hipLaunchKernelGGL(gelu_glu_kernel<float>, g, b, 0, stream, (const float*)gate_up, (float*)z, total, inter, in_stride);
  else if (dtype == 1)
    hipLaunchKernelGGL(gelu_glu_kernel<bf16_t>, g, b, 0, stream, (const bf16_t*)gate_up, (bf16_t*)z, total, inter,
                       in_stride);
  else
    return TL_ERR_ARG;
  return tl_launch_status();
}

// gate: float32 [n_rows, >= dim]; table: [vocab, table_stride] in dtype; z: [n_rows, wide] in dtype.
int tl_gelu_table_rows(const float* gate, int64_t gate_stride, const int32_t* tokens, const void* table, int64_t table_stride,
                       int off, void* z, int n_rows, int dim, int wide, int dtype, hipStream_t stream) {
  if (n_rows <= 0) return TL_OK;
  if (dim <= 0 || wide < dim || off < 0 || off + dim > table_stride || gate_stride < dim || !gate || !tokens || !table || !z)
    return TL_ERR_ARG;
  const int64_t total = (int64_t)n_rows * wide;
  dim3 g((unsigned)ceil_div64(total, kThreads)), b(kThreads);
  if (dtype == 0)
    hipLaunchKernelGGL(gelu_table_rows_kernel<float>, g, b, 0, stream, gate, gate_stride, tokens, (const float*)table,
                       table_stride, off, (float*)z, total, dim, wide);
  else if (dtype == 1)
    hipLaunchKernelGGL(gelu_table_rows_kernel<bf16_t>, g, b, 0, stream, gate, gate_stride, tokens, (const bf16_t*)table,
                       table_stride, off, (bf16_t*)z, total, dim, wide);
  else
    return TL_ERR_ARG;
  return tl_launch_status();
}

// h: [n_rows, K], w: [>= dim, K], table, z as tl_gelu_table_rows; all in dtype.
int tl_token_gate(const void* h, int64_t h_stride, const void* w, const int32_t* tokens, const void* table,
                  int64_t table_stride, int off, void* z, int n_rows, int K, int dim, int wide, int dtype, hipStream_t stream) {
  if (n_rows <= 0) return TL_OK;
  if (dim <= 0 || wide < dim || K <= 0 || off < 0 || off + dim > table_stride || !h || !w || !tokens || !table || !z ||
      (n_rows + kGateRows - 1) / kGateRows > 65535)
    return TL_ERR_ARG;
  dim3 g(wide, (n_rows + kGateRows - 1) / kGateRows), b(kThreads);
  const int vec = K % 8 == 0 && h_stride % 8 == 0 && !(((uintptr_t)h | (uintptr_t)w) & 15);
#define TL_GATE(T)                                                                                                      \
  hipLaunchKernelGGL(token_gate_kernel<T>, g, b, 0, stream, (const T*)h, h_stride, (const T*)w, tokens, (const T*)table, \
                     table_stride, off, (T*)z, n_rows, K, dim, wide, vec)
  if (dtype == 0) TL_GATE(float);
  else if (dtype == 1) TL_GATE(bf16_t);
  else return TL_ERR_ARG;
#undef TL_GATE
  return tl_launch_status();
}

int tl_softcap(float* x, int64_t total, float cap, hipStream_t stream) {
  if (total <= 0) return TL_OK;
  if (!(cap > 0.f)) return TL_ERR_ARG;
  hipLaunchKernelGGL(softcap_kernel, dim3((unsigned)ceil_div64(total, kThreads)), dim3(kThreads), 0, stream, x, total,
                     cap);
  return tl_launch_status();
}

// a, b: float32 [n_rows, width]; operand: [n_rows, 2 * width] in dtype; init: float32 [n_rows, width] (every row
// becomes vec, or zeros without one).
int tl_stream_join(const float* a, const float* b, const float* vec, void* operand, float* init, int n_rows, int width,
                   int dtype, hipStream_t stream) {
  if (n_rows <= 0) return TL_OK;
  if (width <= 0 || !a || !b || !operand || !init) return TL_ERR_ARG;
  const int64_t total = (int64_t)n_rows * 2 * width;
  dim3 g((unsigned)ceil_div64(total, kThreads)), blk(kThreads);
  if (dtype == 0)
    hipLaunchKernelGGL(stream_join_kernel<float>, g, blk, 0, stream, a, b, vec, (float*)operand, init, total, width);
  else if (dtype == 1)
    hipLaunchKernelGGL(stream_join_kernel<bf16_t>, g, blk, 0, stream, a, b, vec, (bf16_t*)operand, init, total, width);
  else
    return TL_ERR_ARG;
  return tl_launch_status();
}

}  // extern "C"
