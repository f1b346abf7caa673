// RMSNorm, optionally fused with the residual add that precedes it, and the
// embedding row gather that starts the residual stream.
//
//   h   = residual (32-bit, may be absent) + delta (storage type, may be absent)
//   out = h * (1 / sqrt(mean(h^2) + eps)) * weight
//
// The residual stream stays in 32-bit; with `write_residual` the sum is stored
// back so that the next block adds to it.  With `rows` only the listed rows are
// normalised (the rows whose logits are wanted) and nothing is stored back.
// Further forms: the embedding with a second table picked by pairs of tokens, a stream that
// takes its blocks' results with weights, and one that takes them normed.
// Formula as in /root/reference/src/transformer/norm.zig:6-33 (32-bit sum of
// squares, weight multiplied after the scale, no bias).
#include "common.h"

// `delta` may be a stack of `n_partials` partial sums (each `partial_stride`
// elements apart): the pieces a projection split along K leaves to its consumer.
// They are added up first, in their order, and the sum is added to the residual.
template <typename TD>
__device__ __forceinline__ float delta_at(const TD* dl, size_t i, int n_partials,
                                          size_t partial_stride) {
  float v = to_f32<TD>(dl[i]);
  for (int p = 1; p < n_partials; ++p) v += to_f32<TD>(dl[i + p * partial_stride]);
  return v;
}

// Four consecutive elements as floats; `p` aligned to four elements.
template <typename T> __device__ __forceinline__ void load4(const T* p, float out[4]);
template <> __device__ __forceinline__ void load4<float>(const float* p, float out[4]) {
  const float4 a = *reinterpret_cast<const float4*>(p);
  out[0] = a.x; out[1] = a.y; out[2] = a.z; out[3] = a.w;
}
template <> __device__ __forceinline__ void load4<bf16_t>(const bf16_t* p, float out[4]) {
  const bf16x4_t v = *reinterpret_cast<const bf16x4_t*>(p);
#pragma unroll
  for (int i = 0; i < 4; ++i) out[i] = (float)v[i];
}
template <typename T> __device__ __forceinline__ void store4(T* p, const float in[4]);
template <> __device__ __forceinline__ void store4<float>(float* p, const float in[4]) {
  *reinterpret_cast<float4*>(p) = make_float4(in[0], in[1], in[2], in[3]);
}
template <> __device__ __forceinline__ void store4<bf16_t>(bf16_t* p, const float in[4]) {
  bf16x4_t v;
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = (bf16_t)in[i];
  *reinterpret_cast<bf16x4_t*>(p) = v;
}

// The same sum as delta_at for the four elements at `i`, with the loads of up to
// eight partial sums issued before the first is waited for.
template <typename TD>
__device__ __forceinline__ void delta4_at(const TD* dl, size_t i, int n_partials,
                                          size_t partial_stride, float v[4]) {
  load4<TD>(dl + i, v);
  for (int p0 = 1; p0 < n_partials; p0 += 8) {
    float t[8][4];
#pragma unroll
    for (int q = 0; q < 8; ++q) {
      if (p0 + q < n_partials) {
        load4<TD>(dl + i + (size_t)(p0 + q) * partial_stride, t[q]);
      } else {
        t[q][0] = t[q][1] = t[q][2] = t[q][3] = 0.f;
      }
    }
#pragma unroll
    for (int q = 0; q < 8; ++q) {
      if (p0 + q < n_partials) {
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] += t[q][e];
      }
    }
  }
}

// General form: two passes over the row, any width.
template <typename TD, typename TO>
__global__ void __launch_bounds__(256)
add_rmsnorm_kernel(float* __restrict__ residual, const TD* __restrict__ delta,
                   const float* __restrict__ weight, TO* __restrict__ out,
                   const int* __restrict__ rows, int width, float eps, int write_residual,
                   int n_partials, size_t partial_stride, const float* __restrict__ bias,
                   int center) {
  __shared__ float scratch[16];
  const int r = blockIdx.x;
  const size_t src = rows ? (size_t)rows[r] : (size_t)r;
  float* x = residual ? residual + src * width : nullptr;
  const TD* dl = delta ? delta + src * width : nullptr;
  TO* o = out + (size_t)r * width;

  float ss = 0.f, sum = 0.f;
  for (int i = threadIdx.x; i < width; i += blockDim.x) {
    float h = x ? x[i] : 0.f;
    if (dl) h += delta_at<TD>(dl, i, n_partials, partial_stride);
    if (write_residual) x[i] = h;
    ss += h * h;
    sum += h;
  }
  float mean = 0.f;
  if (center) {
    // a layer norm: the squared deviations from the mean, summed in a pass of their own
    mean = block_sum(sum, scratch) / (float)width;
    ss = 0.f;
    for (int i = threadIdx.x; i < width; i += blockDim.x) {
      float h;
      if (write_residual) {
        h = x[i];
      } else {
        h = x ? x[i] : 0.f;
        if (dl) h += delta_at<TD>(dl, i, n_partials, partial_stride);
      }
      ss += (h - mean) * (h - mean);
    }
  }
  ss = block_sum(ss, scratch);
  const float scale = 1.0f / sqrtf(ss / (float)width + eps);
  for (int i = threadIdx.x; i < width; i += blockDim.x) {
    float h;
    if (write_residual) {
      h = x[i];  // this thread stored it above
    } else {
      h = x ? x[i] : 0.f;
      if (dl) h += delta_at<TD>(dl, i, n_partials, partial_stride);
    }
    const float y = (h - mean) * scale * weight[i];
    o[i] = from_f32<TO>(bias ? y + bias[i] : y);
  }
}

// Rows of at most 256 * 4 * VPT elements with width % 4 == 0: the row stays in
// registers between the sum of squares and the scaling, one pass over memory.
template <typename TD, typename TO, int VPT>
__global__ void __launch_bounds__(256)
add_rmsnorm_regs_kernel(float* __restrict__ residual, const TD* __restrict__ delta,
                        const float* __restrict__ weight, TO* __restrict__ out,
                        const int* __restrict__ rows, int width, float eps, int write_residual,
                        int n_partials, size_t partial_stride, const float* __restrict__ bias,
                        int center) {
  __shared__ float scratch[16];
  const int r = blockIdx.x;
  const size_t src = rows ? (size_t)rows[r] : (size_t)r;
  float* x = residual ? residual + src * width : nullptr;
  const TD* dl = delta ? delta + src * width : nullptr;
  TO* o = out + (size_t)r * width;
  float h[VPT][4];
  float ss = 0.f, sum = 0.f;
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int i = (threadIdx.x + v * 256) * 4;
    if (i < width) {
      if (x) {
        const float4 t = *reinterpret_cast<const float4*>(x + i);
        h[v][0] = t.x; h[v][1] = t.y; h[v][2] = t.z; h[v][3] = t.w;
      } else {
        h[v][0] = h[v][1] = h[v][2] = h[v][3] = 0.f;
      }
      if (dl) {
        float d4[4];
        delta4_at<TD>(dl, i, n_partials, partial_stride, d4);
#pragma unroll
        for (int e = 0; e < 4; ++e) h[v][e] += d4[e];
      }
      if (write_residual)
        *reinterpret_cast<float4*>(x + i) = make_float4(h[v][0], h[v][1], h[v][2], h[v][3]);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        ss += h[v][e] * h[v][e];
        sum += h[v][e];
      }
    }
  }
  if (center) {
    // a layer norm: the row (already stored, if it is to be) becomes its deviations
    const float mean = block_sum(sum, scratch) / (float)width;
    ss = 0.f;
#pragma unroll
    for (int v = 0; v < VPT; ++v) {
      const int i = (threadIdx.x + v * 256) * 4;
      if (i < width) {
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          h[v][e] -= mean;
          ss += h[v][e] * h[v][e];
        }
      }
    }
  }
  ss = block_sum(ss, scratch);
  const float scale = 1.0f / sqrtf(ss / (float)width + eps);
#pragma unroll
  for (int v = 0; v < VPT; ++v) {
    const int i = (threadIdx.x + v * 256) * 4;
    if (i < width) {
      const float4 w = *reinterpret_cast<const float4*>(weight + i);
      float y[4] = {h[v][0] * scale * w.x, h[v][1] * scale * w.y, h[v][2] * scale * w.z,
                    h[v][3] * scale * w.w};
      if (bias) {
        const float4 b = *reinterpret_cast<const float4*>(bias + i);
        y[0] += b.x; y[1] += b.y; y[2] += b.z; y[3] += b.w;
      }
      store4<TO>(o + i, y);
    }
  }
}

template <typename T>
__global__ void __launch_bounds__(256)
embed_gather_kernel(const int* __restrict__ tokens, const T* __restrict__ table,
                    float* __restrict__ out, int width, int vocab) {
  const int t = blockIdx.x;
  const int tok = tokens[t];
  float* o = out + (size_t)t * width;
  if (tok < 0 || tok >= vocab) {
    // Never read outside the table; an id the host failed to reject poisons its row.
    for (int i = threadIdx.x; i < width; i += blockDim.x) o[i] = __builtin_nanf("");
    return;
  }
  const T* row = table + (size_t)tok * width;
  for (int i = threadIdx.x; i < width; i += blockDim.x) o[i] = to_f32<T>(row[i]);
}

// dtype codes: 0 = float32, 1 = bfloat16
static int add_norm_any(void* residual, const void* delta, int delta_dtype, const float* weight,
                        const float* bias, int center, void* out, int out_dtype, const int* rows,
                        int n_rows, int width, float eps, int write_residual, int n_partials,
                        long long partial_stride, hipStream_t stream) {
  if (n_rows == 0) return 0;
  if (n_rows < 0 || width <= 0 || (!residual && !delta) || !weight || !out || n_partials < 1)
    return ZA_ERR_ARG;
  if (n_partials > 1 && (!delta || partial_stride <= 0)) return ZA_ERR_ARG;
  if (!residual || rows) write_residual = 0;
  dim3 grid(n_rows), block(256);
  float* res = (float*)residual;
  const int vpt = width % 4 == 0 ? (width / 4 + 255) / 256 : 0;   // vectors per thread
#define ZA_NORM_LAUNCH(KERNEL, TD, TO)                                                      \
  hipLaunchKernelGGL((KERNEL), grid, block, 0, stream, res, (const TD*)delta, weight,       \
                     (TO*)out, rows, width, eps, write_residual, n_partials,                \
                     (size_t)partial_stride, bias, center)
#define ZA_NORM_CASE(DD, TD, OD, TO)                                                        \
  if (delta_dtype == DD && out_dtype == OD) {                                               \
    if (vpt == 1) ZA_NORM_LAUNCH((add_rmsnorm_regs_kernel<TD, TO, 1>), TD, TO);             \
    else if (vpt == 2) ZA_NORM_LAUNCH((add_rmsnorm_regs_kernel<TD, TO, 2>), TD, TO);        \
    else if (vpt >= 3 && vpt <= 4) ZA_NORM_LAUNCH((add_rmsnorm_regs_kernel<TD, TO, 4>), TD, TO); \
    else ZA_NORM_LAUNCH((add_rmsnorm_kernel<TD, TO>), TD, TO);                              \
    return za_launch_status();                                                              \
  }
  ZA_NORM_CASE(0, float, 0, float)
  ZA_NORM_CASE(0, float, 1, bf16_t)
  ZA_NORM_CASE(1, bf16_t, 0, float)
  ZA_NORM_CASE(1, bf16_t, 1, bf16_t)
#undef ZA_NORM_CASE
#undef ZA_NORM_LAUNCH
  return ZA_ERR_UNSUPPORTED;
}

extern "C" int za_add_rmsnorm(void* residual, const void* delta, int delta_dtype,
                              const float* weight, void* out, int out_dtype, const int* rows,
                              int n_rows, int width, float eps, int write_residual,
                              int n_partials, long long partial_stride, hipStream_t stream) {
  return add_norm_any(residual, delta, delta_dtype, weight, nullptr, 0, out, out_dtype, rows,
                      n_rows, width, eps, write_residual, n_partials, partial_stride, stream);
}

// The same with the mean taken off first and a bias added last (a layer norm):
//   out = (h - mean(h)) / sqrt(mean((h - mean(h))^2) + eps) * weight + bias
extern "C" int za_add_layernorm(void* residual, const void* delta, int delta_dtype,
                                const float* weight, const float* bias, void* out, int out_dtype,
                                const int* rows, int n_rows, int width, float eps,
                                int write_residual, int n_partials, long long partial_stride,
                                hipStream_t stream) {
  return add_norm_any(residual, delta, delta_dtype, weight, bias, 1, out, out_dtype, rows,
                      n_rows, width, eps, write_residual, n_partials, partial_stride, stream);
}

// x[t] <- x[t] + delta[t] (a tensor or a stack of partial sums, may be absent) + origin[t]
// (32-bit, may be absent) + vec (32-bit [width], may be absent): what enters the stream
// between two run-order entries.
template <typename TD>
__global__ void __launch_bounds__(256)
stream_add_kernel(float* __restrict__ x, const TD* __restrict__ delta, int n_partials,
                  size_t partial_stride, const float* __restrict__ origin,
                  const float* __restrict__ vec, int width, size_t total) {
  const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= total) return;
  float h = x[i];
  if (delta) h += delta_at<TD>(delta, i, n_partials, partial_stride);
  if (origin) h += origin[i];
  if (vec) h += vec[i % width];
  x[i] = h;
}

extern "C" int za_stream_add(float* x, const void* delta, int delta_dtype, int n_partials,
                             long long partial_stride, const float* origin, const float* vec,
                             int n_rows, int width, hipStream_t stream) {
  if (n_rows == 0) return 0;
  if (n_rows < 0 || width <= 0 || !x || n_partials < 1) return ZA_ERR_ARG;
  if (n_partials > 1 && (!delta || partial_stride <= 0)) return ZA_ERR_ARG;
  const size_t total = (size_t)n_rows * width;
  dim3 grid((unsigned)((total + 255) / 256)), block(256);
  if (delta_dtype == 0)
    hipLaunchKernelGGL((stream_add_kernel<float>), grid, block, 0, stream, x, (const float*)delta,
                       n_partials, (size_t)partial_stride, origin, vec, width, total);
  else if (delta_dtype == 1)
    hipLaunchKernelGGL((stream_add_kernel<bf16_t>), grid, block, 0, stream, x,
                       (const bf16_t*)delta, n_partials, (size_t)partial_stride, origin, vec,
                       width, total);
  else
    return ZA_ERR_UNSUPPORTED;
  return za_launch_status();
}

extern "C" int za_embed_gather(const int* tokens, const void* table, int table_dtype, float* out,
                               int n_tokens, int width, int vocab, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  if (n_tokens < 0 || width <= 0 || vocab <= 0 || !tokens || !table || !out) return ZA_ERR_ARG;
  dim3 grid(n_tokens), block(256);
  if (table_dtype == 0) {
    hipLaunchKernelGGL((embed_gather_kernel<float>), grid, block, 0, stream, tokens,
                       (const float*)table, out, width, vocab);
  } else if (table_dtype == 1) {
    hipLaunchKernelGGL((embed_gather_kernel<bf16_t>), grid, block, 0, stream, tokens,
                       (const bf16_t*)table, out, width, vocab);
  } else {
    return ZA_ERR_UNSUPPORTED;
  }
  return za_launch_status();
}

// A residual stream that takes its blocks' results with weights:
//   x <- x + sa * a + sb * b      (b may be absent; 32-bit sum, stored)
//   out = x / sqrt(mean(x^2) + eps) * weight      (when a norm's weight is given)
// `a` and `b` are in the storage type TD.  One workgroup a row, two passes.
#define SA_VPT 16   // values a thread keeps between the sum of squares and the scaling
template <typename TD, typename TO>
__global__ void __launch_bounds__(256)
scaled_add_rmsnorm_kernel(float* __restrict__ residual, const TD* __restrict__ a, float sa,
                          const TD* __restrict__ b, float sb, const float* __restrict__ weight,
                          TO* __restrict__ out, int width, float eps) {
  __shared__ float scratch[16];
  const size_t r = blockIdx.x;
  float* x = residual + r * width;
  const TD* ar = a + r * width;
  const TD* br = b ? b + r * width : nullptr;
  const int bd = blockDim.x;
  float ss = 0.f;
  if (width <= bd * SA_VPT) {
    // the row stays in registers: one trip to memory, every load requested at once
    float h[SA_VPT], wv[SA_VPT];
#pragma unroll
    for (int k = 0; k < SA_VPT; ++k) {
      const int i = threadIdx.x + k * bd;
      const bool in = i < width;
      h[k] = in ? x[i] : 0.f;
      const float av = in ? to_f32<TD>(ar[i]) : 0.f;
      const float bv = (in && br) ? to_f32<TD>(br[i]) : 0.f;
      wv[k] = (in && weight) ? weight[i] : 0.f;
      h[k] = fmaf(sa, av, h[k]);
      if (br) h[k] = fmaf(sb, bv, h[k]);
    }
#pragma unroll
    for (int k = 0; k < SA_VPT; ++k) {
      const int i = threadIdx.x + k * bd;
      if (i < width) x[i] = h[k];
      ss += h[k] * h[k];
    }
    if (!weight) return;
    ss = block_sum(ss, scratch);
    const float scale = 1.0f / sqrtf(ss / (float)width + eps);
    TO* o = out + r * width;
#pragma unroll
    for (int k = 0; k < SA_VPT; ++k) {
      const int i = threadIdx.x + k * bd;
      if (i < width) o[i] = from_f32<TO>(h[k] * scale * wv[k]);
    }
    return;
  }
  for (int i = threadIdx.x; i < width; i += bd) {
    float h = fmaf(sa, to_f32<TD>(ar[i]), x[i]);
    if (br) h = fmaf(sb, to_f32<TD>(br[i]), h);
    x[i] = h;
    ss += h * h;
  }
  if (!weight) return;
  ss = block_sum(ss, scratch);
  const float scale = 1.0f / sqrtf(ss / (float)width + eps);
  TO* o = out + r * width;
  for (int i = threadIdx.x; i < width; i += bd)
    o[i] = from_f32<TO>(x[i] * scale * weight[i]);   // this thread stored x[i] above
}

extern "C" int za_scaled_add_rmsnorm(float* residual, const void* a, float sa, const void* b,
                                     float sb, int delta_dtype, const float* weight, void* out,
                                     int out_dtype, int n_rows, int width, float eps,
                                     hipStream_t stream) {
  if (n_rows == 0) return 0;
  if (n_rows < 0 || width <= 0 || !residual || !a || (weight && !out)) return ZA_ERR_ARG;
  dim3 grid(n_rows), block(width <= 256 ? 64 : 256);
#define ZA_SCALED_ADD(TD, TO)                                                                  \
  hipLaunchKernelGGL((scaled_add_rmsnorm_kernel<TD, TO>), grid, block, 0, stream, residual,    \
                     (const TD*)a, sa, (const TD*)b, sb, weight, (TO*)out, width, eps)
  if (delta_dtype == 0 && out_dtype == 0) ZA_SCALED_ADD(float, float);
  else if (delta_dtype == 1 && out_dtype == 1) ZA_SCALED_ADD(bf16_t, bf16_t);
  else if (delta_dtype == 1 && out_dtype == 0) ZA_SCALED_ADD(bf16_t, float);
  else if (delta_dtype == 0 && out_dtype == 1) ZA_SCALED_ADD(float, bf16_t);
  else return ZA_ERR_UNSUPPORTED;
#undef ZA_SCALED_ADD
  return za_launch_status();
}

// residual += scale * y / sqrt(mean(y^2) + eps) * weight, in 32-bit, in place: something
// that is normed by itself before it enters the stream.  `y` may be a stack of partial sums
// (see delta_at).  With `copy` the sum is also stored there, rounded to the type that the
// next part reads.
template <typename TD, typename TC>
__global__ void __launch_bounds__(256)
normed_add_kernel(float* __restrict__ residual, const TD* __restrict__ y, int n_partials,
                  size_t partial_stride, const float* __restrict__ weight, TC* __restrict__ copy,
                  int width, float eps, float scale) {
  __shared__ float scratch[16];
  const size_t r = blockIdx.x;
  float* x = residual + r * width;
  const TD* yr = y + r * width;
  TC* c = copy ? copy + r * width : nullptr;
  const int bd = blockDim.x;
  float ss = 0.f;
  for (int i = threadIdx.x; i < width; i += bd) {
    const float v = delta_at<TD>(yr, i, n_partials, partial_stride);
    ss += v * v;
  }
  ss = block_sum(ss, scratch);
  const float f = scale / sqrtf(ss / (float)width + eps);
  for (int i = threadIdx.x; i < width; i += bd) {
    const float h = fmaf(delta_at<TD>(yr, i, n_partials, partial_stride) * f, weight[i], x[i]);
    x[i] = h;
    if (c) c[i] = from_f32<TC>(h);
  }
}

// The same for rows of at most 256 * 4 * VPT elements with width % 4 == 0: four elements
// at a time, everything requested at once, one pass over memory.
template <typename TD, typename TC, int VPT>
__global__ void __launch_bounds__(256)
normed_add_regs_kernel(float* __restrict__ residual, const TD* __restrict__ y, int n_partials,
                       size_t partial_stride, const float* __restrict__ weight,
                       TC* __restrict__ copy, int width, float eps, float scale) {
  __shared__ float scratch[16];
  const size_t r = blockIdx.x;
  float* x = residual + r * width;
  const TD* yr = y + r * width;
  float v[VPT][4], h[VPT][4], w[VPT][4];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int i = (threadIdx.x + k * 256) * 4;
    if (i < width) {
      load4<float>(x + i, h[k]);
      load4<float>(weight + i, w[k]);
      delta4_at<TD>(yr, i, n_partials, partial_stride, v[k]);
#pragma unroll
      for (int e = 0; e < 4; ++e) ss += v[k][e] * v[k][e];
    }
  }
  ss = block_sum(ss, scratch);
  const float f = scale / sqrtf(ss / (float)width + eps);
#pragma unroll
  for (int k = 0; k < VPT; ++k) {
    const int i = (threadIdx.x + k * 256) * 4;
    if (i < width) {
#pragma unroll
      for (int e = 0; e < 4; ++e) h[k][e] = fmaf(v[k][e] * f, w[k][e], h[k][e]);
      store4<float>(x + i, h[k]);
      if (copy) store4<TC>(copy + r * width + i, h[k]);
    }
  }
}

// `copy`: null, or [n_rows][width] of `copy_dtype`.
extern "C" int za_normed_add(float* residual, const void* y, int y_dtype, int n_partials,
                             long long partial_stride, const float* weight, void* copy,
                             int copy_dtype, int n_rows, int width, float eps, float scale,
                             hipStream_t stream) {
  if (n_rows == 0) return 0;
  if (n_rows < 0 || width <= 0 || !residual || !y || !weight || n_partials < 1 ||
      (n_partials > 1 && partial_stride < (long long)n_rows * width))
    return ZA_ERR_ARG;
  dim3 grid(n_rows), block(256);
  const int vpt = width % 4 == 0 ? (width / 4 + 255) / 256 : 0;   // vectors per thread
#define ZA_NORMED_ADD(KERNEL, TD, TC)                                                          \
  hipLaunchKernelGGL((KERNEL), grid, block, 0, stream, residual, (const TD*)y, n_partials,     \
                     (size_t)partial_stride, weight, (TC*)copy, width, eps, scale)
#define ZA_NORMED_ADD_CASE(DD, TD, CD, TC)                                                     \
  if (y_dtype == DD && copy_dtype == CD) {                                                     \
    if (vpt == 1) ZA_NORMED_ADD((normed_add_regs_kernel<TD, TC, 1>), TD, TC);                  \
    else if (vpt == 2) ZA_NORMED_ADD((normed_add_regs_kernel<TD, TC, 2>), TD, TC);             \
    else if (vpt >= 3 && vpt <= 4) ZA_NORMED_ADD((normed_add_regs_kernel<TD, TC, 4>), TD, TC); \
    else ZA_NORMED_ADD((normed_add_kernel<TD, TC>), TD, TC);                                   \
    return za_launch_status();                                                                 \
  }
  ZA_NORMED_ADD_CASE(0, float, 0, float)
  ZA_NORMED_ADD_CASE(0, float, 1, bf16_t)
  ZA_NORMED_ADD_CASE(1, bf16_t, 0, float)
  ZA_NORMED_ADD_CASE(1, bf16_t, 1, bf16_t)
#undef ZA_NORMED_ADD_CASE
#undef ZA_NORMED_ADD
  return ZA_ERR_UNSUPPORTED;
}

// The rows that open the stream, with what a token and its predecessor pick from a second
// table added:
//   out[t] = table[tokens[t]] + pairs[row(t)]
//   row(t) = (before * mul_prev + tokens[t] * mul_cur) mod buckets,   before: the token ahead
//            of t in its request; the request's first token (position 0) takes row `buckets`
// The token ahead of a portion's first comes from the request's state, which afterwards holds
// the portion's last token.  One workgroup a token; the workgroup of a portion's first token
// does both, the read before the write, so no other touches the state.  With `copy` the rows are
// also stored rounded.
template <typename T, typename TC>
__global__ void __launch_bounds__(256)
embed_pairs_kernel(const int* __restrict__ tokens, const T* __restrict__ table,
                   const T* __restrict__ pairs, const int* __restrict__ positions,
                   const int* __restrict__ token_seq, const int* __restrict__ seq_start,
                   const int* __restrict__ slot_id, int* __restrict__ state, long long slot_stride,
                   long long buckets, long long mul_prev, long long mul_cur,
                   float* __restrict__ out, TC* __restrict__ copy, int width, int vocab) {
  __shared__ long long picked;
  const int t = blockIdx.x;
  const int tok = tokens[t];
  if (threadIdx.x == 0) {
    const int s = token_seq[t], start = seq_start[s];
    long long before = -1;
    if (t > start) {
      before = tokens[t - 1];
    } else {
      int* last = state + (size_t)slot_id[s] * slot_stride;
      if (positions[t] > 0) before = *last;
      *last = tokens[seq_start[s + 1] - 1];
    }
    long long row = -1;
    if (t == start && positions[t] == 0) row = buckets;
    else if (before >= 0 && before < vocab && tok >= 0) row = (before * mul_prev + tok * mul_cur) % buckets;
    picked = row;
  }
  __syncthreads();
  const long long row = picked;
  float* o = out + (size_t)t * width;
  TC* c = copy ? copy + (size_t)t * width : nullptr;
  // (never read outside a table; an id the host failed to reject poisons its row)
  const bool ok = tok >= 0 && tok < vocab && row >= 0;
  const T* a = table + (size_t)(ok ? tok : 0) * width;
  const T* b = pairs + (size_t)(ok ? row : 0) * width;
  for (int i = threadIdx.x; i < width; i += blockDim.x) {
    const float h = ok ? to_f32<T>(a[i]) + to_f32<T>(b[i]) : __builtin_nanf("");
    o[i] = h;
    if (c) c[i] = from_f32<TC>(h);
  }
}

// `table` [vocab][width] and `pairs` [buckets + 1][width] are of one type; `state`: one int a
// slot, `slot_stride` ints apart.
extern "C" int za_embed_pairs(const int* tokens, const void* table, const void* pairs,
                              int table_dtype, const int* positions, const int* token_seq,
                              const int* seq_start, const int* slot_id, int* state,
                              long long slot_stride, long long buckets, long long mul_prev,
                              long long mul_cur, float* out, void* copy, int copy_dtype,
                              int n_tokens, int width, int vocab, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  if (n_tokens < 0 || width <= 0 || vocab <= 0 || buckets <= 0 || mul_prev < 0 || mul_cur < 0 ||
      mul_prev > 0x7fffffff || mul_cur > 0x7fffffff || slot_stride <= 0 || !tokens || !table ||
      !pairs || !positions || !token_seq || !seq_start || !slot_id || !state || !out)
    return ZA_ERR_ARG;
  dim3 grid(n_tokens), block(256);
#define ZA_EMBED_PAIRS(T, TC)                                                                  \
  hipLaunchKernelGGL((embed_pairs_kernel<T, TC>), grid, block, 0, stream, tokens,              \
                     (const T*)table, (const T*)pairs, positions, token_seq, seq_start, slot_id, \
                     state, slot_stride, buckets, mul_prev, mul_cur, out, (TC*)copy, width, vocab)
  if (table_dtype == 0 && copy_dtype == 0) ZA_EMBED_PAIRS(float, float);
  else if (table_dtype == 0 && copy_dtype == 1) ZA_EMBED_PAIRS(float, bf16_t);
  else if (table_dtype == 1 && copy_dtype == 0) ZA_EMBED_PAIRS(bf16_t, float);
  else if (table_dtype == 1 && copy_dtype == 1) ZA_EMBED_PAIRS(bf16_t, bf16_t);
  else return ZA_ERR_UNSUPPORTED;
#undef ZA_EMBED_PAIRS
  return za_launch_status();
}

// The rows that open the stream, normed:  h = table[tokens[t]],
//   out[t] = h / sqrt(mean(h^2) + eps) * weight
// in 32-bit, and with `copy` also stored rounded.  One workgroup a token; the row is read a
// second time from the cache where it does not fit the registers.
template <typename T, typename TC>
__global__ void __launch_bounds__(256)
embed_norm_kernel(const int* __restrict__ tokens, const T* __restrict__ table,
                  const float* __restrict__ weight, float* __restrict__ out, TC* __restrict__ copy,
                  int width, int vocab, float eps) {
  constexpr int KEEP = 8;
  __shared__ float scratch[16];
  const int t = blockIdx.x, tid = threadIdx.x;
  const int tok = tokens[t];
  // (never read outside the table; an id the host failed to reject poisons its row)
  const bool ok = tok >= 0 && tok < vocab;
  const T* row = table + (size_t)(ok ? tok : 0) * width;
  float* o = out + (size_t)t * width;
  TC* c = copy ? copy + (size_t)t * width : nullptr;
  float kept[KEEP];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int i = tid + k * 256;
    kept[k] = i < width ? to_f32<T>(row[i]) : 0.f;
    ss += kept[k] * kept[k];
  }
  for (int i = tid + KEEP * 256; i < width; i += 256) {
    const float v = to_f32<T>(row[i]);
    ss += v * v;
  }
  ss = block_sum(ss, scratch);
  const float f = ok ? 1.0f / sqrtf(ss / (float)width + eps) : __builtin_nanf("");
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int i = tid + k * 256;
    if (i < width) {
      const float h = kept[k] * f * weight[i];
      o[i] = h;
      if (c) c[i] = from_f32<TC>(h);
    }
  }
  for (int i = tid + KEEP * 256; i < width; i += 256) {
    const float h = to_f32<T>(row[i]) * f * weight[i];
    o[i] = h;
    if (c) c[i] = from_f32<TC>(h);
  }
}

extern "C" int za_embed_norm(const int* tokens, const void* table, int table_dtype,
                             const float* weight, float* out, void* copy, int copy_dtype,
                             int n_tokens, int width, int vocab, float eps, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  if (n_tokens < 0 || width <= 0 || vocab <= 0 || !tokens || !table || !weight || !out)
    return ZA_ERR_ARG;
  dim3 grid(n_tokens), block(256);
#define ZA_EMBED_NORM(T, TC)                                                                 \
  hipLaunchKernelGGL((embed_norm_kernel<T, TC>), grid, block, 0, stream, tokens,             \
                     (const T*)table, weight, out, (TC*)copy, width, vocab, eps)
  if (table_dtype == 0 && copy_dtype == 0) ZA_EMBED_NORM(float, float);
  else if (table_dtype == 0 && copy_dtype == 1) ZA_EMBED_NORM(float, bf16_t);
  else if (table_dtype == 1 && copy_dtype == 0) ZA_EMBED_NORM(bf16_t, float);
  else if (table_dtype == 1 && copy_dtype == 1) ZA_EMBED_NORM(bf16_t, bf16_t);
  else return ZA_ERR_UNSUPPORTED;
#undef ZA_EMBED_NORM
  return za_launch_status();
}
