// What the attention kernels share: what a design adds to scores and masks, reductions over
// the lanes of a query row, page arithmetic, and the merge of partial results.
#pragma once

#include <math.h>

#include "common.h"

#define AT_MAX_D 256
#define AT_DPL (AT_MAX_D / 64)       // head-dim elements per lane, at most
#define ZA_LOG2E 1.44269504088896341f

// What a design may add to the score of a (query, key) pair and to the softmax; every
// field's zero means "not there", and every kernel of this file takes the struct:
//   temperature   q at position p counts (1 + qt_coef * ln(floor((p + 1) / qt_every) + 1))
//                 times (qt_every > 0)
//   cap           s <- softcap * tanh(s / softcap) after the scale (softcap > 0)
//   sink          the softmax's denominator also holds exp(sink[head]): a term with no key
//                 and no value, neither scaled nor capped, counted once however the
//                 context is cut (the kernel that sees the whole context adds it at its end,
//                 otherwise the merge of the ranges does)
//   chunks        positions are counted in chunks of `chunk` from the sequence's start, and
//                 a query sees the keys of its own chunk only (chunk > 0); in the
//                 matrix-core kernels the `SHAPED` instantiations know it
//   kept keys     the first `keep` keys of the sequence count for every query behind them,
//                 whatever the window (the general kernel and attention_planes.hip)
struct ScoreExtras {
  float softcap;
  const float* sink;
  float qt_coef;
  int qt_every;
  int chunk;
  int keep;
};

// first key a query at `position` sees when positions are counted in chunks (0 without)
__device__ __forceinline__ int chunk_start(const ScoreExtras& ex, int position) {
  return ex.chunk > 0 && position > 0 ? (position / ex.chunk) * ex.chunk : 0;
}

// `base2`: the partial maxima are whole numbers on the base-2 scale (what the matrix-core
// kernels keep), so a partial result's weight 2^(m_z - m) is an exact power of two.
template <typename T>
__global__ void __launch_bounds__(64)
attention_combine_kernel(const float* __restrict__ part_acc, const float* __restrict__ part_ml,
                         T* __restrict__ out, int d, int nsplit, int base2,
                         const float* __restrict__ sink, int nh) {
  // `sink`: one number a head whose exponential joins the denominator once (none if null)
  const size_t row = blockIdx.x;  // token * nh + head
  const int lane = threadIdx.x;
  float mx = -INFINITY;
  for (int z = 0; z < nsplit; ++z) mx = fmaxf(mx, part_ml[(row * nsplit + z) * 2]);
  float total = 0.f;
  float acc[AT_DPL];
#pragma unroll
  for (int c = 0; c < AT_DPL; ++c) acc[c] = 0.f;
  for (int z = 0; z < nsplit; ++z) {
    const float mz = part_ml[(row * nsplit + z) * 2];
    const float lz = part_ml[(row * nsplit + z) * 2 + 1];
    if (!(mz > -INFINITY)) continue;
    const float w = base2 ? ldexpf(1.0f, (int)(mz - mx)) : expf(mz - mx);
    total += lz * w;
    const float* pa = part_acc + (row * nsplit + z) * d;
#pragma unroll
    for (int c = 0; c < AT_DPL; ++c) {
      const int dd = lane + 64 * c;
      if (dd < d) acc[c] = fmaf(pa[dd], w, acc[c]);
    }
  }
  if (sink && mx > -INFINITY) {
    const float sk = sink[row % nh];
    total += base2 ? exp2f(sk * 1.4426950408889634f - mx) : expf(sk - mx);
  }
  const float inv = total > 0.f ? 1.0f / total : 0.f;
#pragma unroll
  for (int c = 0; c < AT_DPL; ++c) {
    const int dd = lane + 64 * c;
    if (dd < d) out[row * d + dd] = from_f32<T>(acc[c] * inv);
  }
}

// A query row's scores for a tile are spread over the four lanes l, l ^ 16, l ^ 32,
// l ^ 48.  The swap instructions exchange 16-lane rows (odd rows of the first operand
// with even rows of the second) and 32-lane halves between two registers; fed the
// same value twice they leave in each lane its own value and its partner's, in one
// vector instruction each and without a trip through LDS.
__device__ __forceinline__ float quad_max(float x) {
  const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false,
                                                  false);
  const float y = fmaxf(__uint_as_float(a[0]), __uint_as_float(a[1]));
  const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(y), __float_as_uint(y), false,
                                                  false);
  return fmaxf(__uint_as_float(b[0]), __uint_as_float(b[1]));
}
__device__ __forceinline__ float quad_sum(float x) {
  const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(x), __float_as_uint(x), false,
                                                  false);
  const float y = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(y), __float_as_uint(y), false,
                                                  false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

// Key position -> block-table entry and offset in the page.  Page sizes are powers of
// two nearly always: `shift` is then log2(page_size) and the division (some thirty
// instructions, several times per tile) becomes a shift; otherwise `shift` is -1.
__device__ __forceinline__ int page_shift_of(int page_size) {
  return (page_size & (page_size - 1)) == 0 ? __ffs(page_size) - 1 : -1;
}
__device__ __forceinline__ int page_entry(int kp, int page_size, int shift) {
  return shift >= 0 ? kp >> shift : kp / page_size;
}
__device__ __forceinline__ int page_offset(int kp, int page_size, int shift) {
  return shift >= 0 ? kp & (page_size - 1) : kp % page_size;
}
