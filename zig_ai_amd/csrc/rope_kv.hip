// Per-head RMSNorm of queries and keys, rotary position encoding, and the
// scatter of keys and values into their cache pages: one pass over the fused
// q|k|v projection.
//
// Per (token, head), in 32-bit:
//   q, k:  x <- x * (1/sqrt(mean(x^2) + eps)) * w[head_dim]      (if norm weights are given;
//          before the rotation, never on v: /root/reference/src/transformer/hybrid_attn.zig:371-382)
//   q, k:  for pair p < rotary_dim/2 with angle = position * inv_freq[p]:
//            (a, b) <- (a cos - b sin, a sin + b cos)
//          (/root/reference/src/transformer/rope.zig:40-56); the pair is (p, p + rotary_dim/2)
//          for "half" pairing (the reference's device kernel,
//          /root/reference/src/cuda/layer_kernels.cu:353-365) or (2p, 2p+1) for "adjacent"
//          pairing (rope.zig:46-53).  Elements beyond rotary_dim pass through.
//   k -> cache[page][0][kv_head][offset][head_dim],  slot = page * page_size + offset
//   v -> cache[page][1][kv_head][head_dim][offset]   (turned round: the attention kernels
//        read, for one head-dimension element, consecutive keys side by side)
//   q    -> q_out[token][head][head_dim]
#include "common.h"
#include "rope_math.h"

#define RK_MAX_D 256

template <typename T>
__global__ void __launch_bounds__(256)
qk_norm_rope_kv_write_kernel(const T* __restrict__ qkv, const int* __restrict__ positions,
                             const int* __restrict__ slots, const float* __restrict__ q_norm_w,
                             const float* __restrict__ k_norm_w, const float* __restrict__ inv_freq,
                             T* __restrict__ q_out, T* __restrict__ kv_cache, int nh, int nkv, int d,
                             int rot, int adjacent, float eps, int page_size, int write_kv, int dv,
                             int row_stride, float magnitude) {
  // `dv`: width of a value head (queries and keys have `d`); a row of `qkv` holds
  // nh*d + nkv*d + nkv*dv elements (and may be longer: `row_stride`), a page the keys of
  // all heads and then the values of all heads.  `magnitude`: factor on cosine and sine.
  __shared__ float vec[4][RK_MAX_D];
  const int t = blockIdx.x;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int head = blockIdx.y * 4 + wave;  // 0..nh-1: q; then nkv k heads; then nkv v heads
  const int total = nh + 2 * nkv;
  const bool active = head < total;
  const bool is_q = head < nh;
  const bool is_k = !is_q && head < nh + nkv;
  float* s = vec[wave];

  float ss = 0.f;
  const bool is_v = active && !is_q && !is_k;
  const int width = is_v ? dv : d;
  if (active) {
    const T* src = qkv + (size_t)t * row_stride +
                   (is_v ? (size_t)(nh + nkv) * d + (size_t)(head - nh - nkv) * dv : (size_t)head * d);
    for (int i = lane; i < width; i += 64) {
      const float v = to_f32<T>(src[i]);
      s[i] = v;
      ss += v * v;
    }
  }
  ss = wave_sum(ss);
  __syncthreads();
  const float* nw = is_q ? q_norm_w : (is_k ? k_norm_w : nullptr);
  if (active && nw) {
    const float scale = 1.0f / sqrtf(ss / (float)d + eps);
    for (int i = lane; i < d; i += 64) s[i] = s[i] * scale * nw[i];
  }
  __syncthreads();
  if (active && (is_q || is_k) && rot > 0) {
    const float pos = (float)positions[t];
    const int half = rot / 2;
    for (int p = lane; p < half; p += 64) {
      const int i0 = adjacent ? 2 * p : p;
      const int i1 = adjacent ? 2 * p + 1 : p + half;
      const float angle = pos * inv_freq[p];
      float sn, cs;
      sincosf(angle, &sn, &cs);
      cs *= magnitude;
      sn *= magnitude;
      const float a = s[i0], b = s[i1];
      s[i0] = a * cs - b * sn;
      s[i1] = a * sn + b * cs;
    }
  }
  __syncthreads();
  if (!active) return;
  if (is_q) {
    T* dst = q_out + ((size_t)t * nh + head) * d;
    for (int i = lane; i < d; i += 64) dst[i] = from_f32<T>(s[i]);
  } else if (write_kv) {
    const int slot = slots[t];
    if (slot < 0) return;
    const int page = slot / page_size, off = slot % page_size;
    const int kvh = is_k ? head - nh : head - nh - nkv;
    T* pg = kv_cache + (size_t)page * nkv * page_size * (d + dv);
    if (is_k) {
      T* dst = pg + ((size_t)kvh * page_size + off) * d;
      for (int i = lane; i < d; i += 64) dst[i] = from_f32<T>(s[i]);
    } else {
      T* dst = pg + (size_t)nkv * page_size * d + (size_t)kvh * dv * page_size + off;
      for (int i = lane; i < dv; i += 64) dst[(size_t)i * page_size] = from_f32<T>(s[i]);
    }
  }
}

// The same for head sizes that are powers of two: a block per token, D / 8 lanes per
// head with 16-byte accesses, the token's cosines and sines computed once for all its
// heads, the mean square summed over the head's lanes with lane shuffles.  Half
// pairing needs rotary_dim / 2 to be a multiple of 8, so that a lane's partner
// elements all sit in one other lane.
template <typename T, int D>
__global__ void __launch_bounds__(256)
qk_norm_rope_kv_write_pow2_kernel(const T* __restrict__ qkv, const int* __restrict__ positions,
                                  const int* __restrict__ slots,
                                  const float* __restrict__ q_norm_w,
                                  const float* __restrict__ k_norm_w,
                                  const float* __restrict__ inv_freq, T* __restrict__ q_out,
                                  T* __restrict__ kv_cache, int nh, int nkv, int rot, int adjacent,
                                  float eps, int page_size, int write_kv, int n_tokens,
                                  int value_blocks) {
  constexpr int LPH = D / 8;   // lanes per head
  __shared__ float cs_tab[D / 2], sn_tab[D / 2];
  if ((int)blockIdx.x < value_blocks) {
    // ---- values only, for steps of many tokens: a wave takes eight consecutive tokens
    // and stores, where these lie at eight neighbouring offsets of one page from a
    // multiple of eight on (a stretch of a prompt), each head-dim element's eight
    // values with one 16-byte access (32 bytes in 32-bit) instead of eight 2-byte
    // ones a page row apart.  Other groups (a request's edge, single tokens between
    // prompts) store element by element.
    const int lane = threadIdx.x & 63;
    const int t0 = ((int)blockIdx.x * 4 + ((int)threadIdx.x >> 6)) * 8;   // a wave's 8 tokens
    if (t0 >= n_tokens) return;
    const int total = nh + 2 * nkv;
    int slot[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) slot[j] = t0 + j < n_tokens ? slots[t0 + j] : -1;
    bool side_by_side = page_size % 8 == 0 && slot[0] >= 0 && slot[0] % 8 == 0;
#pragma unroll
    for (int j = 1; j < 8; ++j) side_by_side = side_by_side && slot[j] == slot[0] + j;
    for (int pair = lane; pair < nkv * LPH; pair += 64) {
      const int hv = pair / LPH, e0 = (pair % LPH) * 8;
      float x[8][8];
#pragma unroll
      for (int j = 0; j < 8; ++j)
        if (t0 + j < n_tokens)
          load8<T>(qkv + ((size_t)(t0 + j) * total + nh + nkv + hv) * D + e0, x[j]);
      if (side_by_side) {
        T* dst = kv_cache + (((size_t)(slot[0] / page_size) * 2 + 1) * nkv + hv) * page_size * D +
                 (size_t)e0 * page_size + slot[0] % page_size;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          float run[8];
#pragma unroll
          for (int j = 0; j < 8; ++j) run[j] = x[j][i];
          store8<T>(dst + (size_t)i * page_size, run);
        }
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j)
          if (slot[j] >= 0) {
            T* dst = kv_cache +
                     (((size_t)(slot[j] / page_size) * 2 + 1) * nkv + hv) * page_size * D +
                     (size_t)e0 * page_size + slot[j] % page_size;
#pragma unroll
            for (int i = 0; i < 8; ++i) dst[(size_t)i * page_size] = from_f32<T>(x[j][i]);
          }
      }
    }
    return;
  }
  const int t = (int)blockIdx.x - value_blocks;
  const int half = rot / 2;
  const int total = nh + 2 * nkv;
  const int heads_here = value_blocks > 0 ? nh + nkv : total;   // values go their own way
  const int li = threadIdx.x % LPH;
  const int e0 = li * 8;        // this lane's first element of the head
  // this thread's first head is requested before the angles are worked out, and each
  // further head while the one before it is being processed
  float xn[8];
  if ((int)threadIdx.x / LPH < heads_here)
    load8<T>(qkv + ((size_t)t * total + threadIdx.x / LPH) * D + e0, xn);
  if ((int)threadIdx.x < half) {
    float sn, cs;
    rope_angle(positions[t], inv_freq[threadIdx.x], &cs, &sn);
    cs_tab[threadIdx.x] = cs;
    sn_tab[threadIdx.x] = sn;
  }
  __syncthreads();
  for (int head = threadIdx.x / LPH; head < heads_here; head += 256 / LPH) {
    const bool is_q = head < nh;
    const bool is_k = !is_q && head < nh + nkv;
    float x[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) x[i] = xn[i];
    if (head + 256 / LPH < heads_here)
      load8<T>(qkv + ((size_t)t * total + head + 256 / LPH) * D + e0, xn);
    const float* nw = is_q ? q_norm_w : (is_k ? k_norm_w : nullptr);
    if (nw) {
      // (the decode attention's prologue adds the lanes' sums up in this order too:
      // partners 4 lanes apart first, then 2, then 1)
      float ss = rope_sum_squares8(x);
#pragma unroll
      for (int o = LPH / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
      const float scale = rope_rms_scale(ss, D, eps);
      float w8[8];
      load8<float>(nw + e0, w8);     // two 16-byte loads, not eight of 4 bytes
      rope_scale8(x, scale, w8);
    }
    if ((is_q || is_k) && rot > 0) {
      if (adjacent) {
#pragma unroll
        for (int i = 0; i < 8; i += 2)
          if (e0 + i + 1 < rot) {
            const int p = (e0 + i) / 2;
            const float a = x[i], b = x[i + 1], cs = cs_tab[p], sn = sn_tab[p];
            x[i] = a * cs - b * sn;
            x[i + 1] = a * sn + b * cs;
          }
      } else {
        const bool low = e0 < half, in_rot = e0 < rot;
        const int lane = threadIdx.x & 63;
        const int partner = in_rot ? (low ? lane + half / 8 : lane - half / 8) : lane;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          const float other = __shfl(x[i], partner, 64);
          if (in_rot) {
            const int p = low ? e0 + i : e0 + i - half;
            const float cs = cs_tab[p], sn = sn_tab[p];
            x[i] = low ? rope_rotate_low(x[i], other, cs, sn) : rope_rotate_high(x[i], other, cs, sn);
          }
        }
      }
    }
    if (is_q) {
      store8<T>(q_out + ((size_t)t * nh + head) * D + e0, x);
    } else if (write_kv) {
      const int slot = slots[t];
      if (slot >= 0) {
        const int page = slot / page_size, off = slot % page_size;
        if (is_k) {
          store8<T>(kv_cache + ((((size_t)page * 2) * nkv + (head - nh)) * page_size + off) * D + e0,
                    x);
        } else {
          T* dst = kv_cache + (((size_t)page * 2 + 1) * nkv + (head - nh - nkv)) * page_size * D +
                   (size_t)e0 * page_size + off;
#pragma unroll
          for (int i = 0; i < 8; ++i) dst[(size_t)i * page_size] = from_f32<T>(x[i]);
        }
      }
    }
  }
}

#define RK_VALUE_BLOCKS_FROM 128   // tokens in a step from which values get blocks of their own

template <typename T>
static bool launch_pow2(const void* qkv, const int* positions, const int* slots,
                        const float* q_norm_w, const float* k_norm_w, const float* inv_freq,
                        void* q_out, void* kv_cache, int n_tokens, int nh, int nkv, int d, int rot,
                        int adjacent, float eps, int page_size, int write_kv,
                        hipStream_t stream) {
  if (!adjacent && (rot / 2) % 8 != 0) return false;
  // many tokens (prompt portions): the values are written by blocks of their own, first
  // in the grid, 32 tokens each
  const int value_blocks = (write_kv && n_tokens >= RK_VALUE_BLOCKS_FROM) ? (n_tokens + 31) / 32 : 0;
#define ZA_RK_LAUNCH(DD)                                                                        \
  hipLaunchKernelGGL((qk_norm_rope_kv_write_pow2_kernel<T, DD>), dim3(n_tokens + value_blocks),  \
                     dim3(256), 0, stream, (const T*)qkv, positions, slots, q_norm_w, k_norm_w,  \
                     inv_freq, (T*)q_out, (T*)kv_cache, nh, nkv, rot, adjacent, eps, page_size,  \
                     write_kv, n_tokens, value_blocks)
  switch (d) {
    case 16: ZA_RK_LAUNCH(16); return true;
    case 32: ZA_RK_LAUNCH(32); return true;
    case 64: ZA_RK_LAUNCH(64); return true;
    case 128: ZA_RK_LAUNCH(128); return true;
    case 256: ZA_RK_LAUNCH(256); return true;
    default: return false;
  }
#undef ZA_RK_LAUNCH
}

extern "C" int za_qk_norm_rope_kv_write(const void* qkv, const int* positions, const int* slots,
                                        const float* q_norm_w, const float* k_norm_w,
                                        const float* inv_freq, void* q_out, void* kv_cache,
                                        int dtype, int n_tokens, int nh, int nkv, int d, int rot,
                                        int adjacent, float eps, int page_size, int write_kv,
                                        hipStream_t stream) {
  if (n_tokens == 0) return 0;
  if (n_tokens < 0 || nh <= 0 || nkv <= 0 || d <= 0 || !qkv || !positions || !q_out)
    return ZA_ERR_ARG;
  if (d > RK_MAX_D || rot < 0 || rot > d || (rot % 2) != 0) return ZA_ERR_UNSUPPORTED;
  if (rot > 0 && !inv_freq) return ZA_ERR_ARG;
  if (write_kv && (!kv_cache || !slots || page_size <= 0)) return ZA_ERR_ARG;
  if (dtype != 0 && dtype != 1) return ZA_ERR_UNSUPPORTED;
  const bool fast =
      dtype == 0 ? launch_pow2<float>(qkv, positions, slots, q_norm_w, k_norm_w, inv_freq, q_out,
                                      kv_cache, n_tokens, nh, nkv, d, rot, adjacent, eps,
                                      page_size, write_kv, stream)
                 : launch_pow2<bf16_t>(qkv, positions, slots, q_norm_w, k_norm_w, inv_freq, q_out,
                                       kv_cache, n_tokens, nh, nkv, d, rot, adjacent, eps,
                                       page_size, write_kv, stream);
  if (fast) return za_launch_status();
  dim3 grid(n_tokens, (nh + 2 * nkv + 3) / 4), block(256);
  if (dtype == 0) {
    hipLaunchKernelGGL((qk_norm_rope_kv_write_kernel<float>), grid, block, 0, stream,
                       (const float*)qkv, positions, slots, q_norm_w, k_norm_w, inv_freq,
                       (float*)q_out, (float*)kv_cache, nh, nkv, d, rot, adjacent, eps, page_size,
                       write_kv, d, (nh + 2 * nkv) * d, 1.0f);
  } else if (dtype == 1) {
    hipLaunchKernelGGL((qk_norm_rope_kv_write_kernel<bf16_t>), grid, block, 0, stream,
                       (const bf16_t*)qkv, positions, slots, q_norm_w, k_norm_w, inv_freq,
                       (bf16_t*)q_out, (bf16_t*)kv_cache, nh, nkv, d, rot, adjacent, eps,
                       page_size, write_kv, d, (nh + 2 * nkv) * d, 1.0f);
  } else {
    return ZA_ERR_UNSUPPORTED;
  }
  return za_launch_status();
}

// The same for values of another width than the keys' (`dv`), rows of `qkv` that hold
// more than q|k|v (`row_stride` elements a row: a gate's columns behind them, say), and a factor
// `magnitude` on cosine and sine.  nkv == 0: the rows hold queries only, nothing is stored.
extern "C" int za_qk_norm_rope_kv_write_wide(const void* qkv, const int* positions,
                                             const int* slots, const float* q_norm_w,
                                             const float* k_norm_w, const float* inv_freq,
                                             void* q_out, void* kv_cache, int dtype, int n_tokens,
                                             int nh, int nkv, int d, int dv, int row_stride,
                                             int rot, int adjacent, float eps, int page_size,
                                             int write_kv, float magnitude, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  if (n_tokens < 0 || nh <= 0 || nkv < 0 || d <= 0 || dv <= 0 || !qkv || !positions || !q_out ||
      row_stride < (nh + nkv) * d + nkv * dv || (nkv == 0 && write_kv))
    return ZA_ERR_ARG;
  if (d > RK_MAX_D || dv > RK_MAX_D || rot < 0 || rot > d || (rot % 2) != 0)
    return ZA_ERR_UNSUPPORTED;
  if (rot > 0 && !inv_freq) return ZA_ERR_ARG;
  if (write_kv && (!kv_cache || !slots || page_size <= 0)) return ZA_ERR_ARG;
  dim3 grid(n_tokens, (nh + 2 * nkv + 3) / 4), block(256);
  if (dtype == 0) {
    hipLaunchKernelGGL((qk_norm_rope_kv_write_kernel<float>), grid, block, 0, stream,
                       (const float*)qkv, positions, slots, q_norm_w, k_norm_w, inv_freq,
                       (float*)q_out, (float*)kv_cache, nh, nkv, d, rot, adjacent, eps, page_size,
                       write_kv, dv, row_stride, magnitude);
  } else if (dtype == 1) {
    hipLaunchKernelGGL((qk_norm_rope_kv_write_kernel<bf16_t>), grid, block, 0, stream,
                       (const bf16_t*)qkv, positions, slots, q_norm_w, k_norm_w, inv_freq,
                       (bf16_t*)q_out, (bf16_t*)kv_cache, nh, nkv, d, rot, adjacent, eps,
                       page_size, write_kv, dv, row_stride, magnitude);
  } else {
    return ZA_ERR_UNSUPPORTED;
  }
  return za_launch_status();
}

// Queries and keys normed over their WHOLE projection instead of head by head:
//   q row [nh * d]:  x <- x / sqrt(sum(x^2) / q_count + eps) * q_norm_w[nh * d]
//   k row [nkv * d]: likewise with k_count and k_norm_w[nkv * d]
// (q_count, k_count: how many elements the mean is taken over, fewer than the row has where
// heads are filled up with zeros), then the rotation of every head and the stores of the
// kernels above, `dv`, `row_stride` and `magnitude` as there.  nkv == 0: the rows hold queries
// only, nothing is stored (a layer that reads another layer's keys and values).
//
// A workgroup a token, NP pieces of eight elements a thread, held in registers.  The two sums
// of squares meet once; every thread norms its own pieces and leaves them in LDS, where the
// rotation finds a piece's partners.  In steps of many tokens the values are
// stored by workgroups of their own, first in the grid: a wave takes eight consecutive tokens
// and, where these lie side by side in one page, stores a head-dim element's eight values with
// one access.
template <typename T, int NP>
__global__ void __launch_bounds__(512)
qk_row_norm_rope_kv_write_kernel(const T* __restrict__ qkv, const int* __restrict__ positions,
                                 const int* __restrict__ slots, const float* __restrict__ q_norm_w,
                                 const float* __restrict__ k_norm_w,
                                 const float* __restrict__ inv_freq, T* __restrict__ q_out,
                                 T* __restrict__ kv_cache, int nh, int nkv, int d, int dv,
                                 int row_stride, int rot, int adjacent, float eps, float q_count,
                                 float k_count, float magnitude, int page_size, int write_kv,
                                 int n_tokens, int value_blocks) {
  extern __shared__ __attribute__((aligned(16))) float rows_lds[];   // [(nh + nkv) * d][rot]
  __shared__ float sums[2][16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int n_threads = blockDim.x, n_waves = n_threads >> 6;
  const size_t page_elems = (size_t)nkv * page_size * (d + dv);
  const size_t value_base = (size_t)nkv * page_size * d;
  if ((int)blockIdx.x < value_blocks) {
    const int t0 = ((int)blockIdx.x * n_waves + wave) * 8;   // a wave's 8 tokens
    if (t0 >= n_tokens) return;
    int slot[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) slot[j] = t0 + j < n_tokens ? slots[t0 + j] : -1;
    bool side_by_side = page_size % 8 == 0 && slot[0] >= 0 && slot[0] % 8 == 0;
#pragma unroll
    for (int j = 1; j < 8; ++j) side_by_side = side_by_side && slot[j] == slot[0] + j;
    constexpr int E = 16 / (int)sizeof(T);             // elements of a 16-byte piece
    typedef T piece_t __attribute__((ext_vector_type(E)));
    typedef T run_t __attribute__((ext_vector_type(8)));
    const int pieces = nkv * dv / E;
    const T* src = qkv + (size_t)t0 * row_stride + (size_t)(nh + nkv) * d;
    for (int piece = lane; piece < pieces; piece += 64) {
      piece_t x[8];
#pragma unroll
      for (int j = 0; j < 8; ++j)      // (a token beyond the last reads the last one again)
        x[j] = *reinterpret_cast<const piece_t*>(
            src + (size_t)(min(t0 + j, n_tokens - 1) - t0) * row_stride + piece * E);
      if (side_by_side) {
        T* dst = kv_cache + (size_t)(slot[0] / page_size) * page_elems + value_base +
                 (size_t)piece * E * page_size + slot[0] % page_size;
#pragma unroll
        for (int i = 0; i < E; ++i) {
          run_t run;
#pragma unroll
          for (int j = 0; j < 8; ++j) run[j] = x[j][i];
          *reinterpret_cast<run_t*>(dst + (size_t)i * page_size) = run;
        }
      } else {
#pragma unroll 1
        for (int j = 0; j < 8 && t0 + j < n_tokens; ++j) {   // (a rare group: tokens one by one)
          const int place = slots[t0 + j];
          if (place < 0) continue;
          const piece_t one = *reinterpret_cast<const piece_t*>(src + (size_t)j * row_stride + piece * E);
          T* dst = kv_cache + (size_t)(place / page_size) * page_elems + value_base +
                   (size_t)piece * E * page_size + place % page_size;
#pragma unroll
          for (int i = 0; i < E; ++i) dst[(size_t)i * page_size] = one[i];
        }
      }
    }
    return;
  }
  const int t = (int)blockIdx.x - value_blocks;
  const T* row = qkv + (size_t)t * row_stride;
  const int half = rot / 2;
  const int q_pieces = nh * d / 8;
  const int pieces = q_pieces + (write_kv ? nkv * d / 8 : 0);
  float* cs_tab = rows_lds + (size_t)(nh + nkv) * d;
  float* sn_tab = cs_tab + half;

  // everything the token needs is requested at once
  const int slot = write_kv ? slots[t] : -1;
  float x[NP][8], w[NP][8];
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int piece = tid + j * n_threads;
    if (piece < pieces) {
      load8<T>(row + piece * 8, x[j]);
      load8<float>(piece < q_pieces ? q_norm_w + piece * 8 : k_norm_w + (piece - q_pieces) * 8, w[j]);
    }
  }
  for (int p = tid; p < half; p += n_threads) {
    float cs, sn;
    rope_angle(positions[t], inv_freq[p], &cs, &sn);
    cs_tab[p] = cs * magnitude;
    sn_tab[p] = sn * magnitude;
  }
  float qs = 0.f, ks = 0.f;
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int piece = tid + j * n_threads;
    if (piece >= pieces) continue;
    const float ss = rope_sum_squares8(x[j]);
    if (piece < q_pieces) qs += ss; else ks += ss;
  }
  qs = wave_sum(qs);
  ks = wave_sum(ks);
  if (lane == 0) {
    sums[0][wave] = qs;
    sums[1][wave] = ks;
  }
  __syncthreads();
  qs = ks = 0.f;
  for (int i = 0; i < n_waves; ++i) {
    qs += sums[0][i];
    ks += sums[1][i];
  }
  const float q_scale = 1.0f / sqrtf(qs / q_count + eps);
  const float k_scale = 1.0f / sqrtf(ks / k_count + eps);
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int piece = tid + j * n_threads;
    if (piece >= pieces) continue;
    rope_scale8(x[j], piece < q_pieces ? q_scale : k_scale, w[j]);
    store8<float>(rows_lds + piece * 8, x[j]);
  }
  __syncthreads();
  T* pg = slot >= 0 ? kv_cache + (size_t)(slot / page_size) * page_elems : nullptr;
  const int off = slot >= 0 ? slot % page_size : 0;
  const bool whole_pieces = !adjacent && half % 8 == 0;   // a piece's partners are one piece
#pragma unroll
  for (int j = 0; j < NP; ++j) {
    const int piece = tid + j * n_threads;
    if (piece >= pieces) continue;
    const int head = piece * 8 / d, e0 = piece * 8 % d;
    const float* h = rows_lds + (size_t)head * d;
    if (e0 < rot && whole_pieces) {
      const bool low = e0 < half;
      float other[8], cs[8], sn[8];
      load8<float>(h + (low ? e0 + half : e0 - half), other);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        cs[i] = cs_tab[(low ? e0 : e0 - half) + i];
        sn[i] = sn_tab[(low ? e0 : e0 - half) + i];
      }
#pragma unroll
      for (int i = 0; i < 8; ++i)
        x[j][i] = low ? rope_rotate_low(x[j][i], other[i], cs[i], sn[i])
                      : rope_rotate_high(x[j][i], other[i], cs[i], sn[i]);
    } else if (e0 < rot) {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int e = e0 + i;
        if (e >= rot) continue;
        if (adjacent) {
          const float other = h[e ^ 1], cs = cs_tab[e >> 1], sn = sn_tab[e >> 1];
          x[j][i] = (e & 1) ? rope_rotate_high(x[j][i], other, cs, sn)
                            : rope_rotate_low(x[j][i], other, cs, sn);
        } else if (e < half) {
          x[j][i] = rope_rotate_low(x[j][i], h[e + half], cs_tab[e], sn_tab[e]);
        } else {
          x[j][i] = rope_rotate_high(x[j][i], h[e - half], cs_tab[e - half], sn_tab[e - half]);
        }
      }
    }
    if (piece < q_pieces)
      store8<T>(q_out + (size_t)t * nh * d + piece * 8, x[j]);
    else if (pg)
      store8<T>(pg + ((size_t)(head - nh) * page_size + off) * d + e0, x[j]);
  }
  if (pg && value_blocks == 0) {
    const T* v = row + (size_t)(nh + nkv) * d;
    for (int i = tid; i < nkv * dv; i += n_threads) pg[value_base + (size_t)i * page_size + off] = v[i];
  }
}

#define RK_ROW_MAX_LDS (128 * 1024)

extern "C" int za_qk_row_norm_rope_kv_write(const void* qkv, const int* positions, const int* slots,
                                            const float* q_norm_w, const float* k_norm_w,
                                            const float* inv_freq, void* q_out, void* kv_cache,
                                            int dtype, int n_tokens, int nh, int nkv, int d, int dv,
                                            int row_stride, int rot, int adjacent, float eps,
                                            float q_count, float k_count, float magnitude,
                                            int page_size, int write_kv, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  if (n_tokens < 0 || nh <= 0 || nkv < 0 || d <= 0 || dv <= 0 || !qkv || !positions || !q_out ||
      !q_norm_w || row_stride < (nh + nkv) * d + nkv * dv || !(q_count > 0.f))
    return ZA_ERR_ARG;
  if (d % 8 != 0 || dv % 8 != 0 || row_stride % 8 != 0 || rot < 0 || rot > d || rot % 2 != 0)
    return ZA_ERR_UNSUPPORTED;
  if (rot > 0 && !inv_freq) return ZA_ERR_ARG;
  if (write_kv && (nkv == 0 || !kv_cache || !slots || !k_norm_w || page_size <= 0 || !(k_count > 0.f)))
    return ZA_ERR_ARG;
  const size_t shmem = ((size_t)(nh + nkv) * d + rot) * sizeof(float);
  if (shmem > RK_ROW_MAX_LDS) return ZA_ERR_UNSUPPORTED;
  const int pieces = nh * d / 8 + (write_kv ? nkv * d / 8 : 0);
  int np = 1;
  while (np < 8 && pieces > np * 512) np *= 2;
  if (pieces > np * 1024) return ZA_ERR_UNSUPPORTED;
  const int threads = ((pieces + np - 1) / np + 63) / 64 * 64;
  const int per_block = threads / 64 * 8;   // tokens whose values a workgroup stores
  const int value_blocks =
      (write_kv && n_tokens >= RK_VALUE_BLOCKS_FROM) ? (n_tokens + per_block - 1) / per_block : 0;
#define ZA_RK_ROW_NP(T, NP)                                                                      \
  {                                                                                              \
    auto kernel = qk_row_norm_rope_kv_write_kernel<T, NP>;                                       \
    static size_t allowed = 48 * 1024;                                                           \
    if (shmem > allowed) {                                                                       \
      const hipError_t e = hipFuncSetAttribute(                                                  \
          (const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)shmem);          \
      if (e != hipSuccess) return (int)e;                                                        \
      allowed = shmem;                                                                           \
    }                                                                                            \
    hipLaunchKernelGGL(kernel, dim3(n_tokens + value_blocks), dim3(threads), shmem, stream,      \
                       (const T*)qkv, positions, slots, q_norm_w, k_norm_w, inv_freq, (T*)q_out, \
                       (T*)kv_cache, nh, nkv, d, dv, row_stride, rot, adjacent, eps, q_count,    \
                       k_count, magnitude, page_size, write_kv, n_tokens, value_blocks);         \
    return za_launch_status();                                                                   \
  }
#define ZA_RK_ROW(T)                  \
  {                                   \
    if (np == 1) ZA_RK_ROW_NP(T, 1)   \
    if (np == 2) ZA_RK_ROW_NP(T, 2)   \
    if (np == 4) ZA_RK_ROW_NP(T, 4)   \
    ZA_RK_ROW_NP(T, 8)                \
  }
  if (dtype == 0) ZA_RK_ROW(float)
  if (dtype == 1) ZA_RK_ROW(bf16_t)
#undef ZA_RK_ROW
#undef ZA_RK_ROW_NP
  return ZA_ERR_UNSUPPORTED;
}
