// Mixers that carry a matrix state from token to token, for any mix of prompt
// portions and single decoded tokens in one launch.  Everything that enters a
// recurrence is 32-bit: the state, decays, step sizes, gates and unit norms.
//
// 1. causal_conv_silu: a depth-wise causal convolution over a request's own inputs
//    followed by silu (or, through za_causal_conv, by nothing),
//      y[t, c] = silu(bias[c] + sum_j taps[c, j] * x[t - (L - 1 - j), c]),
//    the L - 1 inputs before a portion coming from the request's state slot, which
//    afterwards holds the portion's last L - 1 inputs.
//
// 2. matrix_recurrence, per (request, head), with a state S of `dk` rows (key
//    channels) and `dv` columns, in these forms:
//      SSD (state-space duality):   S <- a S + dt * b x^T;          y = S^T c + D x
//          a = exp(-exp(A_log) * dt), dt = softplus(raw + dt_bias)      (one per head)
//      gated delta rule:            S <- diag(g) S;  u = beta (v - S^T k);
//                                   S <- S + k u^T;  o = S^T q
//          g = exp(-exp(A_log) * softplus(raw + dt_bias))   (one per head and key channel)
//          q, k made unit vectors (x / sqrt(sum x^2 + 1e-6)), q times dk^(-1/2),
//          beta = sigmoid(raw)
//      fixed decay (retention):      S <- a_h S + k v^T;             o = S^T q
//          a_h a constant of the head; the SSD walk with dt = 1 and no D, q and k rotated
//          and k scaled beforehand by retention_prepare
//      channel decay (gated linear attention):   S <- diag(a) S + k v^T;   o = S^T q
//          a one number a head and key channel, made from the token by channel_decay_prepare
//    A column of S never meets another column: P neighbouring lanes that split its rows
//    keep one column in registers across all tokens of the portion, read it from the
//    slot at the start and store it at the end.  The slot holds S turned round,
//    [head][column][row], so that a lane's rows are consecutive floats.  What a token
//    brings that does not depend on the state (unit vectors, decays, gates) is computed
//    beforehand, for all tokens at once; a workgroup is one wave that walks the tokens in
//    order with the next tokens' vectors already on their way.
//
// 3. gated_group_norm: y * act(gate) and an RMS norm over equal groups of columns, the
//    gate before or after the norm:
//      gate first:  v = y * act(gate);  out = v / rms(v) * w
//      gate last:   out = y / rms(y) * w * act(gate)
#include <math.h>

#include "common.h"
#include "rope_math.h"

#define RC_MAX_TAPS 8

__device__ __forceinline__ float silu_f(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }
// log(1 + exp(x)) without overflow; no clamp
__device__ __forceinline__ float softplus_f(float x) {
  return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x)));
}

// ------------------------------------------------------------------ convolution
// grid.x: blocks of 256 channels; grid.y: first the blocks of `tokens_per_block`
// tokens (bodies: tokens whose L - 1 predecessors lie in the same portion), then one
// block per request (heads: the first L - 1 tokens of its portion and the state).
// `act`: 1 silu, 0 none.  `TO`: what is stored (the state keeps 32-bit inputs either way).
template <typename T, typename TO>
__global__ void __launch_bounds__(256)
causal_conv_silu_kernel(const T* __restrict__ x, int x_stride, int col0,
                        const float* __restrict__ taps, const float* __restrict__ bias,
                        float* __restrict__ state, long long slot_stride,
                        const int* __restrict__ token_seq, const int* __restrict__ seq_start,
                        const int* __restrict__ slot_id, TO* __restrict__ out, int n_tokens,
                        int C, int L, int body_blocks, int tokens_per_block, int act) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= C) return;
  float w[RC_MAX_TAPS];
#pragma unroll
  for (int j = 0; j < RC_MAX_TAPS; ++j) w[j] = j < L ? taps[(size_t)c * L + j] : 0.f;
  const float b = bias ? bias[c] : 0.f;
  if ((int)blockIdx.y < body_blocks) {
    const int t0 = blockIdx.y * tokens_per_block;
    // the L - 1 inputs before the token stay in registers from one token to the next
    float before[RC_MAX_TAPS];
    bool have = false;
    for (int t = t0; t < t0 + tokens_per_block && t < n_tokens; ++t) {
      const int rel = t - seq_start[token_seq[t]];
      if (rel < L - 1) {
        have = false;
        continue;
      }
      if (!have) {
#pragma unroll
        for (int j = 0; j < RC_MAX_TAPS - 1; ++j)
          before[j] = j < L - 1 ? to_f32<T>(x[(size_t)(t - (L - 1 - j)) * x_stride + col0 + c]) : 0.f;
        have = true;
      }
      const float xi = to_f32<T>(x[(size_t)t * x_stride + col0 + c]);
      float acc = b;
#pragma unroll
      for (int j = 0; j < RC_MAX_TAPS - 1; ++j)
        if (j < L - 1) acc = fmaf(w[j], before[j], acc);
      acc = fmaf(w[L - 1], xi, acc);
      out[(size_t)t * C + c] = from_f32<TO>(act ? silu_f(acc) : acc);
#pragma unroll
      for (int j = 0; j < RC_MAX_TAPS - 1; ++j)
        if (j < L - 2) before[j] = before[j + 1];
      if (L >= 2) before[L - 2] = xi;
    }
    return;
  }
  const int s = blockIdx.y - body_blocks;
  const int start = seq_start[s], n = seq_start[s + 1] - start;
  float* st = state + (size_t)slot_id[s] * slot_stride + (size_t)c * (L - 1);
  float hist[RC_MAX_TAPS];      // the L - 1 inputs before the next token, oldest first
#pragma unroll
  for (int j = 0; j < RC_MAX_TAPS; ++j) hist[j] = j < L - 1 ? st[j] : 0.f;
  const int first = n < L - 1 ? n : L - 1;
  for (int i = 0; i < first; ++i) {
    const float xi = to_f32<T>(x[(size_t)(start + i) * x_stride + col0 + c]);
    float acc = b;
#pragma unroll
    for (int j = 0; j < RC_MAX_TAPS - 1; ++j)
      if (j < L - 1) acc = fmaf(w[j], hist[j], acc);
    acc = fmaf(w[L - 1], xi, acc);
    out[(size_t)(start + i) * C + c] = from_f32<TO>(act ? silu_f(acc) : acc);
#pragma unroll
    for (int j = 0; j < RC_MAX_TAPS - 1; ++j)
      if (j < L - 2) hist[j] = hist[j + 1];
    if (L >= 2) hist[L - 2] = xi;
  }
  if (n > L - 1) {
#pragma unroll
    for (int j = 0; j < RC_MAX_TAPS; ++j)
      if (j < L - 1)
        hist[j] = to_f32<T>(x[(size_t)(start + n - (L - 1) + j) * x_stride + col0 + c]);
  }
#pragma unroll
  for (int j = 0; j < RC_MAX_TAPS; ++j)
    if (j < L - 1) st[j] = hist[j];
}

// `act`: 1 silu, 0 none; `out_dtype`: 0 the result as 32-bit floats, 1 as bfloat16.
extern "C" int za_causal_conv(const void* x, int dtype, int x_stride, int col0, const float* taps,
                              const float* bias, float* state, long long slot_stride,
                              const int* token_seq, const int* seq_start, const int* slot_id,
                              void* out, int out_dtype, int act, int n_tokens, int n_seqs, int C,
                              int L, hipStream_t stream) {
  if (n_tokens == 0 || n_seqs == 0) return 0;
  if (n_tokens < 0 || n_seqs < 0 || C <= 0 || !x || !taps || !state || !token_seq || !seq_start ||
      !slot_id || !out || col0 < 0 || col0 + C > x_stride || slot_stride < (long long)C * (L - 1) ||
      act < 0 || act > 1)
    return ZA_ERR_ARG;
  if (L < 1 || L > RC_MAX_TAPS) return ZA_ERR_UNSUPPORTED;
  const int tpb = 16;
  // (single tokens with a state to read: heads only)
  const int body = (n_tokens > n_seqs || L == 1) ? (n_tokens + tpb - 1) / tpb : 0;
  dim3 grid((C + 255) / 256, body + n_seqs), block(256);
#define ZA_CONV(T, TO)                                                                          \
  hipLaunchKernelGGL((causal_conv_silu_kernel<T, TO>), grid, block, 0, stream, (const T*)x,      \
                     x_stride, col0, taps, bias, state, slot_stride, token_seq, seq_start,       \
                     slot_id, (TO*)out, n_tokens, C, L, body, tpb, act)
  if (dtype == 0 && out_dtype == 0) ZA_CONV(float, float);
  else if (dtype == 1 && out_dtype == 0) ZA_CONV(bf16_t, float);
  else if (dtype == 1 && out_dtype == 1) ZA_CONV(bf16_t, bf16_t);
  else return ZA_ERR_UNSUPPORTED;
#undef ZA_CONV
  return za_launch_status();
}

extern "C" int za_causal_conv_silu(const void* x, int dtype, int x_stride, int col0,
                                   const float* taps, const float* bias, float* state,
                                   long long slot_stride, const int* token_seq,
                                   const int* seq_start, const int* slot_id, float* out,
                                   int n_tokens, int n_seqs, int C, int L, hipStream_t stream) {
  return za_causal_conv(x, dtype, x_stride, col0, taps, bias, state, slot_stride, token_seq,
                        seq_start, slot_id, out, 0, 1, n_tokens, n_seqs, C, L, stream);
}

// ------------------------------------------------------------------- recurrence
// What the two forms read, per token row t:
//   conv   [T][conv_width] 32-bit: the convolution's output.
//          SSD:   x of head h at x_col + h*dv, b of group g at k_col + g*dk, c at q_col + g*dk
//          delta: v of head h at x_col + h*dv (q and k come prepared, see below)
//   proj   [T][proj_stride] storage type (SSD): the raw step size of head h at gate_col + h
//   prep   [T][prep_width] 32-bit (delta), written by delta_prepare_kernel:
//          unit q of key head g at g*dk (times dk^-1/2), unit k at G*dk + g*dk, the decay of
//          head h and key channel i at 2*G*dk + h*dk + i, beta of head h at 2*G*dk + H*dk + h
struct RecurrenceArgs {
  const float* conv;
  int conv_width, q_col, k_col, x_col;
  const void* proj;
  int proj_stride, gate_col, proj_bf16;
  const float* prep;
  int prep_width;
  const float* dt_bias;   // SSD: [H]
  const float* A_log;     // SSD: [H]
  const float* D;         // SSD: [H]
  float* state;           // per slot [H][dv][dk]
  long long slot_stride;
  const int* seq_start;
  const int* slot_id;
  float* out;             // [T][H*dv] 32-bit
  int H, G, dk, dv;
  const float* fixed_decay;   // [H], or null: the SSD walk with this decay, dt = 1 and no
                              // raw step sizes (proj, dt_bias, A_log are not read then)
  const int* seq_count;       // [n], or null: the walkers' token counts, where their rows
                              // are given by (start, count) instead of n + 1 starts
  int decay_col;              // channel decay: the decay of head h and key channel i lies in
                              // `conv` at decay_col + h*dk + i
};

// Forms of the walk: SSD and fixed decay, the delta rule, channel decay.
#define RC_SSD 0
#define RC_DELTA 1
#define RC_CHANNEL 2

// Everything of a token that does not depend on the state, for the delta rule: the unit
// vectors, the decays and the write strengths, once per token instead of once per
// workgroup that walks the token.  grid (tokens, jobs): the first 2*G jobs of a token make
// one unit vector each, the others take 256 decays each, the last one also the betas; a
// job is one trip to memory, and the jobs of a token run side by side.
template <typename T>
__global__ void __launch_bounds__(64)
delta_prepare_kernel(const float* __restrict__ conv, int conv_width, int q_col, int k_col,
                     const T* __restrict__ proj, int proj_stride, int gate_col,
                     const T* __restrict__ decay, int decay_stride,
                     const float* __restrict__ dt_bias, const float* __restrict__ A_log,
                     float* __restrict__ prep, int prep_width, int H, int G, int dk) {
  const int t = blockIdx.x, job = blockIdx.y, lane = threadIdx.x;
  float* row = prep + (size_t)t * prep_width;
  if (job < 2 * G) {
    const int is_k = job >= G, g = is_k ? job - G : job;
    const float* src = conv + (size_t)t * conv_width + (is_k ? k_col : q_col) + g * dk;
    float ss = 0.f;
    for (int i = lane; i < dk; i += 64) { const float v = src[i]; ss += v * v; }
    ss = wave_sum(ss);
    float scale = 1.0f / sqrtf(ss + 1e-6f);
    if (!is_k) scale *= 1.0f / sqrtf((float)dk);
    float* dst = row + (is_k ? G * dk : 0) + g * dk;
    for (int i = lane; i < dk; i += 64) dst[i] = src[i] * scale;
    return;
  }
  const int first = (job - 2 * G) * 256;
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    const int idx = first + lane + 64 * k;
    if (idx < H * dk) {
      const float raw = to_f32<T>(decay[(size_t)t * decay_stride + idx]);
      row[2 * G * dk + idx] = expf(-expf(A_log[idx / dk]) * softplus_f(raw + dt_bias[idx]));
    }
  }
  if (job == (int)gridDim.y - 1)
    for (int h = lane; h < H; h += 64)
      row[2 * G * dk + H * dk + h] =
          sigmoid_f(to_f32<T>(proj[(size_t)t * proj_stride + gate_col + h]));
}

#define RC_ROWS 16   // state rows a lane keeps

// LDS index of key channel i when a lane owns RC_ROWS consecutive channels: four floats of
// padding per lane's share, so that a share starts on a 16-byte boundary (four-float
// reads) and the eight shares that eight neighbouring lanes read at once, 20 floats
// apart, cover the 32 banks once
#define RC_SHARE (RC_ROWS + 4)
__device__ __forceinline__ int lds_at(int i) { return i + (i / RC_ROWS) * 4; }

// The sum over the P neighbouring lanes (a power of two, the group starting at a multiple
// of P) that share a column; every lane of the group gets it.  Up to sixteen lanes the
// partners are reached with the vector unit's own lane patterns (pairs, quads, a half
// row and a row of sixteen mirrored), beyond that through the lane exchange.
template <int CTRL>
__device__ __forceinline__ float dpp_add(float x) {
  const int moved = __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), CTRL, 0xF, 0xF, false);
  return x + __builtin_bit_cast(float, moved);
}

template <int P>
__device__ __forceinline__ float group_sum(float x) {
  if (P >= 2) x = dpp_add<0xB1>(x);     // lanes 1 0 3 2 of every four
  if (P >= 4) x = dpp_add<0x4E>(x);     // lanes 2 3 0 1 of every four
  if (P >= 8) x = dpp_add<0x141>(x);    // a half row of eight, mirrored
  if (P >= 16) x = dpp_add<0x140>(x);   // a row of sixteen, mirrored
  if (P >= 32) x += __shfl_xor(x, 16, ZA_WAVE);
  if (P >= 64) x += __shfl_xor(x, 32, ZA_WAVE);
  return x;
}

// One wave a workgroup: 64 / P columns of one head's state, P lanes a column, RC_ROWS rows
// a lane.  The vectors of the next CH tokens are requested into registers while the
// current CH tokens are walked out of LDS, and put into the other LDS buffer afterwards.
// LONG: portions of many tokens (chunks of up to sixteen tokens, so that a chunk's walk
// outlasts the trip to memory of the next one's vectors); otherwise chunks as short as the
// load pattern allows, which leaves LDS for more waves when every portion is a token or two.
// (LONG == 1: half as long chunks, for steps with more waves than the chip has SIMDs, where
// LDS decides how many of them run at once)
template <int P, int FORM, int LONG>
__global__ void __launch_bounds__(64, 2)
matrix_recurrence_kernel(RecurrenceArgs a) {
  constexpr bool DELTA = FORM == RC_DELTA, CHANNEL = FORM == RC_CHANNEL;
  constexpr int R = RC_ROWS;
  constexpr int DKMAX = R * P;
  constexpr int CH_MIN = 4 * P < 64 ? 64 / (4 * P) : 1;
  constexpr int CH_LONG = (P <= 8 ? 16 : (P == 16 ? 8 : (P == 32 ? 4 : 2))) / (LONG == 1 ? 2 : 1);
  constexpr int CH = LONG ? (CH_LONG < CH_MIN ? CH_MIN : CH_LONG) : (CH_MIN < 2 ? 2 : CH_MIN);
  constexpr int NV = DELTA || CHANNEL ? 3 : 2;      // vectors of dk floats a token
  constexpr int KPAD = RC_SHARE * P;
  // a chunk's vectors come four floats a lane and load: LPV lanes cover a vector (or a
  // quarter of a long one), so one load instruction of the wave brings TPL tokens' worth
  constexpr int LPV = 4 * P < 64 ? 4 * P : 64;
  constexpr int TPL = 64 / LPV;
  constexpr int PIECES = DKMAX > 256 ? DKMAX / 256 : 1;
  constexpr int NLOAD = NV * (CH / TPL) * PIECES;    // four-float loads a lane and chunk
  __shared__ __attribute__((aligned(16))) float vecs[2][CH][NV][KPAD];
  __shared__ float scal[2][CH][2];                   // SSD: (decay, dt); delta: (beta, -)

  const int s = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int dk = a.dk, dv = a.dv;
  const int g = h / (a.H / a.G);
  const int col = blockIdx.z * (64 / P) + lane / P, part = lane % P;
  const bool owner = col < dv;
  const int start = a.seq_start[s];
  const int n = a.seq_count ? a.seq_count[s] : a.seq_start[s + 1] - start;

  // where the token's vectors lie: vector v of token t starts at base[v] + t * stride
  const float* base[NV];
  int stride;
  if (DELTA) {
    stride = a.prep_width;
    base[0] = a.prep + a.G * dk + g * dk;            // k
    base[1] = a.prep + g * dk;                       // q
    base[NV - 1] = a.prep + 2 * a.G * dk + h * dk;   // decays
  } else {
    stride = a.conv_width;
    base[0] = a.conv + a.k_col + g * dk;
    base[1] = a.conv + a.q_col + g * dk;
    if (CHANNEL) base[NV - 1] = a.conv + a.decay_col + h * dk;   // decays
  }
  const float* xsrc = a.conv + a.x_col + h * dv + (owner ? col : 0);

  float* st = a.state + (size_t)a.slot_id[s] * a.slot_stride + ((size_t)h * dv + col) * dk + part * R;
  const bool vec_state = (dk % 4 == 0) && (a.slot_stride % 4 == 0) &&
                         ((reinterpret_cast<uintptr_t>(a.state) & 15) == 0);
  float S[R];
#pragma unroll
  for (int r = 0; r < R; ++r) S[r] = 0.f;
  if (owner) {
    if (vec_state) {
#pragma unroll
      for (int r = 0; r < R; r += 4)
        if (part * R + r < dk) {
          const float4 v = *reinterpret_cast<const float4*>(st + r);
          S[r] = v.x; S[r + 1] = v.y; S[r + 2] = v.z; S[r + 3] = v.w;
        }
    } else {
#pragma unroll
      for (int r = 0; r < R; ++r)
        if (part * R + r < dk) S[r] = st[r];
    }
  }
  const bool fixed = FORM == RC_SSD && a.fixed_decay != nullptr;
  const float fixed_a = fixed ? a.fixed_decay[h] : 0.f;
  const float neg_A = (FORM != RC_SSD || fixed) ? 0.f : -expf(a.A_log[h]);
  const float Dh = (FORM != RC_SSD || !a.D) ? 0.f : a.D[h];
  const float dtb = (FORM != RC_SSD || fixed) ? 0.f : a.dt_bias[h];

  // (whole four-float loads need the vectors to start on 16-byte boundaries)
  bool vec_loads = dk % 4 == 0 && stride % 4 == 0;
#pragma unroll
  for (int v = 0; v < NV; ++v)
    vec_loads = vec_loads && (reinterpret_cast<uintptr_t>(base[v]) & 15) == 0;
  const int lane_tt = lane / LPV, lane_i = (lane % LPV) * 4;
  float4 regs[NLOAD];
  float xnext[CH], snext = 0.f;
  int chunk_left = 0;       // tokens of the portion from the requested chunk's start on
  auto request = [&](int c0) {
#pragma unroll
    for (int j = 0; j < NLOAD; ++j) {
      const int v = j % NV, piece = (j / NV) % PIECES, group = j / (NV * PIECES);
      const int tt = group * TPL + lane_tt, i = piece * 256 + lane_i;
      // (a chunk's places beyond the portion's end hold tokens that change nothing: no
      // decay, nothing written, nothing read; the walk then needs no conditions)
      const float idle = (NV == 3 && v == NV - 1 && c0 + tt >= n) ? 1.f : 0.f;
      float4 x = make_float4(idle, idle, idle, idle);
      if (c0 + tt < n && i < dk) {
        const float* src = base[v] + (size_t)(start + c0 + tt) * stride + i;
        if (vec_loads) {
          x = *reinterpret_cast<const float4*>(src);
        } else {
          x.x = src[0];
          if (i + 1 < dk) x.y = src[1];
          if (i + 2 < dk) x.z = src[2];
          if (i + 3 < dk) x.w = src[3];
        }
      }
      regs[j] = x;
    }
#pragma unroll
    for (int tt = 0; tt < CH; ++tt)
      xnext[tt] = c0 + tt < n ? xsrc[(size_t)(start + c0 + tt) * a.conv_width] : 0.f;
    snext = 0.f;
    chunk_left = n - c0;
    if (lane < CH && c0 + lane < n) {
      const size_t t = start + c0 + lane;
      if (DELTA) {
        snext = a.prep[t * a.prep_width + 2 * a.G * dk + a.H * dk + h];
      } else if (FORM == RC_SSD && !fixed) {
        const size_t at = t * a.proj_stride + a.gate_col + h;
        snext = a.proj_bf16 ? (float)((const bf16_t*)a.proj)[at] : ((const float*)a.proj)[at];
      }
    }
  };
  auto deposit = [&](int buf) {
#pragma unroll
    for (int j = 0; j < NLOAD; ++j) {
      const int v = j % NV, piece = (j / NV) % PIECES, group = j / (NV * PIECES);
      // (four channels from a multiple of four lie in one lane's share: side by side)
      *reinterpret_cast<float4*>(&vecs[buf][group * TPL + lane_tt][v][lds_at(piece * 256 + lane_i)]) =
          regs[j];
    }
    if (lane < CH) {
      if (DELTA) {
        scal[buf][lane][0] = snext;
      } else if (FORM == RC_SSD) {
        const float dt = fixed ? 1.f : softplus_f(snext + dtb);
        scal[buf][lane][0] = lane < chunk_left ? (fixed ? fixed_a : expf(neg_A * dt)) : 1.f;
        scal[buf][lane][1] = lane < chunk_left ? dt : 0.f;
      }
    }
  };

  float xcur[CH];
  request(0);
  deposit(0);
#pragma unroll
  for (int tt = 0; tt < CH; ++tt) xcur[tt] = xnext[tt];
  __syncthreads();
  for (int c0 = 0, buf = 0; c0 < n; c0 += CH, buf ^= 1) {
    const bool more = c0 + CH < n;
    if (more) request(c0 + CH);
    const int cn = n - c0 < CH ? n - c0 : CH;
    float result[CH];      // stored after the walk: a store among the requests would make
                           // the walk wait for everything requested before it
#pragma unroll
    for (int tt = 0; tt < CH; ++tt) {
      {
        float kk[R], qq[R];
#pragma unroll
        for (int r = 0; r < R; r += 4) {
          const float4 k4 = *reinterpret_cast<const float4*>(&vecs[buf][tt][0][part * RC_SHARE + r]);
          const float4 q4 = *reinterpret_cast<const float4*>(&vecs[buf][tt][1][part * RC_SHARE + r]);
          kk[r] = k4.x; kk[r + 1] = k4.y; kk[r + 2] = k4.z; kk[r + 3] = k4.w;
          qq[r] = q4.x; qq[r + 1] = q4.y; qq[r + 2] = q4.z; qq[r + 3] = q4.w;
        }
        const float xv = xcur[tt];
        float o;
        if (DELTA) {
          float gg[R];
#pragma unroll
          for (int r = 0; r < R; r += 4) {
            const float4 g4 =
                *reinterpret_cast<const float4*>(&vecs[buf][tt][NV - 1][part * RC_SHARE + r]);
            gg[r] = g4.x; gg[r + 1] = g4.y; gg[r + 2] = g4.z; gg[r + 3] = g4.w;
          }
          float d0 = 0.f, d1 = 0.f, d2 = 0.f, d3 = 0.f;
#pragma unroll
          for (int r = 0; r < R; r += 4) {
            S[r] *= gg[r]; S[r + 1] *= gg[r + 1]; S[r + 2] *= gg[r + 2]; S[r + 3] *= gg[r + 3];
            d0 = fmaf(S[r], kk[r], d0);
            d1 = fmaf(S[r + 1], kk[r + 1], d1);
            d2 = fmaf(S[r + 2], kk[r + 2], d2);
            d3 = fmaf(S[r + 3], kk[r + 3], d3);
          }
          const float dot = group_sum<P>((d0 + d1) + (d2 + d3));
          const float u = scal[buf][tt][0] * (xv - dot);
          float a0 = 0.f, a1 = 0.f, a2 = 0.f, a3 = 0.f;
#pragma unroll
          for (int r = 0; r < R; r += 4) {
            S[r] = fmaf(kk[r], u, S[r]);
            S[r + 1] = fmaf(kk[r + 1], u, S[r + 1]);
            S[r + 2] = fmaf(kk[r + 2], u, S[r + 2]);
            S[r + 3] = fmaf(kk[r + 3], u, S[r + 3]);
            a0 = fmaf(S[r], qq[r], a0);
            a1 = fmaf(S[r + 1], qq[r + 1], a1);
            a2 = fmaf(S[r + 2], qq[r + 2], a2);
            a3 = fmaf(S[r + 3], qq[r + 3], a3);
          }
          o = group_sum<P>((a0 + a1) + (a2 + a3));
        } else if (CHANNEL) {
          float a0 = 0.f, a1 = 0.f, a2 = 0.f, a3 = 0.f;
#pragma unroll
          for (int r = 0; r < R; r += 4) {
            const float4 g4 =
                *reinterpret_cast<const float4*>(&vecs[buf][tt][NV - 1][part * RC_SHARE + r]);
            S[r] = fmaf(g4.x, S[r], xv * kk[r]);
            S[r + 1] = fmaf(g4.y, S[r + 1], xv * kk[r + 1]);
            S[r + 2] = fmaf(g4.z, S[r + 2], xv * kk[r + 2]);
            S[r + 3] = fmaf(g4.w, S[r + 3], xv * kk[r + 3]);
            a0 = fmaf(S[r], qq[r], a0);
            a1 = fmaf(S[r + 1], qq[r + 1], a1);
            a2 = fmaf(S[r + 2], qq[r + 2], a2);
            a3 = fmaf(S[r + 3], qq[r + 3], a3);
          }
          o = group_sum<P>((a0 + a1) + (a2 + a3));
        } else {
          const float decay_t = scal[buf][tt][0], dtx = scal[buf][tt][1] * xv;
          float a0 = 0.f, a1 = 0.f, a2 = 0.f, a3 = 0.f;
#pragma unroll
          for (int r = 0; r < R; r += 4) {
            S[r] = fmaf(decay_t, S[r], dtx * kk[r]);
            S[r + 1] = fmaf(decay_t, S[r + 1], dtx * kk[r + 1]);
            S[r + 2] = fmaf(decay_t, S[r + 2], dtx * kk[r + 2]);
            S[r + 3] = fmaf(decay_t, S[r + 3], dtx * kk[r + 3]);
            a0 = fmaf(S[r], qq[r], a0);
            a1 = fmaf(S[r + 1], qq[r + 1], a1);
            a2 = fmaf(S[r + 2], qq[r + 2], a2);
            a3 = fmaf(S[r + 3], qq[r + 3], a3);
          }
          o = fmaf(Dh, xv, group_sum<P>((a0 + a1) + (a2 + a3)));
        }
        result[tt] = o;
      }
    }
    if (part == 0 && owner) {
#pragma unroll
      for (int tt = 0; tt < CH; ++tt)
        if (tt < cn) a.out[(size_t)(start + c0 + tt) * a.H * dv + h * dv + col] = result[tt];
    }
    if (more) {
      deposit(buf ^ 1);
#pragma unroll
      for (int tt = 0; tt < CH; ++tt) xcur[tt] = xnext[tt];
    }
    __syncthreads();
  }
  if (owner) {
    if (vec_state) {
#pragma unroll
      for (int r = 0; r < R; r += 4)
        if (part * R + r < dk)
          *reinterpret_cast<float4*>(st + r) = make_float4(S[r], S[r + 1], S[r + 2], S[r + 3]);
    } else {
#pragma unroll
      for (int r = 0; r < R; ++r)
        if (part * R + r < dk) st[r] = S[r];
    }
  }
}

template <int FORM>
static int launch_recurrence(const RecurrenceArgs& a, int n_seqs, int P, bool long_portions,
                             hipStream_t stream) {
  dim3 grid(n_seqs, a.H, (a.dv * P + 63) / 64), block(64);
  // more waves than SIMDs (256 compute units of four): shorter chunks, more waves at once
  const bool crowded = (long long)grid.x * grid.y * grid.z > 1024;
#define ZA_RECURRENCE(PP)                                                                      \
  case PP:                                                                                     \
    if (long_portions && crowded)                                                              \
      hipLaunchKernelGGL((matrix_recurrence_kernel<PP, FORM, 1>), grid, block, 0, stream, a); \
    else if (long_portions)                                                                    \
      hipLaunchKernelGGL((matrix_recurrence_kernel<PP, FORM, 2>), grid, block, 0, stream, a); \
    else                                                                                       \
      hipLaunchKernelGGL((matrix_recurrence_kernel<PP, FORM, 0>), grid, block, 0, stream, a); \
    break
  switch (P) {
    ZA_RECURRENCE(1);
    ZA_RECURRENCE(2);
    ZA_RECURRENCE(4);
    ZA_RECURRENCE(8);
    ZA_RECURRENCE(16);
    ZA_RECURRENCE(32);
    ZA_RECURRENCE(64);
    default: return ZA_ERR_UNSUPPORTED;
  }
#undef ZA_RECURRENCE
  return za_launch_status();
}

// `form`: 0 = SSD, 1 = gated delta rule, 2 = fixed decay (`decay` then holds H 32-bit
// decays, one per head; proj, dt_bias, A_log and D are not read).  `lanes` (P): the power of two, at most 64, with
// 16 * P >= dk that splits a column's rows.  `prep` (delta): [n_tokens][prep_width]
// floats of scratch, prep_width >= 2*G*dk + H*dk + H.
extern "C" int za_matrix_recurrence(int form, int dtype, const float* conv, int conv_width,
                                    int q_col, int k_col, int x_col, const void* proj,
                                    int proj_stride, int gate_col, const void* decay,
                                    int decay_stride, const float* dt_bias, const float* A_log,
                                    const float* D, float* prep, int prep_width, float* state,
                                    long long slot_stride, const int* seq_start,
                                    const int* slot_id, float* out, int n_tokens, int n_seqs,
                                    int H, int G, int dk, int dv, int lanes,
                                    hipStream_t stream) {
  if (n_seqs == 0 || n_tokens == 0) return 0;
  if (form < 0 || form > 2) return ZA_ERR_ARG;
  if (n_seqs < 0 || n_tokens < 0 || H <= 0 || G <= 0 || H % G || dk <= 0 || dv <= 0 || !conv ||
      !state || !seq_start || !slot_id || !out)
    return ZA_ERR_ARG;
  if (form != 2 && (!proj || !dt_bias || !A_log)) return ZA_ERR_ARG;
  if (form == 2 && !decay) return ZA_ERR_ARG;
  if (form == 0 && !D) return ZA_ERR_ARG;
  if (form == 1 && (!decay || decay_stride < H * dk || !prep ||
                    prep_width < 2 * G * dk + H * dk + H))
    return ZA_ERR_ARG;
  if (lanes < 1 || lanes > 64 || (lanes & (lanes - 1)) || lanes * RC_ROWS < dk ||
      slot_stride < (long long)H * dk * dv)
    return ZA_ERR_ARG;
  if (dtype != 0 && dtype != 1) return ZA_ERR_UNSUPPORTED;
  RecurrenceArgs a{conv, conv_width, q_col, k_col, x_col, proj, proj_stride, gate_col, dtype,
                   prep, prep_width, dt_bias, A_log, form == 2 ? nullptr : D, state, slot_stride,
                   seq_start, slot_id, out, H, G, dk, dv,
                   form == 2 ? (const float*)decay : nullptr, nullptr, 0};
  // (a function of the step's shape alone, as a recorded step needs it)
  const bool long_portions = n_tokens > 4 * n_seqs;
  if (form != 1) return launch_recurrence<RC_SSD>(a, n_seqs, lanes, long_portions, stream);
  const dim3 prep_grid(n_tokens, 2 * G + (H * dk + 255) / 256);
  if (dtype == 0)
    hipLaunchKernelGGL((delta_prepare_kernel<float>), prep_grid, dim3(64), 0, stream, conv,
                       conv_width, q_col, k_col, (const float*)proj, proj_stride, gate_col,
                       (const float*)decay, decay_stride, dt_bias, A_log, prep, prep_width, H, G,
                       dk);
  else
    hipLaunchKernelGGL((delta_prepare_kernel<bf16_t>), prep_grid, dim3(64), 0, stream, conv,
                       conv_width, q_col, k_col, (const bf16_t*)proj, proj_stride, gate_col,
                       (const bf16_t*)decay, decay_stride, dt_bias, A_log, prep, prep_width, H, G,
                       dk);
  const int rc = za_launch_status();
  if (rc != 0) return rc;
  return launch_recurrence<RC_DELTA>(a, n_seqs, lanes, long_portions, stream);
}

// ------------------------------------------------- fixed decay, long portions in chunks
// With a constant decay a head the state is linear in what the tokens bring, so a long
// portion need not be walked in one chain.  It is cut into chunks (the step's work items
// of CHUNK consecutive rows of one request):
//   1. every chunk is walked by itself from an empty state (matrix_recurrence_kernel with
//      one walker a chunk), leaving o_local[t] and its own final state L_c;
//   2. chunk_state_prefix: per request, in the order of its chunks, the state BEFORE chunk c,
//      B_c = B_(c-1) d^n(c-1) + L_(c-1), B_0 the request's carried state; the last one goes
//      back to the request's slot.  One thread a state element.
//   3. chunk_correct: o[t] = o_local[t] + d^(j+1) B_c^T q_t for token j of chunk c.
// All in 32-bit; powers of the decay as exp2(n log2 d).  A prompt of 2,048 tokens becomes
// eight chains of 256 tokens side by side instead of one of 2,048.
__global__ void __launch_bounds__(256)
chunk_state_prefix_kernel(float* __restrict__ chunk_state, float* __restrict__ state,
                          long long slot_stride, const int* __restrict__ slot_id,
                          const int* __restrict__ item_seq, const int* __restrict__ item_count,
                          int n_items, const float* __restrict__ decay, int elems, int per_head) {
  const int s = blockIdx.x;
  const int e = blockIdx.y * 256 + threadIdx.x;
  if (e >= elems) return;
  const float l2 = log2f(decay[e / per_head]);
  float* slot = state + (size_t)slot_id[s] * slot_stride + e;
  float S = *slot;
  for (int i = 0; i < n_items; ++i) {
    if (item_seq[i] != s) continue;
    float* at = chunk_state + (size_t)i * elems + e;
    const float local = *at;
    *at = S;
    const float a = decay[e / per_head] == 0.f ? 0.f : exp2f((float)item_count[i] * l2);
    S = fmaf(a, S, local);
  }
  *slot = S;
}

#define CC_TOKENS 16    // tokens whose queries are staged at a time
template <int DKR>      // rows of a state column kept in registers: dk <= DKR
__global__ void __launch_bounds__(128)
chunk_correct_kernel(const float* __restrict__ vectors, int width, int q_col,
                     const float* __restrict__ chunk_state, const int* __restrict__ item_row0,
                     const int* __restrict__ item_count, const float* __restrict__ decay,
                     float* __restrict__ out, int H, int dk, int dv, int tokens_per_block) {
  __shared__ float qs[CC_TOKENS][DKR];
  const int item = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int row0 = item_row0[item], cnt = item_count[item];
  const int t_begin = blockIdx.z * tokens_per_block;
  int t_end = t_begin + tokens_per_block;
  if (t_end > cnt) t_end = cnt;
  if (t_begin >= cnt) return;
  const float d = decay[h];
  const float l2 = log2f(d);
  const size_t elems = (size_t)H * dv * dk;
  for (int c0 = 0; c0 < dv; c0 += 128) {
    const int col = c0 + tid;
    float S[DKR];
#pragma unroll
    for (int r = 0; r < DKR; ++r) S[r] = 0.f;
    if (col < dv) {
      const float* src = chunk_state + (size_t)item * elems + ((size_t)h * dv + col) * dk;
#pragma unroll
      for (int r = 0; r < DKR; ++r)
        if (r < dk) S[r] = src[r];
    }
    for (int tb = t_begin; tb < t_end; tb += CC_TOKENS) {
      __syncthreads();
      // (rows beyond dk and tokens beyond the block's end are zeros: every product below
      // runs over all DKR rows)
      for (int idx = tid; idx < CC_TOKENS * DKR; idx += 128) {
        const int tt = idx / DKR, r = idx % DKR;
        qs[tt][r] = (r < dk && tb + tt < t_end)
                        ? vectors[(size_t)(row0 + tb + tt) * width + q_col + h * dk + r] : 0.f;
      }
      __syncthreads();
      if (col < dv) {
        // what the tokens' read-outs hold is requested for all of them before the first
        // product, and four sums run side by side in each
        float* o = out + (size_t)(row0 + tb) * H * dv + h * dv + col;
        float old[CC_TOKENS];
#pragma unroll
        for (int tt = 0; tt < CC_TOKENS; ++tt)
          old[tt] = tb + tt < t_end ? o[(size_t)tt * H * dv] : 0.f;
#pragma unroll
        for (int tt = 0; tt < CC_TOKENS; ++tt) {
          float d0 = 0.f, d1 = 0.f, d2 = 0.f, d3 = 0.f;
#pragma unroll
          for (int r = 0; r < DKR; r += 4) {
            d0 = fmaf(S[r], qs[tt][r], d0);
            d1 = fmaf(S[r + 1], qs[tt][r + 1], d1);
            d2 = fmaf(S[r + 2], qs[tt][r + 2], d2);
            d3 = fmaf(S[r + 3], qs[tt][r + 3], d3);
          }
          const float w = d == 0.f ? 0.f : exp2f((float)(tb + tt + 1) * l2);
          if (tb + tt < t_end) o[(size_t)tt * H * dv] = fmaf(w, (d0 + d1) + (d2 + d3), old[tt]);
        }
      }
    }
  }
}

// `vectors` as retention_prepare leaves them; `item_*`: the step's work items of at most
// `chunk` rows (n_items of them; with n_items == n_seqs the plain walk does the same); `iota`:
// 0 .. n_items - 1; `chunk_state`: n_items * H*dv*dk floats, zero on entry.
extern "C" int za_retention_chunked(const float* vectors, int width, int q_col, int k_col,
                                    int x_col, const float* decay, float* state,
                                    long long slot_stride, const int* slot_id,
                                    const int* item_seq, const int* item_row0,
                                    const int* item_count, const int* iota, int n_items,
                                    int n_seqs, int chunk, float* chunk_state, float* out,
                                    int n_tokens, int H, int dk, int dv, int lanes,
                                    hipStream_t stream) {
  if (n_tokens == 0 || n_items == 0) return 0;
  if (n_tokens < 0 || n_items < n_seqs || n_seqs <= 0 || chunk <= 0 || H <= 0 || dk <= 0 || dv <= 0 ||
      !vectors || !decay || !state || !slot_id || !item_seq || !item_row0 || !item_count ||
      !iota || !chunk_state || !out)
    return ZA_ERR_ARG;
  if (dk > 128) return ZA_ERR_UNSUPPORTED;
  if (lanes < 1 || lanes > 64 || (lanes & (lanes - 1)) || lanes * RC_ROWS < dk ||
      slot_stride < (long long)H * dk * dv)
    return ZA_ERR_ARG;
  const long long elems = (long long)H * dk * dv;
  RecurrenceArgs a{vectors, width, q_col, k_col, x_col, nullptr, 0, 0, 0, nullptr, 0, nullptr,
                   nullptr, nullptr, chunk_state, elems, item_row0, iota, out, H, H, dk, dv,
                   decay, item_count, 0};
  int rc = launch_recurrence<RC_SSD>(a, n_items, lanes, n_tokens > 4 * n_items, stream);
  if (rc != 0) return rc;
  hipLaunchKernelGGL(chunk_state_prefix_kernel, dim3(n_seqs, (unsigned)((elems + 255) / 256)),
                     dim3(256), 0, stream, chunk_state, state, slot_stride, slot_id, item_seq,
                     item_count, n_items, decay, (int)elems, dk * dv);
  rc = za_launch_status();
  if (rc != 0) return rc;
  const int tokens_per_block = 64;      // an item has at most `chunk` rows
  dim3 grid(n_items, H, (unsigned)((chunk + tokens_per_block - 1) / tokens_per_block));
  if (dk <= 64)
    hipLaunchKernelGGL((chunk_correct_kernel<64>), grid, dim3(128), 0, stream, vectors, width,
                       q_col, chunk_state, item_row0, item_count, decay, out, H, dk, dv,
                       tokens_per_block);
  else
    hipLaunchKernelGGL((chunk_correct_kernel<128>), grid, dim3(128), 0, stream, vectors, width,
                       q_col, chunk_state, item_row0, item_count, decay, out, H, dk, dv,
                       tokens_per_block);
  return za_launch_status();
}

// ------------------------------------------------------ a decay a head and key channel
// What the channel-decay walk reads, from the opening projection's rows, per token as 32-bit
// floats
//   out[t] = [q * q_scale: H*dk | k: H*dk | a: H*dk | v: H*dv]  (padded to `out_width`)
// with the decays a = sigmoid(z)^(1/root), z = up low[t] + bias: `low` the token's `rank` columns
// of the projection, `up` [H*dk][rank] a second, small product taken here in 32-bit.  The power
// is taken through the logarithm, log sigmoid(z) = -softplus(-z).
// grid (tokens / GP_TOKENS, channels / workgroup size).
#define GP_TOKENS 8
#define GP_RANK 256     // columns of `low` staged at a time
template <typename T, typename TW>
__global__ void __launch_bounds__(256)
channel_decay_prepare_kernel(const T* __restrict__ proj, int proj_stride, int q_col, int k_col,
                             int v_col, int low_col, int rank, const TW* __restrict__ up,
                             const float* __restrict__ bias, float inv_root, float q_scale,
                             float* __restrict__ out, int out_width, int n_tokens, int hk, int hv) {
  __shared__ float low[GP_TOKENS][GP_RANK];
  const int bd = blockDim.x;
  const int t0 = blockIdx.x * GP_TOKENS, c = blockIdx.y * bd + threadIdx.x;
  const int nt = n_tokens - t0 < GP_TOKENS ? n_tokens - t0 : GP_TOKENS;
  // (what is only converted is requested first; tokens beyond the last repeat it)
  float z[GP_TOKENS], q[GP_TOKENS], k[GP_TOKENS], v[GP_TOKENS];
#pragma unroll
  for (int i = 0; i < GP_TOKENS; ++i) {
    const T* row = proj + (size_t)(t0 + (i < nt ? i : nt - 1)) * proj_stride;
    z[i] = 0.f;
    q[i] = to_f32<T>(row[q_col + (c < hk ? c : 0)]);
    k[i] = to_f32<T>(row[k_col + (c < hk ? c : 0)]);
    v[i] = to_f32<T>(row[v_col + (c < hv ? c : 0)]);
  }
  for (int r0 = 0; r0 < rank; r0 += GP_RANK) {
    const int rn = rank - r0 < GP_RANK ? rank - r0 : GP_RANK;
    __syncthreads();
    for (int idx = threadIdx.x; idx < GP_TOKENS * rn; idx += bd) {
      const int i = idx / rn, r = idx % rn;
      low[i][r] = i < nt ? to_f32<T>(proj[(size_t)(t0 + i) * proj_stride + low_col + r0 + r]) : 0.f;
    }
    __syncthreads();
    if (c < hk) {
      const TW* w = up + (size_t)c * rank + r0;
      int r = 0;
      if (rank % 8 == 0) {       // (rows of `up` start on 16-byte boundaries)
#pragma unroll 2
        for (; r + 8 <= rn; r += 8) {
          float w8[8];
          load8<TW>(w + r, w8);
#pragma unroll
          for (int e = 0; e < 8; ++e)
#pragma unroll
            for (int i = 0; i < GP_TOKENS; ++i) z[i] = fmaf(w8[e], low[i][r + e], z[i]);
        }
      }
      for (; r < rn; ++r) {
        const float wv = to_f32<TW>(w[r]);
#pragma unroll
        for (int i = 0; i < GP_TOKENS; ++i) z[i] = fmaf(wv, low[i][r], z[i]);
      }
    }
  }
  const float b = c < hk ? bias[c] : 0.f;
#pragma unroll
  for (int i = 0; i < GP_TOKENS; ++i) {
    if (i >= nt) continue;
    float* dst = out + (size_t)(t0 + i) * out_width;
    if (c < hk) {
      dst[c] = q[i] * q_scale;
      dst[hk + c] = k[i];
      dst[2 * hk + c] = expf(-softplus_f(-(z[i] + b)) * inv_root);
    }
    if (c < hv) dst[3 * hk + c] = v[i];
  }
}

extern "C" int za_channel_decay_prepare(const void* proj, int dtype, int proj_stride, int q_col,
                                        int k_col, int v_col, int low_col, int rank,
                                        const void* up, int up_dtype, const float* bias, float root,
                                        float q_scale, float* out, int out_width, int n_tokens,
                                        int H, int dk, int dv, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  if (n_tokens < 0 || H <= 0 || dk <= 0 || dv <= 0 || rank <= 0 || !(root > 0.f) || !proj || !up ||
      !bias || !out || q_col < 0 || k_col < 0 || v_col < 0 || low_col < 0 ||
      q_col + H * dk > proj_stride || k_col + H * dk > proj_stride ||
      v_col + H * dv > proj_stride || low_col + rank > proj_stride ||
      out_width < 3 * H * dk + H * dv)
    return ZA_ERR_ARG;
  const int hk = H * dk, hv = H * dv, most = hk > hv ? hk : hv;
  const int bd = n_tokens <= 64 ? 64 : 256;      // a decode batch: more, smaller workgroups
  dim3 grid((n_tokens + GP_TOKENS - 1) / GP_TOKENS, (most + bd - 1) / bd), block(bd);
#define ZA_CDP(T, TW)                                                                          \
  hipLaunchKernelGGL((channel_decay_prepare_kernel<T, TW>), grid, block, 0, stream,            \
                     (const T*)proj, proj_stride, q_col, k_col, v_col, low_col, rank,          \
                     (const TW*)up, bias, 1.0f / root, q_scale, out, out_width, n_tokens, hk, hv)
  if (dtype == 0 && up_dtype == 0) ZA_CDP(float, float);
  else if (dtype == 1 && up_dtype == 1) ZA_CDP(bf16_t, bf16_t);
  else if (dtype == 1 && up_dtype == 0) ZA_CDP(bf16_t, float);
  else return ZA_ERR_UNSUPPORTED;
#undef ZA_CDP
  return za_launch_status();
}

// Portions of many tokens: blocks of up to CM_TOKENS tokens at a time, as matrix products on the
// matrix cores in their 32-bit form (v_mfma_f32_16x16x4_f32: products and sums in full
// 32-bit).  Within a block that starts from state S, with a_1 its first token's decays and
// L_i = a_2 ... a_i (per channel, L_1 = 1; S' = diag(a_1) S):
//     o_i = S'^T (q_i L_i) + sum_(j <= i) ((q_i L_i) . (k_j / L_j)) v_j
//     S  <- diag(L_n) (S' + sum_j (k_j / L_j) v_j^T)
// A block ends before a token that would take any channel's L below CM_FLOOR, so that k / L stays
// finite and every sum keeps the precision of its largest term; the token then opens the next
// block, where its own decays only multiply the state: decays may be as small as they like,
// zero included, and only make blocks shorter.
// A workgroup serves 64 columns of one walker's head, 16 a wave: a wave keeps its columns'
// state in accumulators, whose layout (rows 4 g + i of a tile in register i of lane group g)
// is that of the second operand when k runs as 4 g + j, so S enters q S and leaves K^T V
// without moving.  What a token brings is requested one block ahead.
#define CM_TOKENS 16
#define CM_FLOOR 7.8886090522101181e-31f     // 2^-100
#define CM_LD (CM_TOKENS + 4)                // padded row of 16 tokens, 16-byte aligned

struct ChannelArgs {
  const float* vectors;    // [T][width]: q | k | decays | v
  int width;
  float* state;            // per slot [H][dv][dk]
  long long slot_stride;
  const int* start;        // first row of walker w
  const int* count;        // its rows, or null: start[w + 1] - start[w]
  const int* slot_id;      // null: walker w uses slot w, and starts from an empty state
  float* out;              // [T][H*dv]
  float* scaled_q;         // null, or [T][H*dk]: q times all decays since the walker's start
  float* total;            // null, or [walkers][H*dk]: the product of all its decays
  int H, dk, dv;
};

template <int NT>     // tiles of 16 key channels
__global__ void __launch_bounds__(256)
channel_blocks_kernel(ChannelArgs a) {
  constexpr int DK = NT * 16, QLD = DK + 4;
  constexpr int UNITS = 2 * DK;                       // (q or k) x channel
  constexpr int U = UNITS <= 256 ? 1 : UNITS / 256;   // units a thread
  __shared__ __attribute__((aligned(16))) float qs[CM_TOKENS][QLD];     // q L
  __shared__ __attribute__((aligned(16))) float ks[CM_TOKENS][QLD];     // k / L
  __shared__ __attribute__((aligned(16))) float kt[DK][CM_LD];          // the same, turned round
  __shared__ __attribute__((aligned(16))) float part[4][16][CM_LD];     // q L . k / L, by range of k
  __shared__ __attribute__((aligned(16))) float grow[DK];               // the state's next factor
  __shared__ int shortest;

  const int w = blockIdx.x, h = blockIdx.y;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int r16 = lane & 15, g = lane >> 4;
  const int dk = a.dk, dv = a.dv, hk = a.H * dk;
  const int row0 = a.start[w], n_rows = a.count ? a.count[w] : a.start[w + 1] - row0;
  const int col = blockIdx.z * 64 + wave * 16 + r16;
  const bool col_ok = col < dv;
  const float* rows = a.vectors + (size_t)row0 * a.width;
  const float* vcol = rows + 3 * hk + h * dv + (col_ok ? col : 0);
  float* st = a.state + (size_t)(a.slot_id ? a.slot_id[w] : w) * a.slot_stride +
              ((size_t)h * dv + (col_ok ? col : 0)) * dk;
  const bool aligned = dk % 4 == 0 && a.slot_stride % 4 == 0 &&
                       (reinterpret_cast<uintptr_t>(a.state) & 15) == 0;

  f32x4_t S[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    S[t] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int c = t * 16 + 4 * g;
    if (!a.slot_id || !col_ok) continue;
    if (aligned) {
      if (c < dk) S[t] = *reinterpret_cast<const f32x4_t*>(st + c);
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (c + i < dk) S[t][i] = st[c + i];
    }
  }

  // this thread's units: channel uc[u], q (first DK units) or k
  float dec[U][CM_TOKENS], x[U][CM_TOKENS], v[4];
  float carried[U], since[U];     // L_n of the block before; the product of all decays so far
  int uc[U];
  bool is_q[U], unit[U];
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int id = tid + u * 256;
    unit[u] = id < UNITS;
    is_q[u] = id < DK;
    uc[u] = is_q[u] ? id : id - DK;
    carried[u] = since[u] = 1.f;
  }
  auto request = [&](int t0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const bool in = unit[u] && uc[u] < dk;
      const float* ap = rows + (size_t)t0 * a.width + 2 * hk + h * dk + (in ? uc[u] : 0);
      const float* xp = ap - (is_q[u] ? 2 * hk : hk);
#pragma unroll
      for (int i = 0; i < CM_TOKENS; ++i) {
        const bool ok = in && t0 + i < n_rows;
        dec[u][i] = ok ? ap[(size_t)i * a.width] : 1.f;
        x[u][i] = ok ? xp[(size_t)i * a.width] : 0.f;
      }
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      v[j] = col_ok && t0 + 4 * g + j < n_rows ? vcol[(size_t)(t0 + 4 * g + j) * a.width] : 0.f;
  };

  int n = 0;
  request(0);
  for (int t0 = 0; t0 < n_rows; t0 += n) {
    // ---- L of every token of the block, and where the block ends
    const int left = n_rows - t0;
    bool all = true;
    float L[U][CM_TOKENS];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      float p = 1.f;
#pragma unroll
      for (int i = 0; i < CM_TOKENS; ++i) {
        if (i > 0) p *= dec[u][i];
        L[u][i] = p;
      }
      all = all && p >= CM_FLOOR;
    }
    if (tid == 0) shortest = CM_TOKENS;
    n = left < CM_TOKENS ? left : CM_TOKENS;
    // (also: every wave is done with the block before)
    if (!__syncthreads_and(all)) {
      int fits = CM_TOKENS;
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int i = CM_TOKENS - 1; i > 0; --i)
          if (!(L[u][i] >= CM_FLOOR) && i < fits) fits = i;
      atomicMin(&shortest, fits);
      __syncthreads();
      n = shortest < n ? shortest : n;
    }
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (!unit[u]) continue;
      const int c = uc[u];
      float last = 1.f;
#pragma unroll
      for (int i = 0; i < CM_TOKENS; ++i) {
        const bool in = i < n;
        if (in) last = L[u][i];
        const float y = !in ? 0.f : is_q[u] ? x[u][i] * L[u][i] : x[u][i] / L[u][i];
        if (is_q[u]) {
          qs[i][c] = y;
          if (a.scaled_q && blockIdx.z == 0 && in && c < dk)
            a.scaled_q[(size_t)(row0 + t0 + i) * hk + h * dk + c] =
                x[u][i] * (since[u] * dec[u][0] * L[u][i]);
        } else {
          ks[i][c] = y;
          kt[c][i] = y;
        }
      }
      if (!is_q[u]) grow[c] = carried[u] * dec[u][0];
      carried[u] = last;
      since[u] *= dec[u][0] * last;
    }
    float vb[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) vb[j] = 4 * g + j < n ? v[j] : 0.f;
    __syncthreads();
    if (t0 + n < n_rows) request(t0 + n);

    // ---- the scores of the block's own tokens, each wave over a quarter of the channels
    f32x4_t sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      if ((t & 3) != wave) continue;
      const f32x4_t fq = *reinterpret_cast<const f32x4_t*>(&qs[r16][t * 16 + 4 * g]);
      const f32x4_t fk = *reinterpret_cast<const f32x4_t*>(&ks[r16][t * 16 + 4 * g]);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        sc = __builtin_amdgcn_mfma_f32_16x16x4f32(fq[j], fk[j], sc, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) part[wave][4 * g + i][r16] = sc[i];

    // ---- what the state gives
    f32x4_t o[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const f32x4_t f = *reinterpret_cast<const f32x4_t*>(&grow[t * 16 + 4 * g]);
      S[t] *= f;
      const f32x4_t fq = *reinterpret_cast<const f32x4_t*>(&qs[r16][t * 16 + 4 * g]);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        o[t & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(fq[j], S[t][j], o[t & 1], 0, 0, 0);
    }
    __syncthreads();

    // ---- what the block's own tokens give
    f32x4_t p = *reinterpret_cast<const f32x4_t*>(&part[0][r16][4 * g]);
#pragma unroll
    for (int q = 1; q < 4; ++q)
      if (q < NT) p += *reinterpret_cast<const f32x4_t*>(&part[q][r16][4 * g]);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float pj = 4 * g + j <= r16 ? p[j] : 0.f;
      o[0] = __builtin_amdgcn_mfma_f32_16x16x4f32(pj, vb[j], o[0], 0, 0, 0);
    }
    o[0] += o[1];
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (col_ok && 4 * g + i < n)
        a.out[(size_t)(row0 + t0 + 4 * g + i) * a.H * dv + h * dv + col] = o[0][i];

    // ---- what they leave in the state
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const f32x4_t fk = *reinterpret_cast<const f32x4_t*>(&kt[t * 16 + r16][4 * g]);
#pragma unroll
      for (int j = 0; j < 4; ++j)
        S[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(fk[j], vb[j], S[t], 0, 0, 0);
    }
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < U; ++u) {
    if (!unit[u]) continue;
    if (!is_q[u]) grow[uc[u]] = carried[u];
    else if (a.total && blockIdx.z == 0 && uc[u] < dk)
      a.total[(size_t)w * hk + h * dk + uc[u]] = since[u];
  }
  __syncthreads();
  if (!col_ok) return;
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int c = t * 16 + 4 * g;
    const f32x4_t f = *reinterpret_cast<const f32x4_t*>(&grow[c]);
    S[t] *= f;
    if (aligned) {
      if (c < dk) *reinterpret_cast<f32x4_t*>(st + c) = S[t];
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (c + i < dk) st[c + i] = S[t][i];
    }
  }
}

#define CM_MAX_DK 256
static int launch_channel_blocks(const ChannelArgs& a, int walkers, hipStream_t stream) {
  dim3 grid(walkers, a.H, (a.dv + 63) / 64), block(256);
#define ZA_BLOCKS(NT) hipLaunchKernelGGL((channel_blocks_kernel<NT>), grid, block, 0, stream, a)
  if (a.dk <= 32) ZA_BLOCKS(2);
  else if (a.dk <= 64) ZA_BLOCKS(4);
  else if (a.dk <= 128) ZA_BLOCKS(8);
  else if (a.dk <= CM_MAX_DK) ZA_BLOCKS(16);
  else return ZA_ERR_UNSUPPORTED;
#undef ZA_BLOCKS
  return za_launch_status();
}

// Every request's portion by one walker from its own state (`vectors` as channel_decay_prepare
// leaves them): token by token where portions are a few tokens, in blocks otherwise (a function
// of the step's shape alone, as a recorded step needs it).
extern "C" int za_channel_recurrence(const float* vectors, int width, float* state,
                                     long long slot_stride, const int* seq_start,
                                     const int* slot_id, float* out, int n_tokens, int n_seqs, int H,
                                     int dk, int dv, int lanes, hipStream_t stream) {
  if (n_tokens == 0 || n_seqs == 0) return 0;
  if (n_tokens < 0 || n_seqs < 0 || H <= 0 || dk <= 0 || dv <= 0 || !vectors || !state ||
      !seq_start || !slot_id || !out || width < 3 * H * dk + H * dv || lanes < 1 || lanes > 64 ||
      (lanes & (lanes - 1)) || lanes * RC_ROWS < dk || slot_stride < (long long)H * dk * dv)
    return ZA_ERR_ARG;
  const int hk = H * dk;
  const bool long_portions = n_tokens > 4 * n_seqs;
  if (long_portions && dk <= CM_MAX_DK)
    return launch_channel_blocks(ChannelArgs{vectors, width, state, slot_stride, seq_start, nullptr,
                                             slot_id, out, nullptr, nullptr, H, dk, dv},
                                 n_seqs, stream);
  RecurrenceArgs a{vectors, width, 0, hk, 3 * hk, nullptr, 0, 0, 0, nullptr, 0, nullptr, nullptr,
                   nullptr, state, slot_stride, seq_start, slot_id, out, H, H, dk, dv, nullptr,
                   nullptr, 2 * hk};
  return launch_recurrence<RC_CHANNEL>(a, n_seqs, lanes, long_portions, stream);
}

// Long portions in chunks, as for the fixed decay: every chunk is walked by itself from an
// empty state, and what the state before it adds to its read-outs is linear in that state:
//   1. channel_blocks, one walker a chunk:        o_local[t], the chunk's own final state L_c,
//      with A_t the product of the chunk's decays up to and including token t (at most one, so
//      nothing overflows) the queries q_t * A_t, and A_c = A at the chunk's end
//   2. channel_prefix: the state before chunk c,  B_c = diag(A_(c-1)) B_(c-1) + L_(c-1)
//   3. channel_readout:                           o[t] = o_local[t] + B_c^T (q_t * A_t)

// One thread a state element; the chunks of a request are neighbours in the list.
__global__ void __launch_bounds__(256)
channel_prefix_kernel(float* __restrict__ chunk_state, float* __restrict__ state,
                      long long slot_stride, const int* __restrict__ slot_id,
                      const int* __restrict__ item_seq, int n_items,
                      const float* __restrict__ total, int elems, int hk, int dk, int dv) {
  __shared__ int bounds[2];
  const int s = blockIdx.x, e = blockIdx.y * 256 + threadIdx.x;
  if (threadIdx.x == 0) { bounds[0] = n_items; bounds[1] = 0; }
  __syncthreads();
  for (int i = threadIdx.x; i < n_items; i += 256)
    if (item_seq[i] == s) {
      atomicMin(&bounds[0], i);
      atomicMax(&bounds[1], i + 1);
    }
  __syncthreads();
  if (e >= elems) return;
  const int first = bounds[0], last = bounds[1];
  const int channel = e / (dk * dv) * dk + e % dk;
  float* slot = state + (size_t)slot_id[s] * slot_stride + e;
  float S = *slot;
  for (int i0 = first; i0 < last; i0 += 8) {
    float local[8], a[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const bool in = i0 + j < last;
      local[j] = in ? chunk_state[(size_t)(i0 + j) * elems + e] : 0.f;
      a[j] = in ? total[(size_t)(i0 + j) * hk + channel] : 1.f;
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      if (i0 + j < last) chunk_state[(size_t)(i0 + j) * elems + e] = S;
      S = fmaf(a[j], S, local[j]);
    }
  }
  *slot = S;
}

// Four consecutive floats, those at and beyond `n` as zeros.
__device__ __forceinline__ f32x4_t four_or_fewer(const float* p, int n, bool aligned) {
  f32x4_t v = {0.f, 0.f, 0.f, 0.f};
  if (aligned && n >= 4) return *reinterpret_cast<const f32x4_t*>(p);
#pragma unroll
  for (int j = 0; j < 4; ++j)
    if (j < n) v[j] = p[j];
  return v;
}

// grid (items, heads, tokens / 64 * columns / 64); four waves of 16 tokens x 64 columns.
// Operand layout of v_mfma_f32_16x16x4_f32: lane l supplies row (l % 16), k-slot (l / 16) of
// either operand and receives rows (l / 16) * 4 .. + 3, column (l % 16).  The order in which k
// runs is free as long as both operands agree: slot g of step j is channel 4 g + j of a
// block of 16, so that a lane's four steps are four neighbouring floats.
__global__ void __launch_bounds__(256)
channel_readout_kernel(const float* __restrict__ scaled_q,
                       const float* __restrict__ chunk_state, const int* __restrict__ item_row0,
                       const int* __restrict__ item_count, float* __restrict__ out, int H, int dk,
                       int dv, int column_blocks) {
  const int item = blockIdx.x, h = blockIdx.y;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int r16 = lane & 15, g = lane >> 4;
  const int row0 = item_row0[item], cnt = item_count[item];
  const int t0 = (blockIdx.z / column_blocks) * 64 + wave * 16;
  const int n0 = (blockIdx.z % column_blocks) * 64;
  if (t0 >= cnt) return;
  const bool row_ok = t0 + r16 < cnt;
  const float* q = scaled_q + ((size_t)(row0 + (row_ok ? t0 + r16 : 0)) * H + h) * dk;
  const float* B = chunk_state + ((size_t)item * H + h) * dv * dk;
  const bool aligned = dk % 4 == 0;
  f32x4_t acc[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) acc[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < dk; k0 += 16) {
    const int k = k0 + 4 * g, left = dk - k;
    const f32x4_t fq = row_ok ? four_or_fewer(q + k, left, aligned) : f32x4_t{0.f, 0.f, 0.f, 0.f};
    f32x4_t fb[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + j * 16 + r16;
      fb[j] = n < dv ? four_or_fewer(B + (size_t)n * dk + k, left, aligned)
                     : f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int step = 0; step < 4; ++step)
#pragma unroll
      for (int j = 0; j < 4; ++j)
        acc[j] = __builtin_amdgcn_mfma_f32_16x16x4f32(fq[step], fb[j][step], acc[j], 0, 0, 0);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = t0 + g * 4 + i;
    if (t >= cnt) continue;
    float* o = out + (size_t)(row0 + t) * H * dv + h * dv;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int n = n0 + j * 16 + r16;
      if (n < dv) o[n] += acc[j][i];
    }
  }
}

// `item_*`: the step's work items of at most `chunk` rows; scratch: `chunk_state` n_items *
// H*dv*dk floats, `scaled_q` n_tokens * H*dk, `total` n_items * H*dk.
extern "C" int za_channel_recurrence_chunked(const float* vectors, int width, float* state,
                                             long long slot_stride, const int* slot_id,
                                             const int* item_seq, const int* item_row0,
                                             const int* item_count, int n_items, int n_seqs,
                                             int chunk, float* chunk_state, float* scaled_q,
                                             float* total, float* out, int n_tokens, int H, int dk,
                                             int dv, hipStream_t stream) {
  if (n_tokens == 0 || n_items == 0) return 0;
  if (n_tokens < 0 || n_seqs <= 0 || n_items < n_seqs || chunk <= 0 || H <= 0 || dk <= 0 ||
      dv <= 0 || !vectors || !state || !slot_id || !item_seq || !item_row0 || !item_count ||
      !chunk_state || !scaled_q || !total || !out || width < 3 * H * dk + H * dv ||
      slot_stride < (long long)H * dk * dv)
    return ZA_ERR_ARG;
  const long long elems = (long long)H * dk * dv;
  if (dk > CM_MAX_DK || elems > 0x7fffffffLL) return ZA_ERR_UNSUPPORTED;
  int rc = launch_channel_blocks(ChannelArgs{vectors, width, chunk_state, elems, item_row0,
                                             item_count, nullptr, out, scaled_q, total, H, dk, dv},
                                 n_items, stream);
  if (rc != 0) return rc;
  hipLaunchKernelGGL(channel_prefix_kernel, dim3(n_seqs, (unsigned)((elems + 255) / 256)),
                     dim3(256), 0, stream, chunk_state, state, slot_stride, slot_id, item_seq,
                     n_items, total, (int)elems, H * dk, dk, dv);
  rc = za_launch_status();
  if (rc != 0) return rc;
  const int column_blocks = (dv + 63) / 64;
  hipLaunchKernelGGL(channel_readout_kernel,
                     dim3(n_items, H, (unsigned)((chunk + 63) / 64 * column_blocks)), dim3(256), 0,
                     stream, scaled_q, chunk_state, item_row0, item_count, out, H, dk, dv,
                     column_blocks);
  return za_launch_status();
}

// ------------------------------------------------------------ retention's vectors
// What the fixed-decay walk reads, from the opening projection's rows: per token the
// queries and keys of every head with the first `rot` elements of each rotated by the
// token's position (element i paired with i + rot/2, angle = position * inv_freq[i]) and
// the keys times `k_scale`, then the values, all as 32-bit floats:
//   prep[t] = [q: H*dk | k: H*dk | v: H*dv]
// grid (tokens, heads), one wave.
template <typename T>
__global__ void __launch_bounds__(64)
retention_prepare_kernel(const T* __restrict__ proj, int proj_stride, int q_col, int k_col,
                         int v_col, const int* __restrict__ positions,
                         const float* __restrict__ inv_freq, float* __restrict__ prep, int H,
                         int dk, int dv, int rot, float k_scale, int act) {
  const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const T* row = proj + (size_t)t * proj_stride;
  float* dst = prep + (size_t)t * (2 * H * dk + H * dv);
  const int pos = positions[t], half = rot / 2;
  for (int i = lane; i < dk; i += 64) {
    // (`act` 1: silu on what the projection gave, before anything else)
    float q = to_f32<T>(row[q_col + h * dk + i]);
    float k = to_f32<T>(row[k_col + h * dk + i]);
    if (act) { q = silu_f(q); k = silu_f(k); }
    float qo = q, ko = k;
    if (i < rot) {
      const bool low = i < half;
      const int j = low ? i : i - half, partner = low ? i + half : i - half;
      float cs, sn;
      rope_angle(pos, inv_freq[j], &cs, &sn);
      float qp = to_f32<T>(row[q_col + h * dk + partner]);
      float kp = to_f32<T>(row[k_col + h * dk + partner]);
      if (act) { qp = silu_f(qp); kp = silu_f(kp); }
      qo = low ? rope_rotate_low(q, qp, cs, sn) : rope_rotate_high(q, qp, cs, sn);
      ko = low ? rope_rotate_low(k, kp, cs, sn) : rope_rotate_high(k, kp, cs, sn);
    }
    dst[h * dk + i] = qo;
    dst[H * dk + h * dk + i] = ko * k_scale;
  }
  for (int i = lane; i < dv; i += 64) {
    const float v = to_f32<T>(row[v_col + h * dv + i]);
    dst[2 * H * dk + h * dv + i] = act ? silu_f(v) : v;
  }
}

extern "C" int za_retention_prepare_act(const void* proj, int dtype, int proj_stride, int q_col,
                                    int k_col, int v_col, const int* positions,
                                    const float* inv_freq, float* prep, int n_tokens, int H, int dk,
                                    int dv, int rot, float k_scale, int act, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  if (n_tokens < 0 || H <= 0 || dk <= 0 || dv <= 0 || !proj || !positions || !prep || rot < 0 ||
      rot > dk || rot % 2 || (rot > 0 && !inv_freq) || q_col < 0 || k_col < 0 || v_col < 0 ||
      act < 0 || act > 1 || q_col + H * dk > proj_stride || k_col + H * dk > proj_stride ||
      v_col + H * dv > proj_stride)
    return ZA_ERR_ARG;
  dim3 grid(n_tokens, H), block(64);
  if (dtype == 0)
    hipLaunchKernelGGL((retention_prepare_kernel<float>), grid, block, 0, stream,
                       (const float*)proj, proj_stride, q_col, k_col, v_col, positions, inv_freq,
                       prep, H, dk, dv, rot, k_scale, act);
  else if (dtype == 1)
    hipLaunchKernelGGL((retention_prepare_kernel<bf16_t>), grid, block, 0, stream,
                       (const bf16_t*)proj, proj_stride, q_col, k_col, v_col, positions, inv_freq,
                       prep, H, dk, dv, rot, k_scale, act);
  else
    return ZA_ERR_UNSUPPORTED;
  return za_launch_status();
}

extern "C" int za_retention_prepare(const void* proj, int dtype, int proj_stride, int q_col,
                                    int k_col, int v_col, const int* positions,
                                    const float* inv_freq, float* prep, int n_tokens, int H, int dk,
                                    int dv, int rot, float k_scale, hipStream_t stream) {
  return za_retention_prepare_act(proj, dtype, proj_stride, q_col, k_col, v_col, positions,
                                  inv_freq, prep, n_tokens, H, dk, dv, rot, k_scale, 0, stream);
}

// ------------------------------------------------------------- gated group norm
// grid (tokens, groups); a workgroup reduces one group of `group` columns.
#define GN_VPT 16   // values a thread keeps between the sum of squares and the scaling
template <typename T>
__global__ void __launch_bounds__(256)
gated_group_norm_kernel(const float* __restrict__ y, const T* __restrict__ gate, int gate_stride,
                        int gate_col, const float* __restrict__ w, int wlen, T* __restrict__ out,
                        int out_stride, int out_col, int width, int group, float eps, int silu_gate,
                        int gate_first, float out_scale) {
  __shared__ float scratch[16];
  const int t = blockIdx.x, c0 = blockIdx.y * group;
  const float* yr = y + (size_t)t * width + c0;
  const T* gr = gate + (size_t)t * gate_stride + gate_col + c0;
  T* o = out + (size_t)t * out_stride + out_col + c0;
  const int bd = blockDim.x;
  float ss = 0.f;
  if (group <= bd * GN_VPT) {
    // one trip to memory: every load is requested before anything is summed
    float v[GN_VPT], act[GN_VPT], wv[GN_VPT];
#pragma unroll
    for (int k = 0; k < GN_VPT; ++k) {
      const int i = threadIdx.x + k * bd;
      v[k] = i < group ? yr[i] : 0.f;
      act[k] = i < group ? to_f32<T>(gr[i]) : 0.f;
      wv[k] = i < group ? w[(c0 + i) % wlen] : 0.f;
    }
#pragma unroll
    for (int k = 0; k < GN_VPT; ++k) {
      act[k] = silu_gate ? silu_f(act[k]) : sigmoid_f(act[k]);
      if (gate_first) v[k] *= act[k];
      ss += v[k] * v[k];
    }
    ss = block_sum(ss, scratch);
    const float scale = 1.0f / sqrtf(ss / (float)group + eps);
#pragma unroll
    for (int k = 0; k < GN_VPT; ++k) {
      const int i = threadIdx.x + k * bd;
      float r = v[k] * scale * wv[k];
      if (!gate_first) r *= act[k];
      if (i < group) o[i] = from_f32<T>(r * out_scale);
    }
    return;
  }
  for (int i = threadIdx.x; i < group; i += bd) {
    float v = yr[i];
    if (gate_first) {
      const float gv = to_f32<T>(gr[i]);
      v *= silu_gate ? silu_f(gv) : sigmoid_f(gv);
    }
    ss += v * v;
  }
  ss = block_sum(ss, scratch);
  const float scale = 1.0f / sqrtf(ss / (float)group + eps);
  for (int i = threadIdx.x; i < group; i += bd) {
    const float gv = to_f32<T>(gr[i]);
    const float act = silu_gate ? silu_f(gv) : sigmoid_f(gv);
    float v = yr[i];
    if (gate_first) v *= act;
    v = v * scale * w[(c0 + i) % wlen];
    if (!gate_first) v *= act;
    o[i] = from_f32<T>(v * out_scale);
  }
}

// The same for groups of at most 256 columns (a head's width): a wave a group, four
// groups a workgroup, the group's values in registers, the sum over the wave's lanes
// alone (no barrier).  grid: ceil(tokens * groups / 4).
template <typename T>
__global__ void __launch_bounds__(256)
gated_group_norm_wave_kernel(const float* __restrict__ y, const T* __restrict__ gate,
                             int gate_stride, int gate_col, const float* __restrict__ w, int wlen,
                             T* __restrict__ out, int out_stride, int out_col, int width, int group,
                             float eps, int silu_gate, int gate_first, float out_scale,
                             long long n_groups_total) {
  const int lane = threadIdx.x & 63;
  const long long gi = (long long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (gi >= n_groups_total) return;
  const int per_token = width / group;
  const size_t t = (size_t)(gi / per_token);
  const int c0 = (int)(gi % per_token) * group;
  const float* yr = y + t * width + c0;
  const T* gr = gate + t * gate_stride + gate_col + c0;
  T* o = out + t * out_stride + out_col + c0;
  float v[4], act[4], wv[4];
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    const int i = lane + 64 * k;
    v[k] = i < group ? yr[i] : 0.f;
    act[k] = i < group ? to_f32<T>(gr[i]) : 0.f;
    wv[k] = i < group ? w[(c0 + i) % wlen] : 0.f;
  }
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    act[k] = silu_gate ? silu_f(act[k]) : sigmoid_f(act[k]);
    if (gate_first) v[k] *= act[k];
    ss += v[k] * v[k];
  }
  ss = wave_sum(ss);
  const float scale = 1.0f / sqrtf(ss / (float)group + eps);
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    const int i = lane + 64 * k;
    float r = v[k] * scale * wv[k];
    if (!gate_first) r *= act[k];
    if (i < group) o[i] = from_f32<T>(r * out_scale);
  }
}

extern "C" int za_gated_group_norm(const float* y, const void* gate, int dtype, int gate_stride,
                                   int gate_col, const float* w, int wlen, void* out,
                                   int out_stride, int out_col, int n_tokens, int width, int group,
                                   float eps, int silu_gate, int gate_first, float out_scale,
                                   hipStream_t stream) {
  if (n_tokens == 0) return 0;
  if (n_tokens < 0 || width <= 0 || group <= 0 || width % group || !y || !gate || !w || !out ||
      wlen <= 0 || gate_col < 0 || gate_col + width > gate_stride || out_col < 0 ||
      out_col + width > out_stride)
    return ZA_ERR_ARG;
  if (group <= 256 && dtype >= 0 && dtype <= 1) {
    // small groups (a head each): a wave a group
    const long long total = (long long)n_tokens * (width / group);
    dim3 wgrid((unsigned)((total + 3) / 4)), wblock(256);
    if (dtype == 0)
      hipLaunchKernelGGL((gated_group_norm_wave_kernel<float>), wgrid, wblock, 0, stream, y,
                         (const float*)gate, gate_stride, gate_col, w, wlen, (float*)out, out_stride,
                         out_col, width, group, eps, silu_gate, gate_first, out_scale, total);
    else
      hipLaunchKernelGGL((gated_group_norm_wave_kernel<bf16_t>), wgrid, wblock, 0, stream, y,
                         (const bf16_t*)gate, gate_stride, gate_col, w, wlen, (bf16_t*)out,
                         out_stride, out_col, width, group, eps, silu_gate, gate_first, out_scale,
                         total);
    return za_launch_status();
  }
  dim3 grid(n_tokens, width / group), block(group <= 64 ? 64 : (group <= 128 ? 128 : 256));
  if (dtype == 0)
    hipLaunchKernelGGL((gated_group_norm_kernel<float>), grid, block, 0, stream, y,
                       (const float*)gate, gate_stride, gate_col, w, wlen, (float*)out, out_stride,
                       out_col, width, group, eps, silu_gate, gate_first, out_scale);
  else if (dtype == 1)
    hipLaunchKernelGGL((gated_group_norm_kernel<bf16_t>), grid, block, 0, stream, y,
                       (const bf16_t*)gate, gate_stride, gate_col, w, wlen, (bf16_t*)out,
                       out_stride, out_col, width, group, eps, silu_gate, gate_first, out_scale);
  else
    return ZA_ERR_UNSUPPORTED;
  return za_launch_status();
}
