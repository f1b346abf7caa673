// Attention on the matrix cores over a plane of keys and a plane of values of any widths
// (multiples of 8 up to 256), with a window and kept first keys, chunks and a sink a head.
//
//   query i sees key j  if  j <= i  and  (no window, or i - j < window, or j < keep)
//                           and  (no chunks, or j in i's chunk)
//   o[t,h] = sum_j e^(s_j) v_j / (sum_j e^(s_j) + e^(sink_h)),  s_j = (q . k_j) * scale
//
// A page holds the keys of all heads, [kv_head][offset][d], then the values turned round,
// [kv_head][dv][offset] (attention.hip).  The streaming softmax is the one of that file's
// matrix-core kernels: base-2 scale, the running maximum rounded up to a whole number so that
// every rescaling factor is an exact power of two, the sum taken over the rounded
// probabilities.
//
// Which keys a work item meets.  Behind a window most of a long context does not count for
// any row of an item: the item walks a list of tiles of 64 keys, first the tiles with kept keys
// that end before the window's first tile, then those from the window's first tile to the
// item's last position:
//   tile v of the list starts at key  v * 64  (v < n_kept),  first + (v - n_kept) * 64  (else)
// A list may be cut into `nsplit` ranges of `tiles_per_split` tiles (the last range takes what
// is left); the ranges' partial results are merged by attention_combine_kernel.
//
// The kernels are made for a few capacities DK >= d, DV >= dv.  Elements of a row beyond `d`
// (`dv`) are never read: the addresses are held inside the row (the piece before is read
// again), the queries' elements there are zero, and what comes out there is not stored.
#include "attention_common.h"

#define AP_KT 64       // keys of a tile
#define AP_ROWS 128    // rows (token, head) of a work item of the kernel for prompt portions

struct PlanesArgs {
  const bf16_t* q;             // [tokens][nh][d]
  bf16_t* out;                 // [tokens][nh][dv]
  const bf16_t* kv;
  const int* block_table;
  const int* positions;
  const int* wi_seq;
  const int* wi_row0;
  const int* wi_count;
  float* part_acc;             // [tokens][nh][nsplit][dv]
  float* part_ml;              // [tokens][nh][nsplit][2]
  const float* sink;           // [nh] or null
  int bt_stride, n_items, nh, nkv, d, dv, page_size;
  float scale_log2e;
  int window, keep, chunk, tiles_per_split, nsplit;
};

// The list of tiles of an item whose rows stand at positions pos_first .. pos_last.
struct TileList {
  int lo;        // first key of the window (or chunk) of the item's first row
  int hi;        // last key of all
  int first;     // first key of the first tile behind the kept ones
  int n_kept;    // tiles with kept keys ahead of it
  int n;         // tiles in all
  __device__ __forceinline__ int start(int v) const {
    return v < n_kept ? v * AP_KT : first + (v - n_kept) * AP_KT;
  }
};

__device__ __forceinline__ int planes_lo(const PlanesArgs& a, int position) {
  int lo = a.window > 0 && position - a.window + 1 > 0 ? position - a.window + 1 : 0;
  if (a.chunk > 0 && position > 0) {
    const int c = (position / a.chunk) * a.chunk;
    if (c > lo) lo = c;
  }
  return lo;
}

__device__ __forceinline__ TileList tile_list(const PlanesArgs& a, int pos_first, int pos_last) {
  TileList l;
  l.lo = planes_lo(a, pos_first);
  l.hi = pos_last;
  l.first = (l.lo / AP_KT) * AP_KT;
  const int kept = (a.keep + AP_KT - 1) / AP_KT, before = l.first / AP_KT;
  l.n_kept = kept < before ? kept : before;
  l.n = l.n_kept + (l.hi - l.first) / AP_KT + 1;
  return l;
}

// ------------------------------------------------------------- prompt portions
// A workgroup serves up to 128 rows of one work item and one key/value head; each of its
// eight waves owns 16 rows.  Keys and values go through two LDS buffers: while a tile is being
// computed the next one is on its way into registers.  See paged_attention_mfma_kernel
// (attention.hip) for the products' operand layout.
template <int DK, int DV>
__global__ void __launch_bounds__(512)
planes_attention_kernel(PlanesArgs a) {
  constexpr int NW = 8, NT = NW * 64, KT = AP_KT;
  constexpr int LDK = DK + 8, LDV = KT + 8;        // padded rows, in elements
  constexpr int KSTEPS = DK / 32, DBLK = DV / 16;
  constexpr int KCOLS = DK / 8;                    // 16-byte pieces of a key
  constexpr int KVEC = (KT * KCOLS + NT - 1) / NT;
  constexpr int VRUNS = KT / 4;                    // runs of 4 keys in a tile
  constexpr int VVEC = (DV * VRUNS + NT - 1) / NT;
  constexpr int JB = KT / 16, KK = KT / 32;
  extern __shared__ __attribute__((aligned(16))) unsigned char ap_smem[];
  bf16_t* Ks = reinterpret_cast<bf16_t*>(ap_smem);   // [2][key][dim]
  bf16_t* Vt = Ks + 2 * KT * LDK;                    // [2][dim][key slot]

  const int gkv = blockIdx.x, z = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int r16 = lane & 15, grp = lane >> 4;
  const int nh = a.nh, nkv = a.nkv, d = a.d, dv = a.dv, page_size = a.page_size;
  const int window = a.window, keep = a.keep;
  const int G = nh / nkv;
  const bf16x8_t zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  const int last_entry = a.bt_stride - 1;
  const int ps_shift = page_shift_of(page_size);

  // (an item's work grows with its place in a prompt: the second half of the grid takes its
  // items in descending order, so that neighbours weigh about the same in pairs)
  int item = blockIdx.y;
  {
    const int half = a.n_items / 2;
    if (item >= half) item = a.n_items - 1 - (item - half);
  }
  const int seq = a.wi_seq[item], row0 = a.wi_row0[item];
  int count = a.wi_count[item];
  if (count * G > AP_ROWS) count = AP_ROWS / G;   // the host never asks for more
  const int rows = count * G;
  const int* table = a.block_table + (size_t)seq * a.bt_stride;

  const int rr = wave * 16 + r16;
  const bool row_valid = rr < rows;
  const int tok = row0 + (row_valid ? rr / G : 0);
  const int head = gkv * G + (row_valid ? rr % G : 0);
  const int pos_row = row_valid ? a.positions[tok] : -1;
  bf16x8_t qf[KSTEPS];
#pragma unroll
  for (int ks = 0; ks < KSTEPS; ++ks) {
    const int e = ks * 32 + grp * 8;
    qf[ks] = row_valid && e < d
                 ? *reinterpret_cast<const bf16x8_t*>(a.q + ((size_t)tok * nh + head) * d + e) : zero8;
  }

  const TileList list = tile_list(a, a.positions[row0], a.positions[row0 + count - 1]);
  const int lo = list.lo, hi = list.hi;
  const int v_first = z * a.tiles_per_split;
  const int v_end = z == a.nsplit - 1 ? list.n : min(list.n, v_first + a.tiles_per_split);
  const int row_lo = row_valid ? planes_lo(a, pos_row) : 0;
  // what this wave's rows can see
  const int wave_first_row = wave * 16;
  const bool wave_active = wave_first_row < rows;
  const bool wave_full = wave_first_row + 16 <= rows;
  const int wave_last_tok = min((wave_first_row + 15) / G, count - 1);
  const int wave_hi = wave_active ? a.positions[row0 + wave_last_tok] : -1;
  const int wave_lo = wave_active ? a.positions[row0 + wave_first_row / G] : 0;
  const int seen_from = planes_lo(a, wave_lo);     // first key any row of the wave sees
  const int full_from = planes_lo(a, wave_hi);     // from here every row of the wave sees

  f32x4_t o[DBLK], lsum = {0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY;
  bf16x8_t ones8;
#pragma unroll
  for (int i = 0; i < 8; ++i) ones8[i] = (bf16_t)1.0f;
#pragma unroll
  for (int db = 0; db < DBLK; ++db) o[db] = (f32x4_t){0.f, 0.f, 0.f, 0.f};

  // This thread's pieces of a tile: KVEC 16-byte pieces of keys, and VVEC 8-byte runs of 4
  // consecutive keys (run vkr of the tile) for head-dim elements vdd0 + v * (NT / VRUNS).
  const unsigned page_stride = (unsigned)nkv * (unsigned)page_size * (unsigned)(d + dv);
  const bf16_t* kbase = a.kv + (size_t)gkv * page_size * d;
  const bf16_t* vbase = a.kv + (size_t)nkv * page_size * d + (size_t)gkv * page_size * dv;
  int krow[KVEC], kcol[KVEC];
#pragma unroll
  for (int v = 0; v < KVEC; ++v) {
    const int piece = min(tid + v * NT, KT * KCOLS - 1);
    krow[v] = piece / KCOLS;
    kcol[v] = (piece % KCOLS) * 8;
  }
  const int vkr = tid & (VRUNS - 1), vdd0 = tid / VRUNS;
  int voff[VVEC];
#pragma unroll
  for (int v = 0; v < VVEC; ++v) voff[v] = min(vdd0 + v * (NT / VRUNS), dv - 1) * page_size;

  int kpg[KVEC], vpg;
  bf16x8_t kreg[KVEC];
  bf16x4_t vreg[VVEC];
  auto load_pages = [&](int tile0) {
#pragma unroll
    for (int v = 0; v < KVEC; ++v) {
      const int e = page_entry(tile0 + krow[v], page_size, ps_shift);
      kpg[v] = table[e < last_entry ? e : last_entry];
    }
    const int e = page_entry(tile0 + vkr * 4, page_size, ps_shift);
    vpg = table[e < last_entry ? e : last_entry];
  };
  // Loads never leave the pool: an unused table entry (-1) reads page 0 instead, and
  // tiles beyond the last one are fetched like any other.  A key that must not count is
  // masked in the scores, whatever its row holds; its values are cleared on their way
  // into LDS, since 0 * (not a number) would not be 0.
  auto load_data = [&](int tile0) {
#pragma unroll
    for (int v = 0; v < KVEC; ++v) {
      const int off = page_offset(tile0 + krow[v], page_size, ps_shift);
      const unsigned page = kpg[v] < 0 ? 0u : (unsigned)kpg[v];
      const int col = min(kcol[v], d - 8);
      kreg[v] = *reinterpret_cast<const bf16x8_t*>(
          kbase + ((size_t)page * page_stride + (unsigned)(off * d + col)));
    }
    const int off = page_offset(tile0 + vkr * 4, page_size, ps_shift);
    const unsigned page = vpg < 0 ? 0u : (unsigned)vpg;
    const bf16_t* src = vbase + ((size_t)page * page_stride + (unsigned)off);
#pragma unroll
    for (int v = 0; v < VVEC; ++v)
      vreg[v] = *reinterpret_cast<const bf16x4_t*>(src + voff[v]);
  };
  // keys jb * 16 + g4 * 4 .. + 3 of the tile sit in slots: 32-key step, then lane group,
  // then block
  const int vslot = (vkr >> 3) * 32 + (vkr & 3) * 8 + ((vkr >> 2) & 1) * 4;
  auto store_tile = [&](int buf, int tile0) {
    bf16_t* ks = Ks + buf * KT * LDK;
    bf16_t* vt = Vt + buf * DV * LDV;
#pragma unroll
    for (int v = 0; v < KVEC; ++v)
      if ((v + 1) * NT <= KT * KCOLS || tid + v * NT < KT * KCOLS)
        *reinterpret_cast<bf16x8_t*>(ks + krow[v] * LDK + kcol[v]) = kreg[v];
    const int kp = tile0 + vkr * 4;
    const bool edge_tile = tile0 < lo || tile0 + KT - 1 > hi;   // the same for all threads
#pragma unroll
    for (int v = 0; v < VVEC; ++v) {
      bf16x4_t x = vreg[v];
      if (edge_tile) {
        // keys that no row sees (pages that are not there are among them)
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if ((kp + e < lo && kp + e >= keep) || kp + e > hi) x[e] = (bf16_t)0.f;
      }
      const int dd = vdd0 + v * (NT / VRUNS);
      if ((v + 1) * NT <= DV * VRUNS || dd < DV)
        *reinterpret_cast<bf16x4_t*>(vt + dd * LDV + vslot) = x;
    }
  };

  if (v_first < v_end) {
    const int tile0 = list.start(v_first);
    load_pages(tile0);
    load_data(tile0);
    load_pages(list.start(v_first + 1));
    store_tile(0, tile0);
  }
  __syncthreads();

  for (int v = v_first; v < v_end; ++v) {
    const int tile0 = list.start(v);
    const int buf = (v - v_first) & 1;
    const int tile1 = list.start(v + 1);
    load_data(tile1);
    load_pages(list.start(v + 2));

    const bool wave_sees =
        wave_active && tile0 <= wave_hi && (tile0 + KT - 1 >= seen_from || tile0 < keep);
    if (wave_sees) {
      const bf16_t* ks = Ks + buf * KT * LDK;
      const bf16_t* vt = Vt + buf * DV * LDV;
      f32x4_t s[JB];
#pragma unroll
      for (int jb = 0; jb < JB; ++jb) {
        s[jb] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks_ = 0; ks_ < KSTEPS; ++ks_) {
          const bf16x8_t kf = *reinterpret_cast<const bf16x8_t*>(
              ks + (jb * 16 + r16) * LDK + ks_ * 32 + grp * 8);
          s[jb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[ks_], s[jb], 0, 0, 0);
        }
      }
      // a tile every key of which counts for every row of the wave needs no mask
      const bool needs_mask = !wave_full || tile0 + KT - 1 > wave_lo ||
                              (tile0 < full_from && tile0 + KT > keep);
      if (needs_mask) {
        // key jb * 16 + grp * 4 + i of the tile counts for this lane's row if it is at most
        // `last` and at least `first` or below `kept`, all relative to the lane's own keys
        const int base = tile0 + grp * 4;
        const int last = pos_row - base, first = row_lo - base, kept = keep - base;
#pragma unroll
        for (int jb = 0; jb < JB; ++jb)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int k = jb * 16 + i;
            if (!(k <= last && (k >= first || k < kept))) s[jb][i] = -INFINITY;
          }
      }
      float tmax = -INFINITY;
#pragma unroll
      for (int jb = 0; jb < JB; ++jb)
#pragma unroll
        for (int i = 0; i < 4; ++i) tmax = fmaxf(tmax, s[jb][i]);
      tmax = quad_max(tmax);
      const float m_new = fmaxf(m, ceilf(tmax * a.scale_log2e));   // the factor is positive
      const float m_use = m_new > -INFINITY ? m_new : 0.f;
      const float alpha = m > -INFINITY ? ldexpf(1.0f, (int)(m - m_use)) : 1.0f;
#pragma unroll
      for (int jb = 0; jb < JB; ++jb)
#pragma unroll
        for (int i = 0; i < 4; ++i)   // masked scores (-inf) give 0
          s[jb][i] = __builtin_amdgcn_exp2f(fmaf(s[jb][i], a.scale_log2e, -m_use));
      m = m_new;
      if (__any(alpha != 1.0f)) {
#pragma unroll
        for (int i = 0; i < 4; ++i) lsum[i] *= alpha;
#pragma unroll
        for (int db = 0; db < DBLK; ++db)
#pragma unroll
          for (int i = 0; i < 4; ++i) o[db][i] *= alpha;
      }
      bf16x8_t pf[KK];
#pragma unroll
      for (int kk = 0; kk < KK; ++kk) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          pf[kk][i] = (bf16_t)s[2 * kk][i];
          pf[kk][4 + i] = (bf16_t)s[2 * kk + 1][i];
        }
        lsum = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones8, pf[kk], lsum, 0, 0, 0);
      }
#pragma unroll
      for (int db = 0; db < DBLK; ++db)
#pragma unroll
        for (int kk = 0; kk < KK; ++kk) {
          const bf16x8_t vf = *reinterpret_cast<const bf16x8_t*>(
              vt + (db * 16 + r16) * LDV + kk * 32 + grp * 8);
          o[db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pf[kk], o[db], 0, 0, 0);
        }
    }
    if (v + 1 < v_end) store_tile(buf ^ 1, tile1);
    __syncthreads();
  }

  if (!row_valid) return;
  const size_t orow = (size_t)tok * nh + head;
  if (a.nsplit > 1) {
    // unnormalised accumulator, and (maximum, sum), the maximum on the base-2 scale
    float* pa = a.part_acc + (orow * a.nsplit + z) * dv;
#pragma unroll
    for (int db = 0; db < DBLK; ++db)
      if (db * 16 + grp * 4 < dv) *reinterpret_cast<f32x4_t*>(pa + db * 16 + grp * 4) = o[db];
    if (grp == 0) {
      a.part_ml[(orow * a.nsplit + z) * 2] = m;
      a.part_ml[(orow * a.nsplit + z) * 2 + 1] = lsum[0];
    }
    return;
  }
  float total = lsum[0];
  if (a.sink && m > -INFINITY) total += exp2f(a.sink[head] * ZA_LOG2E - m);
  const float inv = total > 0.f ? 1.0f / total : 0.f;
  bf16_t* dst = a.out + orow * dv;
#pragma unroll
  for (int db = 0; db < DBLK; ++db) {
    bf16x4_t ov;
#pragma unroll
    for (int i = 0; i < 4; ++i) ov[i] = (bf16_t)(o[db][i] * inv);
    if (db * 16 + grp * 4 < dv) *reinterpret_cast<bf16x4_t*>(dst + db * 16 + grp * 4) = ov;
  }
}

// -------------------------------------------------------------------- decoding
// Every request brings one token: row i of q is request i's.  The G <= 16 query heads of a
// key/value head are the columns of the second operand; the waves of a workgroup take the tiles
// of the workgroup's range in turn and never wait for each other inside the loop, keys and
// values go from memory straight into first-operand fragments.  See
// paged_attention_decode_mfma_kernel (attention.hip) for how a tile's keys are dealt to the
// fragments' rows.  AHEAD: the next tile is fetched while this one is being computed (narrow
// heads; the fragments of two tiles must fit the registers).
template <int DK, int DV, int NWV, bool AHEAD>
__global__ void __launch_bounds__(NWV * 64)
planes_decode_kernel(PlanesArgs a) {
  constexpr int KSTEPS = DK / 32, DBLK = DV / 16, KT = AP_KT;
  extern __shared__ __attribute__((aligned(16))) unsigned char ap_smem[];
  __shared__ float mg_m[NWV][16], mg_l[NWV][16];
  float* mg_o = reinterpret_cast<float*>(ap_smem);   // [NWV][DBLK][4][64]

  const int item = blockIdx.x, gkv = blockIdx.y, z = blockIdx.z;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int r16 = lane & 15, grp = lane >> 4;
  const int nh = a.nh, nkv = a.nkv, d = a.d, dv = a.dv, page_size = a.page_size, keep = a.keep;
  const int G = nh / nkv;
  const int* table = a.block_table + (size_t)item * a.bt_stride;
  const int pos = a.positions[item];
  const bool row_valid = r16 < G;
  const int head = gkv * G + (row_valid ? r16 : 0);
  const bf16x8_t zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  bf16x8_t qf[KSTEPS];
#pragma unroll
  for (int ks = 0; ks < KSTEPS; ++ks) {
    const int e = ks * 32 + grp * 8;
    qf[ks] = row_valid && e < d
                 ? *reinterpret_cast<const bf16x8_t*>(a.q + ((size_t)item * nh + head) * d + e) : zero8;
  }

  f32x4_t o[DBLK];
#pragma unroll
  for (int db = 0; db < DBLK; ++db) o[db] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, l = 0.f;

  const int last_entry = a.bt_stride - 1;
  const int ps_shift = page_shift_of(page_size);
  const bool wide = page_size % 8 == 0;
  const int krow_in_pair = (r16 >> 2) * 8 + (r16 & 3);   // + (jb / 2) * 32 + (jb % 2) * 4
  const size_t page_stride = (size_t)nkv * page_size * (d + dv);
  const bf16_t* kbase = a.kv + (size_t)gkv * page_size * d;
  const bf16_t* vbase = a.kv + (size_t)nkv * page_size * d + (size_t)gkv * page_size * dv;
  int kelem[KSTEPS], velem[DBLK];
#pragma unroll
  for (int ks = 0; ks < KSTEPS; ++ks) kelem[ks] = min(ks * 32 + grp * 8, d - 8);
#pragma unroll
  for (int db = 0; db < DBLK; ++db) velem[db] = min(db * 16 + r16, dv - 1) * page_size;

  const TileList list = tile_list(a, pos, pos);
  const int lo = list.lo, hi = list.hi;
  const int v_end = z == a.nsplit - 1 ? list.n : min(list.n, (z + 1) * a.tiles_per_split);
  auto entry_of = [&](int key) {
    const int e = page_entry(key, page_size, ps_shift);
    return table[e < last_entry ? e : last_entry];
  };
  // With pages of 16, 32, 64 ... keys a block of 16 keys lies in one page: the entries of the
  // wave's next sixteen tiles are read by ONE vector load, lane i * 4 + b taking block b of the
  // i-th tile, and handed out lane by lane.
  int tbl = 0;
  auto load_entries = [&](int v) {
    const int key = list.start(v + (lane >> 2) * NWV) + (lane & 3) * 16;
    const int e = key >> (ps_shift >= 4 ? ps_shift : 4);
    tbl = table[e < last_entry ? e : last_entry];
  };
  auto fetch = [&](int tile0, int nth, bf16x8_t (&kfr)[4][KSTEPS], bf16x8_t (&vfr)[DBLK][2]) {
    int kpage[4], vpage[4];      // vpage: per run of 4 keys, kk * 2 + half
    if (ps_shift >= 4) {
      const int first = __builtin_amdgcn_readfirstlane(nth) * 4;
      int pg[4];
#pragma unroll
      for (int b = 0; b < 4; ++b) pg[b] = __builtin_amdgcn_readlane(tbl, first + b);
#pragma unroll
      for (int jb = 0; jb < 4; ++jb) {
        kpage[jb] = (r16 & 8) ? pg[(jb >> 1) * 2 + 1] : pg[(jb >> 1) * 2];
        vpage[jb] = (grp & 2) ? pg[(jb >> 1) * 2 + 1] : pg[(jb >> 1) * 2];
      }
    } else {
#pragma unroll
      for (int jb = 0; jb < 4; ++jb) {
        kpage[jb] = entry_of(tile0 + (jb >> 1) * 32 + (jb & 1) * 4 + krow_in_pair);
        vpage[jb] = entry_of(tile0 + (jb >> 1) * 32 + grp * 8 + (jb & 1) * 4);
      }
    }
#pragma unroll
    for (int jb = 0; jb < 4; ++jb) {
      const int kp = tile0 + (jb >> 1) * 32 + (jb & 1) * 4 + krow_in_pair;
      const size_t page = kpage[jb] < 0 ? 0 : kpage[jb];
      const bf16_t* krow = kbase + page * page_stride + page_offset(kp, page_size, ps_shift) * d;
#pragma unroll
      for (int ks = 0; ks < KSTEPS; ++ks)
        kfr[jb][ks] = *reinterpret_cast<const bf16x8_t*>(krow + kelem[ks]);
    }
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      const int kp = tile0 + kk * 32 + grp * 8;          // this lane's eight keys
      const size_t page_a = vpage[2 * kk] < 0 ? 0 : vpage[2 * kk];
      const size_t page_b = vpage[2 * kk + 1] < 0 ? 0 : vpage[2 * kk + 1];
      const bf16_t* va = vbase + page_a * page_stride + page_offset(kp, page_size, ps_shift);
      const bf16_t* vb = vbase + page_b * page_stride + page_offset(kp + 4, page_size, ps_shift);
#pragma unroll
      for (int db = 0; db < DBLK; ++db) {
        bf16x8_t x;
        if (wide) {
          x = *reinterpret_cast<const bf16x8_t*>(va + velem[db]);
        } else {
          const bf16x4_t xa = *reinterpret_cast<const bf16x4_t*>(va + velem[db]);
          const bf16x4_t xb = *reinterpret_cast<const bf16x4_t*>(vb + velem[db]);
          x = __builtin_shufflevector(xa, xb, 0, 1, 2, 3, 4, 5, 6, 7);
        }
        vfr[db][kk] = x;
      }
    }
  };

  bf16x8_t kf[4][KSTEPS];
  bf16x8_t vf[DBLK][2];
  int v = z * a.tiles_per_split + wave;
  int nth = 0;
  if (v < v_end) {
    if (ps_shift >= 4) load_entries(v);
    if (AHEAD) fetch(list.start(v), 0, kf, vf);
  }
  for (; v < v_end; v += NWV) {
    const int tile0 = list.start(v);
    [[maybe_unused]] bf16x8_t kfn[AHEAD ? 4 : 1][KSTEPS];
    [[maybe_unused]] bf16x8_t vfn[AHEAD ? DBLK : 1][2];
    const int next = v + NWV;
    if constexpr (AHEAD) {
      if (next < v_end) {
        if (++nth == 16) {
          nth = 0;
          if (ps_shift >= 4) load_entries(next);
        }
        fetch(list.start(next), nth, kfn, vfn);
      }
    } else {
      if (nth == 16) {
        nth = 0;
        if (ps_shift >= 4) load_entries(v);
      }
      fetch(tile0, nth++, kf, vf);
    }
    // A key that must not count is masked in the scores, whatever its row holds; its
    // values are cleared, since 0 * (not a number) would not be 0.
    if (tile0 < lo || tile0 + KT - 1 > hi) {
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const int kp = tile0 + kk * 32 + grp * 8;
#pragma unroll
        for (int db = 0; db < DBLK; ++db)
#pragma unroll
          for (int e = 0; e < 8; ++e)
            if ((kp + e < lo && kp + e >= keep) || kp + e > hi) vf[db][kk][e] = (bf16_t)0.f;
      }
    }

    f32x4_t s[4];
#pragma unroll
    for (int jb = 0; jb < 4; ++jb) {
      s[jb] = (f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ks = 0; ks < KSTEPS; ++ks)
        s[jb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[jb][ks], qf[ks], s[jb], 0, 0, 0);
    }
    float tmax = -INFINITY;
#pragma unroll
    for (int jb = 0; jb < 4; ++jb)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int kp = tile0 + (jb >> 1) * 32 + grp * 8 + (jb & 1) * 4 + i;
        const bool valid = row_valid && kp <= hi && (kp >= lo || kp < keep);
        s[jb][i] = valid ? s[jb][i] * a.scale_log2e : -INFINITY;
        tmax = fmaxf(tmax, s[jb][i]);
      }
    tmax = quad_max(tmax);
    const float m_new = fmaxf(m, ceilf(tmax));
    const float m_use = m_new > -INFINITY ? m_new : 0.f;
    const float alpha = m > -INFINITY ? ldexpf(1.0f, (int)(m - m_use)) : 1.0f;
#pragma unroll
    for (int jb = 0; jb < 4; ++jb)
#pragma unroll
      for (int i = 0; i < 4; ++i) s[jb][i] = __builtin_amdgcn_exp2f(s[jb][i] - m_use);
    m = m_new;
#pragma unroll
    for (int db = 0; db < DBLK; ++db)
#pragma unroll
      for (int i = 0; i < 4; ++i) o[db][i] *= alpha;
    bf16x8_t pf[2];
    float psum = 0.f;
#pragma unroll
    for (int kk = 0; kk < 2; ++kk)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        pf[kk][i] = (bf16_t)s[2 * kk][i];
        pf[kk][4 + i] = (bf16_t)s[2 * kk + 1][i];
        psum += (float)pf[kk][i] + (float)pf[kk][4 + i];
      }
    psum = quad_sum(psum);
    l = l * alpha + psum;
#pragma unroll
    for (int db = 0; db < DBLK; ++db)
#pragma unroll
      for (int kk = 0; kk < 2; ++kk)
        o[db] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[db][kk], pf[kk], o[db], 0, 0, 0);
    if constexpr (AHEAD) {
      if (next < v_end) {
#pragma unroll
        for (int jb = 0; jb < 4; ++jb)
#pragma unroll
          for (int ks = 0; ks < KSTEPS; ++ks) kf[jb][ks] = kfn[jb][ks];
#pragma unroll
        for (int db = 0; db < DBLK; ++db) {
          vf[db][0] = vfn[db][0];
          vf[db][1] = vfn[db][1];
        }
      }
    }
  }

  // merge the waves' partial results: wave w merges head-dim blocks w, w + NWV, ...
  if (grp == 0) {
    mg_m[wave][r16] = m;
    mg_l[wave][r16] = l;
  }
#pragma unroll
  for (int db = 0; db < DBLK; ++db)
    *reinterpret_cast<f32x4_t*>(mg_o + ((wave * DBLK + db) * 64 + lane) * 4) = o[db];
  __syncthreads();
  if (!row_valid) return;
  float mx = mg_m[0][r16];
#pragma unroll
  for (int w = 1; w < NWV; ++w) mx = fmaxf(mx, mg_m[w][r16]);
  const float mu = mx > -INFINITY ? mx : 0.f;
  float wgt[NWV], total = 0.f;
#pragma unroll
  for (int w = 0; w < NWV; ++w) {
    wgt[w] = mg_m[w][r16] > -INFINITY ? ldexpf(1.0f, (int)(mg_m[w][r16] - mu)) : 0.f;
    total += mg_l[w][r16] * wgt[w];
  }
  if (a.sink && a.nsplit == 1 && mx > -INFINITY) total += exp2f(a.sink[head] * ZA_LOG2E - mu);
  const float inv = total > 0.f ? 1.0f / total : 0.f;
  const size_t orow = (size_t)item * nh + head;
  for (int db = wave; db < DBLK; db += NWV) {
    if (db * 16 + grp * 4 >= dv) continue;
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < NWV; ++w) {
      const f32x4_t x = *reinterpret_cast<const f32x4_t*>(mg_o + ((w * DBLK + db) * 64 + lane) * 4);
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i] = fmaf(x[i], wgt[w], acc[i]);
    }
    if (a.nsplit == 1) {
      bf16x4_t ov;
#pragma unroll
      for (int i = 0; i < 4; ++i) ov[i] = (bf16_t)(acc[i] * inv);
      *reinterpret_cast<bf16x4_t*>(a.out + orow * dv + db * 16 + grp * 4) = ov;
    } else {
      *reinterpret_cast<f32x4_t*>(a.part_acc + (orow * a.nsplit + z) * dv + db * 16 + grp * 4) = acc;
    }
  }
  if (a.nsplit > 1 && wave == 0 && grp == 0) {
    a.part_ml[(orow * a.nsplit + z) * 2] = mx;
    a.part_ml[(orow * a.nsplit + z) * 2 + 1] = total;
  }
}

static int allow_lds(const void* kernel, size_t bytes, bool* done) {
  if (*done) return 0;
  const hipError_t e =
      hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
  if (e != hipSuccess) return (int)e;
  *done = true;
  return 0;
}

template <int DK, int DV>
static int launch_planes(const PlanesArgs& a, hipStream_t stream) {
  constexpr size_t shmem =
      ((size_t)2 * AP_KT * (DK + 8) + (size_t)2 * DV * (AP_KT + 8)) * sizeof(bf16_t);
  auto kernel = planes_attention_kernel<DK, DV>;
  static bool allowed = false;
  if (const int rc = allow_lds((const void*)kernel, shmem, &allowed)) return rc;
  // the key/value head runs fastest, so that workgroups that follow each other (and
  // are dealt to the chip's eight dies in turn) read different heads' keys and values
  hipLaunchKernelGGL(kernel, dim3(a.nkv, a.n_items, a.nsplit), dim3(512), shmem, stream, a);
  return za_launch_status();
}

#define AP_DECODE_WIDE_BELOW 384   // workgroups: up to here all but the widest heads run eight waves

template <int DK, int DV, int NWV>
static int launch_planes_decode_waves(const PlanesArgs& a, hipStream_t stream) {
  constexpr size_t shmem = (size_t)NWV * (DV / 16) * 64 * 4 * sizeof(float);
  // (two tiles' fragments at once where they fit the registers of NWV waves)
  auto kernel = planes_decode_kernel<DK, DV, NWV, (DK + DV <= (NWV == 8 ? 160 : 256))>;
  static bool allowed = false;
  if (const int rc = allow_lds((const void*)kernel, shmem, &allowed)) return rc;
  hipLaunchKernelGGL(kernel, dim3(a.n_items, a.nkv, a.nsplit), dim3(NWV * 64), shmem, stream, a);
  return za_launch_status();
}

template <int DK, int DV>
static int launch_planes_decode(const PlanesArgs& a, hipStream_t stream) {
  if constexpr (DK + DV <= 256) {
    if ((long long)a.n_items * a.nkv * a.nsplit <= AP_DECODE_WIDE_BELOW)
      return launch_planes_decode_waves<DK, DV, 8>(a, stream);
  }
  return launch_planes_decode_waves<DK, DV, 4>(a, stream);
}

// The capacities the kernels are built for: the first pair that holds (d, dv).
#define AP_FOR_CAPACITIES(CASE)                                                                \
  CASE(64, 32) CASE(64, 64) CASE(96, 48) CASE(96, 64) CASE(96, 96) CASE(128, 64) CASE(128, 96) \
  CASE(128, 128) CASE(192, 96) CASE(192, 128) CASE(192, 192) CASE(256, 128) CASE(256, 256)

// bfloat16; d and dv multiples of 8 up to 256; page sizes that are multiples of 4; a positive
// scale.  wi_seq null: a step of single tokens, row i of q is request i's token (n_items ==
// n_tokens, at most 16 query heads a key/value head); otherwise work items of at most
// 128 / (nh / nkv) query tokens.
extern "C" int za_planes_attention(const void* q, void* out, const void* kv, const int* block_table,
                                   int bt_stride, const int* positions, const int* wi_seq,
                                   const int* wi_row0, const int* wi_count, int n_items,
                                   int n_tokens, float* part_acc, float* part_ml, int nh, int nkv,
                                   int d, int dv, int page_size, float scale, int window, int keep,
                                   int chunk, int tiles_per_split, int nsplit, const float* sink,
                                   hipStream_t stream) {
  if (n_items == 0 || n_tokens == 0) return 0;
  if (n_items < 0 || n_tokens < 0 || nh <= 0 || nkv <= 0 || nh % nkv != 0 || page_size <= 0 ||
      bt_stride <= 0 || nsplit < 1 || !q || !out || !kv || !block_table || !positions ||
      window < 0 || keep < 0 || chunk < 0)
    return ZA_ERR_ARG;
  if (nsplit > 1 && (!part_acc || !part_ml || tiles_per_split <= 0)) return ZA_ERR_ARG;
  if (wi_seq && (!wi_row0 || !wi_count)) return ZA_ERR_ARG;
  if (!wi_seq && n_items != n_tokens) return ZA_ERR_ARG;
  if (d <= 0 || dv <= 0 || d % 8 != 0 || dv % 8 != 0 || page_size % 4 != 0 || !(scale > 0.f) ||
      nkv > 65535 || nsplit > 65535 || n_items > 65535 ||
      (unsigned long long)nkv * page_size * (d + dv) > 0xffffffffull ||
      nh / nkv > (wi_seq ? AP_ROWS : 16))
    return ZA_ERR_UNSUPPORTED;
  const PlanesArgs a = {(const bf16_t*)q, (bf16_t*)out, (const bf16_t*)kv, block_table, positions,
                        wi_seq, wi_row0, wi_count, part_acc, part_ml, sink, bt_stride, n_items, nh,
                        nkv, d, dv, page_size, scale * ZA_LOG2E, window, keep,
                        chunk, nsplit > 1 ? tiles_per_split : 0, nsplit};
  int rc = ZA_ERR_UNSUPPORTED;
#define AP_CASE(DK, DV)                                                              \
  if (rc == ZA_ERR_UNSUPPORTED && d <= DK && dv <= DV)                               \
    rc = wi_seq ? launch_planes<DK, DV>(a, stream) : launch_planes_decode<DK, DV>(a, stream);
  AP_FOR_CAPACITIES(AP_CASE)
#undef AP_CASE
  if (rc != 0 || nsplit == 1) return rc;
  hipLaunchKernelGGL((attention_combine_kernel<bf16_t>), dim3((unsigned)((size_t)n_tokens * nh)),
                     dim3(64), 0, stream, part_acc, part_ml, (bf16_t*)out, dv, nsplit, 1, sink, nh);
  return za_launch_status();
}
