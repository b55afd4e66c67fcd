// Paged causal attention on the matrix cores (v_mfma_f32_16x16x32_bf16), bfloat16 in, float softmax.
//
// One wave owns NT*16 *columns* of one (request, key/value head): a column is a (token, query head of the
// group) pair, so every key and value that is loaded serves all query heads that share it, and in a prompt
// portion also NT*16/group consecutive tokens.  Keys are walked in blocks of 32:
//
//   S^T[key, col]  = K[key, :] . Q^T[:, col]        A operand: 16 keys x 32 dims, read in place from the
//                                                   page (a lane reads 16 contiguous bytes of one key);
//                                                   B operand: the query, kept in registers
//   online softmax per column in float, in log2 units (scale * log2(e) is folded into the exponent's
//   multiply-add); the running reference follows the maximum in steps, so rescaling is rare
//   O^T[dim, col] += V^T[dim, key] . P^T[key, col]  B operand: P^T straight from the S^T accumulators (a lane
//                                                   holds 4+4 keys of its own column: no transpose);
//                                                   A operand: V^T, which is why value pages are stored
//                                                   transposed, [page][kv head][dim][page_size]: a lane reads
//                                                   8 contiguous bytes (4 keys) of one dim from each page.
//
// The WAVES waves of a block share a column tile and take its key blocks in turn (wave w: blocks w, w + WAVES,
// ...), each with its own running maximum, sum and accumulators; at the end they are merged through LDS by
// wave 0 in a fixed order.  That shortens the chain of dependent key blocks (a late prompt tile, a long
// context) by WAVES and puts several waves on every SIMD to hide the latency of the page reads.  The next
// block's keys and values are loaded while the current one is multiplied.  Keys beyond a column's own
// position are masked, values beyond the last visible key are zeroed before use, and pages past the
// context are never dereferenced, so what a reused page still holds cannot reach the result.
//
// Two launch shapes: general (any mix of portions and single tokens; grid = column tiles x kv heads x
// requests, surplus tiles leave at once; a decode-only batch is the case of one tile per request) and
// split (every request has one token and a long context: the keys are also split over several blocks which
// write unnormalised partial results, and a second kernel combines them).
#include "common.h"
#include "api.h"
#include <algorithm>

namespace {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

__device__ __forceinline__ float fast_exp2(float x) { return __builtin_amdgcn_exp2f(x); }

__device__ __forceinline__ float fast_sigmoid(float x) {
  return __builtin_amdgcn_rcpf(1.0f + fast_exp2(-1.4426950408889634f * x));
}

constexpr float REF_SLACK = 8.0f;   // log2 units by which a column's maximum may run ahead of its reference

template <int D>
struct KeyBlock {          // one block of 32 keys as this lane sees it
  bf16x8 k[2][D / 32];     // [16-key subtile][32-dim step]
};
template <int CT>
struct ValueBlock {        // and its values, for the CT tiles of 16 dims that this block works out
  bf16x4 v[CT][2];         // [16-dim tile][subtile]: 4 keys of one dim; the two subtiles are one MFMA operand
};

// Page arithmetic: pages of a power of two (page_shift >= 0) need no division.
struct PageGeom {
  int size, shift;
  __device__ __forceinline__ int index(int key) const { return shift >= 0 ? key >> shift : key / size; }
  __device__ __forceinline__ int offset(int key) const { return shift >= 0 ? key & (size - 1) : key % size; }
};

// The pages of the two 16-key halves of the block at `base` (the same for every lane, so they are kept in
// scalar registers and so is all address arithmetic that follows from them); past the context: the null page.
__device__ __forceinline__ void pages_of(const int* __restrict__ table, int base, int key_hi, PageGeom pg,
                                         int* pages) {
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int kb = base + u * 16;
    pages[u] = kb <= key_hi ? __builtin_amdgcn_readfirstlane(table[pg.index(kb)]) : 0;
  }
}

// Where the two 16-key halves of a block start inside their page's part of one kv head: uniform values.
struct BlockPlace {
  size_t head[2];   // element offset of (page, kv head) in the keys' pool
  size_t vhead[2];  // and in the values' pool (the same unless values are narrower than keys)
  int off[2];       // first key inside the page
};

__device__ __forceinline__ BlockPlace place_of(const int* pages, int base, int g, int nkv, PageGeom pg, int D,
                                               int DV) {
  BlockPlace bp;
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    bp.head[u] = ((size_t)pages[u] * nkv + g) * pg.size * D;
    bp.vhead[u] = DV == D ? bp.head[u] : ((size_t)pages[u] * nkv + g) * pg.size * DV;
    bp.off[u] = pg.offset(base + u * 16);
  }
  return bp;
}

template <int D>
__device__ __forceinline__ void load_keys(KeyBlock<D>& b, const bf16* __restrict__ k_pages, const BlockPlace& bp,
                                          int lane) {
  const int k_lane = (lane & 15) * D + (lane >> 4) * 8;   // this lane's key and dims inside a 16-key half
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const bf16* kp = k_pages + bp.head[u] + bp.off[u] * D;
#pragma unroll
    for (int s = 0; s < D / 32; ++s) b.k[u][s] = *reinterpret_cast<const bf16x8*>(kp + k_lane + s * 32);
  }
}

template <int CT, bool NARROW>
__device__ __forceinline__ void load_values(ValueBlock<CT>& b, const bf16* __restrict__ vt_pages,
                                            const BlockPlace& bp, PageGeom pg, int dim0, int lane, int live) {
  const int v_lane = (dim0 + (lane & 15)) * pg.size + (lane >> 4) * 4;   // this lane's dim and keys inside a tile
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const bf16* vp = vt_pages + bp.vhead[u] + bp.off[u];
#pragma unroll
    for (int c = 0; c < CT; ++c)
      if (!NARROW || c < live) b.v[c][u] = *reinterpret_cast<const bf16x4*>((vp + c * 16 * pg.size) + v_lane);
  }
}

// Two waves of a wide tile on every SIMD (256 registers each) hide each other's waits; narrow tiles fit anyway.
//
// VS > 1 (narrow tiles only) shares one tile among VS blocks: each works out all scores and the whole softmax
// but only D / VS of the output's dims, so it reads all keys and 1 / VS of the values.  A compute unit draws
// its data at a small fraction of the chip's rate, so when a step has fewer tiles than the chip has units this
// shortens the longest chain without a second kernel; the blocks write disjoint dims and share nothing.
//
// EXTRA = CHANGED: the scores are changed on their way into the softmax: a scaled score x becomes cap * tanh(x / cap) (cap > 0),
// then slope * (the key's distance from the query) is taken off it, one slope per query head; at the end every head's
// result is multiplied by out_scale and by the sigmoid of a gate, one number per token and head or one per entry.  Such
// scores are kept in log2 units from the start, and the block's maxima are those of the changed scores.
// EXTRA = BOUNDED: as CHANGED with a cap of at most BOUNDED_CAP and no slopes.  Such scores lie in [-cap, cap], whose
// exponentials and their sums and products with values are well inside float's range, so the softmax needs no running
// maximum: the reference stays where it starts (0; for the wave that holds a positive sink, the sink).
constexpr int PLAIN = 0, CHANGED = 1, BOUNDED = 2;
constexpr float BOUNDED_CAP = 60.f;

struct AttnExtras {
  float scale;               // of the raw scores, natural units
  float cap;                 // 0: no cap
  float exp_arg;             // 2 log2(e) / cap: tanh(x / cap) = 1 - 2 / (2^(x exp_arg) + 1)
  const float* slopes;       // [nh] or null
  const bf16* gate;          // [N, >= nh * gate_width] or null
  size_t gate_stride;
  int gate_width;            // 1, or the value size
  float out_scale;
  int value_dim;             // the value size (NARROW variants: below the key size)
};

// The CHANGED variants need more registers than two wide tiles to a SIMD leave: a wide tile of theirs has the SIMD to
// itself, as has a BOUNDED one with narrow values at the largest head size.  Narrow tiles over sixteen waves (128 registers a lane) and the narrow tile of the largest
// head over eight have no such variant, nor have wide tiles over eight waves; the launcher picks a neighbour.
template <int D, int NT, int WAVES, int VS>
constexpr bool extra_variant() {
  return !(NT == 1 && WAVES == 16) && !(D == 128 && NT == 1 && WAVES == 8 && VS == 1) && !(NT > 1 && WAVES == 8);
}

// NARROW: values have fewer dims than keys (a multiple of 16); the tiles of 16 dims past them are neither read nor
// multiplied, which a branch that is the same for the whole launch decides.
template <int D, int NT, int WAVES, bool SPLIT, int VS, bool SINK, int EXTRA = PLAIN, bool NARROW = false>
__global__ void __launch_bounds__(WAVES * MS_WAVE, (NT > 1 && EXTRA != CHANGED && !(NARROW && D == 128) ? 2 : 1))
attention_mfma_kernel(const bf16* __restrict__ q, size_t q_stride, const bf16* __restrict__ k_pages,
                      const bf16* __restrict__ vt_pages, const int* __restrict__ block_table, int table_stride,
                      const int* __restrict__ table_rows, const int* __restrict__ q_start,
                      const int* __restrict__ context_lens, bf16* __restrict__ out, size_t out_stride,
                      float* __restrict__ part_o, float* __restrict__ part_ml, int nh, int nkv, int page_size,
                      int page_shift, float scale_log2e, int window, int min_blocks, int n_splits,
                      const float* __restrict__ sink, AttnExtras ex = AttnExtras()) {
  // SPLIT: min_blocks and n_splits say how a request's key blocks are spread.  Else min_blocks != 0 asks for
  // the order of tiles in which a long tile's companion on its CU is a short one (see below), and n_splits is
  // the number of requests whose tiles the grid's second dimension runs over (0: one tile to a request)
  __shared__ float sm_m[WAVES][NT][16], sm_l[WAVES][NT][16];
  static_assert(VS == 1 || (NT == 1 && !SPLIT), "only narrow tiles of the general shape share their dims out");
  static_assert((D / 16) % VS == 0, "whole tiles of 16 dims to a block");
  static_assert(!NARROW || (EXTRA && VS == 1), "narrow values come with the variants that change their scores");
  constexpr int CT = D / 16 / VS;
  const int DV = NARROW ? ex.value_dim : D;
  const int live = NARROW ? DV / 16 : CT;     // tiles of 16 value dims
  __shared__ f32x4 sm_o[WAVES > 1 ? WAVES - 1 : 1][CT][NT][MS_WAVE];
  const int lane = threadIdx.x & (MS_WAVE - 1);
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / MS_WAVE);   // the same for the whole wave
  const int col16 = lane & 15, kq = lane >> 4;
  // general shape: grid (kv heads, column tiles of the whole step, blocks that share a tile's dims): blocks are
  // handed out with the kv head running fastest; split shape: grid (splits, kv heads, requests)
  const int g = SPLIT ? blockIdx.y : blockIdx.x;
  const int bx = SPLIT ? blockIdx.x : blockIdx.z;
  const int rep = nh / nkv;
  const PageGeom pg = {page_size, page_shift};
  // Which request, and which of its tiles.  A request owns ceil(columns / tile width) tiles, requests in order,
  // so the launch needs to know only how many tokens and requests a step has, not how the tokens are dealt out
  // (a captured graph serves every mix).  The waves of a block find their place alike: a lane per request
  // works out its tiles, a prefix sum over the wave and a vote say where this block's tile falls.
  int r, rank, n_tiles;
  if (SPLIT) {
    r = blockIdx.z; rank = 0; n_tiles = 1;
  } else if (n_splits == 0) {
    r = blockIdx.y; rank = 0; n_tiles = 1;
  } else if (n_splits == 1) {
    r = 0; rank = blockIdx.y;
    n_tiles = ((q_start[1] - q_start[0]) * rep + 16 * NT - 1) / (16 * NT);
    if (rank >= n_tiles) return;
  } else {
    const int flat = blockIdx.y;
    int before = 0;
    r = -1; rank = 0; n_tiles = 0;
    for (int base = 0; base < n_splits; base += MS_WAVE) {
      const int i = base + lane;
      int mine = 0;
      if (i < n_splits) mine = ((q_start[i + 1] - q_start[i]) * rep + 16 * NT - 1) / (16 * NT);
      int upto = mine;   // tiles of the requests base..i
#pragma unroll
      for (int o = 1; o < MS_WAVE; o <<= 1) {
        const int v = __shfl_up(upto, o, MS_WAVE);
        if (lane >= o) upto += v;
      }
      const unsigned long long hit = __builtin_amdgcn_ballot_w64(flat < before + upto);
      if (hit) {
        const int first = __builtin_ctzll(hit);
        r = base + first;
        n_tiles = __shfl(mine, first, MS_WAVE);
        rank = flat - before - (__shfl(upto, first, MS_WAVE) - n_tiles);
        break;
      }
      before += __shfl(upto, MS_WAVE - 1, MS_WAVE);
    }
    if (r < 0) return;   // the grid has room for a partial tile of every request; this block is surplus
    r = __builtin_amdgcn_readfirstlane(r);
    rank = __builtin_amdgcn_readfirstlane(rank);
    n_tiles = __builtin_amdgcn_readfirstlane(n_tiles);
  }
  const int row = table_rows ? table_rows[r] : r;
  const int* table = block_table + (size_t)row * table_stride;
  // Without a window a wave's first key block is known before the request's lengths are: ask for its page
  // ids at once, so that they travel together with the lengths instead of after them.
  int first_pages[2] = {0, 0};
  const bool early = !SPLIT && window <= 0;
  if (early) {
#pragma unroll
    for (int u = 0; u < 2; ++u)
      first_pages[u] = __builtin_amdgcn_readfirstlane(table[min(pg.index(wave * 32 + u * 16), table_stride - 1)]);
  }
  const int q0 = q_start[r];
  const int qlen = q_start[r + 1] - q0;
  const int start_pos = context_lens[r] - qlen;
  const int ncols = qlen * rep;
  // Late tiles of a prompt see the most keys: they go first, so that the long ones do not finish last.  When
  // all blocks fit on the chip at once (two to a CU), only the later half goes first, latest tile first, and
  // then the earlier half, earliest first: blocks that start one round of the chip apart tend to share a CU, and
  // so a long tile's companion is a short one that soon leaves the SIMDs to it (2,048 tokens: 34.0 -> 29.4 us).
  const int dim0 = VS > 1 ? bx * CT * 16 : 0;   // the first of this block's output dims
  const int half = (!SPLIT && min_blocks) ? (n_tiles + 1) / 2 : n_tiles;
  const int tile = rank < half ? n_tiles - 1 - rank : rank - half;
  const int c0 = SPLIT ? 0 : tile * 16 * NT;
  if (c0 >= ncols) return;

  // key range of the tile: from the first column's window start to the last column's own position
  const int last_col = min(ncols, c0 + 16 * NT) - 1;
  int key_hi = start_pos + last_col / rep;
  int key_lo = 0;
  if (window > 0) key_lo = max(0, start_pos + c0 / rep - window + 1);
  int blk_begin = key_lo / 32, blk_end = key_hi / 32 + 1;
  // a block whose keys every column of the tile sees needs no mask: all keys at or before the first column's
  // position (and, with a window, after the last column's window start); tiles with idle columns always mask
  const int first_pos = start_pos + c0 / rep;
  const bool full_tile = c0 + 16 * NT <= ncols;
  if (SPLIT) {
    // every request spreads its own key blocks evenly over the splits (at least min_blocks each)
    const int per = max(min_blocks, (blk_end - blk_begin + n_splits - 1) / n_splits);
    blk_begin += bx * per;
    blk_end = min(blk_end, blk_begin + per);
    if (blk_begin >= blk_end) return;
  }

  // this lane's columns
  int pos[NT];   // -1: an idle column (sees no key; its result is not written)
  float slope[EXTRA == CHANGED ? NT : 1];
  const float sl2 = EXTRA ? 1.0f : scale_log2e;   // what turns a kept score into log2 units
  // the fields the loop reads, as scalars of their own (the struct itself stays in the kernel's arguments)
  const float ex_scale = ex.scale, ex_cap = ex.cap, ex_arg = ex.exp_arg;
  const float* const ex_slopes = ex.slopes;
  const float raw_arg = ex.scale * ex.exp_arg, cap2 = ex.cap * 1.4426950408889634f;     // BOUNDED: log2 units
  bf16x8 qv[NT][D / 32];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int c = c0 + t * 16 + col16;
    const int cc = min(c, ncols - 1);
    const int tok = q0 + cc / rep, head = g * rep + cc % rep;
    pos[t] = c < ncols ? start_pos + cc / rep : -1;
    if (EXTRA == CHANGED) slope[t] = ex_slopes ? ex_slopes[head] : 0.f;
    const bf16* qp = q + (size_t)tok * q_stride + (size_t)head * D + kq * 8;
#pragma unroll
    for (int s = 0; s < D / 32; ++s) qv[t][s] = *reinterpret_cast<const bf16x8*>(qp + s * 32);
  }

  // The sums of the exponentials come from the matrix cores too: one more product per column tile, of P^T with
  // a V^T of ones, gives every lane its columns' sums over all 32 keys of the block (of the same bfloat16 values
  // that the weighted sum of the values uses), where adding them up lane by lane took 32 additions and, at the
  // end, two exchanges between lanes; the matrix pipe has the time.
  // (The widest tile at head size 64 has no registers left for it and adds its exponentials up on the vector
  // pipe, a lane's share at a time, with two exchanges between lanes at the end.)
  constexpr bool SUMS_BY_MATRIX = !(D == 64 && NT == 4);
  float m[NT], lvec[NT];
  f32x4 o[CT][NT], lsum[SUMS_BY_MATRIX ? NT : 1];
  bf16x8 ones;
#pragma unroll
  for (int i = 0; i < 8; ++i) ones[i] = (__bf16)1.0f;
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    m[t] = EXTRA == BOUNDED ? 0.f : -INFINITY;
    lvec[t] = 0.f;
    if (SUMS_BY_MATRIX) lsum[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < CT; ++c) o[c][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  // A sink is one more term of the denominator with no key and no value: the running softmax of one wave (the first
  // wave of the block, of the first split) starts as if it had already seen a key with that score, unscaled, and a
  // value of zero.  Everything after (moving the reference, merging waves and splits) treats it as any other term.
  if (SINK && sink && wave == 0 && (!SPLIT || bx == 0)) {
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int cc = min(c0 + t * 16 + col16, ncols - 1);
      m[t] = sink[g * rep + cc % rep] * 1.4426950408889634f;
      float one = 1.0f;
      if (EXTRA == BOUNDED) { one = fast_exp2(fminf(m[t], 0.f)); m[t] = fmaxf(m[t], 0.f); }
      lvec[t] = kq == 0 ? one : 0.f;
      if (SUMS_BY_MATRIX) lsum[t] = f32x4{one, one, one, one};
    }
  }

  // A narrow tile (decode) has registers to spare and few waves to hide a wait behind: it fetches the next
  // block's values early, together with its keys.  A wide tile fetches values at the top of the pass that
  // uses them (the score products and the softmax run meanwhile, and so does the SIMD's other wave).
  constexpr bool VALUES_EARLY = NT == 1 && !EXTRA;   // (changed scores need the registers)
  KeyBlock<D> buf_k[2];
  ValueBlock<CT> buf_v[2];
  BlockPlace buf_at[2];
  if (blk_begin + wave < blk_end) {
    KeyBlock<D>& cur_k = buf_k[0];
    ValueBlock<CT>& cur_v = buf_v[0];
    BlockPlace& cur_at = buf_at[0];
    const int base = (blk_begin + wave) * 32;
    int pages[2];
    if (early) {  // blk_begin is 0 here; halves past the last key fall back to the null page
#pragma unroll
      for (int u = 0; u < 2; ++u) pages[u] = base + u * 16 <= key_hi ? first_pages[u] : 0;
    } else {
      pages_of(table, base, key_hi, pg, pages);
    }
    cur_at = place_of(pages, base, g, nkv, pg, D, DV);
    load_keys<D>(cur_k, k_pages, cur_at, lane);
    if (VALUES_EARLY) load_values<CT, NARROW>(cur_v, vt_pages, cur_at, pg, dim0, lane, live);
  }
  // The page ids of a block are asked for one block before its keys are: the keys' loads then go out at the top of
  // an iteration instead of behind a table lookup (8,192 tokens of the 0.5B shape: 235 -> 232 us; 2,048 tokens at
  // head size 128: 99.9 -> 96.7 us).  (Keeping the loads of two blocks in flight for narrow tiles was measured and
  // dropped: a decode tile's time is what its CU can draw, 102 KB at about 43 GB/s at 640 keys, not its waits.)
  int ahead_pages[2] = {0, 0};
  if (blk_begin + wave + WAVES < blk_end) pages_of(table, (blk_begin + wave + WAVES) * 32, key_hi, pg, ahead_pages);
  // One block of 32 keys: the step works on the buffers it is handed as current and fills those it is handed
  // as next; the loop below calls it with the two sets of buffers in turn, so nothing is copied between them.
  auto step = [&](int blk, KeyBlock<D>& cur_k, ValueBlock<CT>& cur_v, BlockPlace& cur_at, KeyBlock<D>& nxt_k,
                  ValueBlock<CT>& nxt_v, BlockPlace& nxt_at) __attribute__((always_inline)) {
    const int base = blk * 32;
    if (!VALUES_EARLY) load_values<CT, NARROW>(cur_v, vt_pages, cur_at, pg, dim0, lane, live);
    if (blk + WAVES < blk_end) {
      nxt_at = place_of(ahead_pages, base + WAVES * 32, g, nkv, pg, D, DV);
      load_keys<D>(nxt_k, k_pages, nxt_at, lane);
      if (VALUES_EARLY) load_values<CT, NARROW>(nxt_v, vt_pages, nxt_at, pg, dim0, lane, live);
      if (blk + 2 * WAVES < blk_end) pages_of(table, base + 2 * WAVES * 32, key_hi, pg, ahead_pages);
    }

    // scores: s[u][t] holds keys base + u*16 + kq*4 + (0..3) of column t*16 + col16
    f32x4 s[2][NT];
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < D / 32; ++ks) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(cur_k.k[u][ks], qv[t][ks], acc, 0, 0, 0);
        s[u][t] = acc;
      }

    if (EXTRA == CHANGED) {
      // slope * (pos - key) = slope * (pos - base - 4 kq) - slope * (16 u + i): one product per column, then constants
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const float off = -slope[t] * (float)(pos[t] - base - kq * 4);
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            float x = s[u][t][i] * ex_scale;
            if (ex_cap > 0.f) x = fmaf(-2.0f * ex_cap, __builtin_amdgcn_rcpf(fast_exp2(x * ex_arg) + 1.0f), ex_cap);
            s[u][t][i] = (x + fmaf(slope[t], (float)(u * 16 + i), off)) * 1.4426950408889634f;
          }
      }
    }

    // values past the last visible key may be anything a reused page still holds: make them zero
    if (base + 31 > key_hi) {
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (base + u * 16 + kq * 4 + i > key_hi) {
#pragma unroll
            for (int c = 0; c < CT; ++c)
              if (!NARROW || c < live) cur_v.v[c][u][i] = (__bf16)0.0f;
          }
    }

    const bool unmasked = full_tile && base + 31 <= first_pos && (window <= 0 || base > key_hi - window);
    bf16x8 p[NT];
    float m_safe[NT];
    if constexpr (EXTRA != BOUNDED) {
      float corr[NT], bmax[NT];
      bool moved = false;
      // the block's maxima of the raw scores (the scale is positive, so they are the maxima of the scaled ones
      // too); one branch for the whole tile, so that what follows is straight-line code for all its columns
      if (unmasked) {
#pragma unroll
        for (int t = 0; t < NT; ++t) {
          float bm = -INFINITY;
#pragma unroll
          for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int i = 0; i < 4; ++i) bm = fmaxf(bm, s[u][t][i]);
          bmax[t] = bm;
        }
      } else {
#pragma unroll
        for (int t = 0; t < NT; ++t) {
          float bm = -INFINITY;
#pragma unroll
          for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              const int key = base + u * 16 + kq * 4 + i;
              const bool see = key <= pos[t] && (window <= 0 || key > pos[t] - window);
              const float v = see ? s[u][t][i] : -INFINITY;
              s[u][t][i] = v;
              bm = fmaxf(bm, v);
            }
          bmax[t] = bm;
        }
      }
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        float bm = bmax[t];
        bm = fmaxf(bm, __shfl_xor(bm, 16, MS_WAVE));
        bm = fmaxf(bm, __shfl_xor(bm, 32, MS_WAVE));
        bm *= sl2;
        // m is the reference that the exponents are taken against, not necessarily the maximum: it follows the
        // maximum only when that has run ahead by more than REF_SLACK (a factor 2^REF_SLACK in the terms, far
        // inside float's range), so that the accumulators are rescaled rarely.  Any reference gives the same
        // softmax; all lanes of a column decide alike because bm is the same in all of them.
        const bool step = bm > m[t] + REF_SLACK;
        const float m_new = step ? bm : m[t];
        corr[t] = step ? fast_exp2(m[t] - m_new) : 1.0f;   // m = -inf: 0
        moved |= step;
        m[t] = m_new;
        m_safe[t] = m_new == -INFINITY ? 0.f : m_new;
      }
      if (NT == 1 || __builtin_amdgcn_ballot_w64(moved) != 0) {   // the same branch for the whole wave
#pragma unroll
        for (int t = 0; t < NT; ++t) {
          if (SUMS_BY_MATRIX) lsum[t] *= corr[t]; else lvec[t] *= corr[t];
#pragma unroll
          for (int c = 0; c < CT; ++c) o[c][t] *= corr[t];
        }
      }
    }
    // column by column, so that the products of one column run on the matrix cores while the next column's
    // exponentials are taken
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      if (EXTRA == BOUNDED) {     // cap tanh(x / cap) = cap - 2 cap / (2^(x arg) + 1)
        const float top = cap2 - m[t];
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
          for (int i = 0; i < 4; ++i)
            s[u][t][i] = fmaf(-2.0f * cap2, __builtin_amdgcn_rcpf(fast_exp2(s[u][t][i] * raw_arg) + 1.0f), top);
        if (!unmasked) {
#pragma unroll
          for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
              const int key = base + u * 16 + kq * 4 + i;
              if (key > pos[t] || (window > 0 && key <= pos[t] - window)) s[u][t][i] = -INFINITY;
            }
        }
      }
#pragma unroll
      for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float e = EXTRA == BOUNDED ? fast_exp2(s[u][t][i]) : fast_exp2(fmaf(s[u][t][i], sl2, -m_safe[t]));
          if (!SUMS_BY_MATRIX) lvec[t] += e;
          p[t][u * 4 + i] = (__bf16)e;
        }
      if (SUMS_BY_MATRIX) lsum[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, p[t], lsum[t], 0, 0, 0);
#pragma unroll
      for (int c = 0; c < CT; ++c) {
        if (NARROW && c >= live) break;
        bf16x8 vv;
#pragma unroll
        for (int i = 0; i < 4; ++i) { vv[i] = cur_v.v[c][0][i]; vv[4 + i] = cur_v.v[c][1][i]; }
        o[c][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv, p[t], o[c][t], 0, 0, 0);
      }
    }
  };
  for (int blk = blk_begin + wave; blk < blk_end; blk += 2 * WAVES) {
    step(blk, buf_k[0], buf_v[0], buf_at[0], buf_k[1], buf_v[1], buf_at[1]);
    if (blk + WAVES < blk_end) step(blk + WAVES, buf_k[1], buf_v[1], buf_at[1], buf_k[0], buf_v[0], buf_at[0]);
  }

  float l[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    if (SUMS_BY_MATRIX) {
      l[t] = lsum[t][0];   // every row of the product of ones is the column's sum
    } else {               // a column's sum is spread over the four lane groups
      l[t] = lvec[t] + __shfl_xor(lvec[t], 16, MS_WAVE);
      l[t] += __shfl_xor(l[t], 32, MS_WAVE);
    }
  }
  // The variants that change their scores share the end out: each wave merges, gates and writes a part of the dims.
  constexpr bool SHARED_END = EXTRA != PLAIN && WAVES > 1 && CT % WAVES == 0;
  if constexpr (SHARED_END) {
    constexpr int OWN = CT / WAVES;
    const bool by_entry = !SPLIT && ex.gate && ex.gate_width != 1;
    bf16x4 gv[NT][OWN];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      if (kq == 0) { sm_m[wave][t][col16] = m[t]; sm_l[wave][t][col16] = l[t]; }
#pragma unroll
      for (int c = 0; c < CT; ++c)
        if (c / OWN != wave) sm_o[wave < c / OWN ? wave : wave - 1][c][t][lane] = o[c][t];
      if (by_entry && pos[t] >= 0) {      // the gate's numbers are on their way while the waves wait for each other
        const int c = c0 + t * 16 + col16;
        const bf16* gp = ex.gate + (size_t)(q0 + c / rep) * ex.gate_stride + (size_t)(g * rep + c % rep) * DV + dim0 + kq * 4;
#pragma unroll
        for (int j = 0; j < OWN; ++j)
          if (!NARROW || wave * OWN + j < live) gv[t][j] = *reinterpret_cast<const bf16x4*>(gp + (wave * OWN + j) * 16);
      }
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      float big = -INFINITY, den = 0.f, f[WAVES];
#pragma unroll
      for (int w = 0; w < WAVES; ++w) { f[w] = sm_m[w][t][col16]; big = fmaxf(big, f[w]); }
      const float safe = big == -INFINITY ? 0.f : big;
#pragma unroll
      for (int w = 0; w < WAVES; ++w) { f[w] = fast_exp2(f[w] - safe); den = fmaf(f[w], sm_l[w][t][col16], den); }
      if (pos[t] < 0) continue;
      const int col = c0 + t * 16 + col16;
      const int tok = q0 + col / rep, head = g * rep + col % rep;
      const size_t slot = SPLIT ? ((size_t)r * nh + head) * n_splits + bx : 0;
      float inv = 1.0f;
      if (SPLIT) {
        if (kq == 0 && wave == 0) { part_ml[slot * 2] = big; part_ml[slot * 2 + 1] = den; }
      } else {
        inv = ex.out_scale / den;
        if (ex.gate && !by_entry) inv *= fast_sigmoid(__bfloat162float(ex.gate[(size_t)tok * ex.gate_stride + head]));
      }
#pragma unroll
      for (int c = 0; c < CT; ++c) {
        if (c / OWN != wave || (NARROW && c >= live)) continue;
        f32x4 sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < WAVES; ++w)
          sum += (w == c / OWN ? o[c][t] : sm_o[w < c / OWN ? w : w - 1][c][t][lane]) * f[w];
        if (SPLIT) {
          *reinterpret_cast<f32x4*>(part_o + slot * DV + kq * 4 + c * 16) = sum;
        } else {
          bf16x4 w4;
#pragma unroll
          for (int i = 0; i < 4; ++i)
            w4[i] = (__bf16)(by_entry ? sum[i] * inv * fast_sigmoid((float)gv[t][c % OWN][i]) : sum[i] * inv);
          *reinterpret_cast<bf16x4*>(out + (size_t)tok * out_stride + (size_t)head * DV + dim0 + kq * 4 + c * 16) = w4;
        }
      }
    }
    return;
  }
  if (WAVES > 1) {
    // merge the waves' partial results (each relative to its own maximum) in wave order
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      if (kq == 0) { sm_m[wave][t][col16] = m[t]; sm_l[wave][t][col16] = l[t]; }
      if (wave > 0) {
#pragma unroll
        for (int c = 0; c < CT; ++c) sm_o[wave - 1][c][t][lane] = o[c][t];
      }
    }
    __syncthreads();
    if (wave > 0) return;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      float big = m[t];
      for (int w = 1; w < WAVES; ++w) big = fmaxf(big, sm_m[w][t][col16]);
      const float safe = big == -INFINITY ? 0.f : big;
      const float f0 = fast_exp2(m[t] - safe);
      float lsum = l[t] * f0;
#pragma unroll
      for (int c = 0; c < CT; ++c) o[c][t] *= f0;
      for (int w = 1; w < WAVES; ++w) {
        const float f = fast_exp2(sm_m[w][t][col16] - safe);
        lsum += f * sm_l[w][t][col16];
#pragma unroll
        for (int c = 0; c < CT; ++c) o[c][t] += sm_o[w - 1][c][t][lane] * f;
      }
      m[t] = big;
      l[t] = lsum;
    }
  }

#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const float lt = l[t];
    if (pos[t] < 0) continue;
    const int c = c0 + t * 16 + col16;   // worked out again rather than kept through the loop
    const int tok = q0 + c / rep, head = g * rep + c % rep;
    if (SPLIT) {
      // unnormalised: O, the running maximum (log2 units) and the sum; the combine kernel weighs the splits
      const size_t slot = ((size_t)r * nh + head) * n_splits + bx;
      float* po = part_o + slot * DV + kq * 4;
#pragma unroll
      for (int c = 0; c < CT; ++c)
        if (!NARROW || c < live) *reinterpret_cast<f32x4*>(po + c * 16) = o[c][t];
      if (kq == 0) { part_ml[slot * 2] = m[t]; part_ml[slot * 2 + 1] = lt; }
    } else {
      float inv = 1.0f / lt;
      if (EXTRA) {
        inv *= ex.out_scale;
        if (ex.gate && ex.gate_width == 1)
          inv *= fast_sigmoid(__bfloat162float(ex.gate[(size_t)tok * ex.gate_stride + head]));
      }
      const bool by_entry = EXTRA && ex.gate && ex.gate_width != 1;
      const bf16* gp = by_entry ? ex.gate + (size_t)tok * ex.gate_stride + (size_t)head * DV + dim0 + kq * 4 : nullptr;
      bf16* op = out + (size_t)tok * out_stride + (size_t)head * DV + dim0 + kq * 4;
#pragma unroll
      for (int c = 0; c < CT; ++c) {
        if (NARROW && c >= live) break;
        bf16x4 w;
#pragma unroll
        for (int i = 0; i < 4; ++i) w[i] = (__bf16)(o[c][t][i] * inv);
        if (by_entry) {
          const bf16x4 gv = *reinterpret_cast<const bf16x4*>(gp + c * 16);
#pragma unroll
          for (int i = 0; i < 4; ++i) w[i] = (__bf16)(o[c][t][i] * inv * fast_sigmoid((float)gv[i]));
        }
        *reinterpret_cast<bf16x4*>(op + c * 16) = w;
      }
    }
  }
}

// out[r, h, :] = sum_s 2^(m_s - M) O_s / sum_s 2^(m_s - M) l_s over the splits that request r used.
// One block per (request, head): the splits' maxima and sums are fetched side by side, the
// weights are worked out once into LDS, then a thread per dim adds the weighted partial results in split order.
constexpr int COMBINE_MAX_SPLITS = 128;

template <int D>
__global__ void __launch_bounds__(D < 64 ? 64 : D)
attention_combine_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml,
                         const int* __restrict__ q_start, const int* __restrict__ context_lens,
                         bf16* __restrict__ out, size_t out_stride, int nh, int dv, int window, int min_blocks,
                         int n_splits, const bf16* __restrict__ gate, size_t gate_stride, int gate_width, float out_scale) {
  __shared__ float sm_m[COMBINE_MAX_SPLITS], sm_w[COMBINE_MAX_SPLITS];
  const int r = blockIdx.x / nh, h = blockIdx.x % nh;
  if (q_start[r + 1] == q_start[r]) return;   // a row that pads a captured batch: no token, nothing to write
  const int key_hi = context_lens[r] - 1;
  const int key_lo = window > 0 ? max(0, key_hi - window + 1) : 0;
  const int blocks = key_hi / 32 + 1 - key_lo / 32;
  const int per = max(min_blocks, (blocks + n_splits - 1) / n_splits);
  const int used = (blocks + per - 1) / per;
  const size_t slot0 = ((size_t)r * nh + h) * n_splits;
  const int t = threadIdx.x;
  for (int s = t; s < used; s += blockDim.x) sm_m[s] = part_ml[(slot0 + s) * 2];
  __syncthreads();
  float big = -INFINITY;
  for (int s = 0; s < used; ++s) big = fmaxf(big, sm_m[s]);
  __syncthreads();
  // the weights, and in sm_m (no longer needed) the splits' weighted sums for the denominator in split order
  for (int s = t; s < used; s += blockDim.x) {
    const float w = fast_exp2(sm_m[s] - big);
    sm_w[s] = w;
    sm_m[s] = w * part_ml[(slot0 + s) * 2 + 1];
  }
  __syncthreads();
  float den = 0.f;
  for (int s = 0; s < used; ++s) den += sm_m[s];
  float inv = out_scale / den;
  const bf16* gp = gate ? gate + (size_t)q_start[r] * gate_stride + (size_t)h * gate_width : nullptr;
  if (gate && gate_width == 1) inv *= 1.0f / (1.0f + expf(-__bfloat162float(*gp)));
  bf16* op = out + (size_t)q_start[r] * out_stride + (size_t)h * dv;
  for (int d = t; d < dv; d += blockDim.x) {
    float acc = 0.f;
#pragma unroll 8
    for (int s = 0; s < used; ++s) acc += sm_w[s] * part_o[(slot0 + s) * dv + d];
    acc *= inv;
    if (gate && gate_width != 1) acc /= 1.0f + expf(-__bfloat162float(gp[d]));
    op[d] = __float2bfloat16(acc);
  }
}

int g_force_nt = 0, g_force_waves = 0, g_force_vs = 0;

inline int page_shift_of(int page_size) {   // log2 of a power of two, else -1
  if (page_size & (page_size - 1)) return -1;
  int sh = 0;
  while ((1 << sh) < page_size) ++sh;
  return sh;
}

inline bool bounded_scores(const AttnExtras& ex) { return ex.cap > 0.f && ex.cap <= BOUNDED_CAP && ex.slopes == nullptr; }

template <int D, int NT, int WAVES, int VS>
int launch_general(const bf16* q, size_t q_stride, const bf16* k, const bf16* vt, const int* table, int table_stride,
                   const int* table_rows, const int* q_start, const int* ctx, bf16* out, size_t out_stride,
                   int n_requests, int n_tokens, int max_q_len, int nh, int nkv, int page_size, float scale,
                   int window, const float* sink, const AttnExtras* extras, hipStream_t stream) {
  const int rep = nh / nkv;
  const long long per_request = ((long long)max_q_len * rep + 16 * NT - 1) / (16 * NT);
  // every request may end in a partial tile; no step has more tiles than if each request were the longest
  long long tiles = (long long)n_tokens * rep / (16 * NT) + n_requests;
  if (tiles > per_request * n_requests) tiles = per_request * n_requests;
  if (tiles > 65535) return MS_UNSUPPORTED;   // grid.y
  const int pair_order = tiles * VS * nkv <= 2LL * ms_compute_units() ? 1 : 0;
  const int scan = per_request == 1 ? 0 : n_requests;   // one tile to a request: the tile's index is the request's
  dim3 grid(nkv, (unsigned)tiles, VS), block(WAVES * MS_WAVE);
  if constexpr (D == 64 && NT == 4) {     // no variant with a sink or changed scores at this shape (its registers are spent)
    if (sink || extras) return MS_UNSUPPORTED;
  } else if (extras) {
    const bool bounded = bounded_scores(*extras);
    if constexpr (!extra_variant<D, NT, WAVES, VS>()) {
      return MS_UNSUPPORTED;
    } else {
#define LAUNCH_EXTRA(EX, NARROW) attention_mfma_kernel<D, NT, WAVES, false, VS, true, EX, NARROW><<<grid, block, 0, stream>>>(q, q_stride, k, vt, table, table_stride, table_rows, q_start, ctx, out, out_stride, nullptr, nullptr, nh, nkv, page_size, page_shift_of(page_size), scale * 1.4426950408889634f, window, pair_order, scan, sink, *extras)
      if (extras->value_dim != D) {
        if constexpr (VS == 1) {
          if (bounded) LAUNCH_EXTRA(BOUNDED, true); else LAUNCH_EXTRA(CHANGED, true);
        } else {
          return MS_UNSUPPORTED;
        }
      } else {
        if (bounded) LAUNCH_EXTRA(BOUNDED, false); else LAUNCH_EXTRA(CHANGED, false);
      }
#undef LAUNCH_EXTRA
      return ms_launch_status();
    }
  } else if (sink) {
    attention_mfma_kernel<D, NT, WAVES, false, VS, true><<<grid, block, 0, stream>>>(q, q_stride, k, vt, table, table_stride, table_rows, q_start, ctx, out, out_stride, nullptr, nullptr, nh, nkv, page_size, page_shift_of(page_size), scale * 1.4426950408889634f, window, pair_order, scan, sink);
    return ms_launch_status();
  }
  attention_mfma_kernel<D, NT, WAVES, false, VS, false><<<grid, block, 0, stream>>>(q, q_stride, k, vt, table, table_stride, table_rows, q_start, ctx, out, out_stride, nullptr, nullptr, nh, nkv, page_size, page_shift_of(page_size), scale * 1.4426950408889634f, window, pair_order, scan, nullptr);
  return ms_launch_status();
}

template <int D>
int launch_split(const bf16* q, size_t q_stride, const bf16* k, const bf16* vt, const int* table, int table_stride,
                 const int* table_rows, const int* q_start, const int* ctx, bf16* out, size_t out_stride, float* part_o, float* part_ml,
                 int n_requests, int nh, int nkv, int page_size, float scale, int window, int min_blocks,
                 int n_splits, const float* sink, const AttnExtras* extras, hipStream_t stream) {
  dim3 grid(n_splits, nkv, n_requests), block(4 * MS_WAVE);
#define LAUNCH_EXTRA(EX, NARROW) attention_mfma_kernel<D, 1, 4, true, 1, true, EX, NARROW><<<grid, block, 0, stream>>>(q, q_stride, k, vt, table, table_stride, table_rows, q_start, ctx, out, out_stride, part_o, part_ml, nh, nkv, page_size, page_shift_of(page_size), scale * 1.4426950408889634f, window, min_blocks, n_splits, sink, *extras)
  if (extras && extras->value_dim != D) {
    if (bounded_scores(*extras)) LAUNCH_EXTRA(BOUNDED, true); else LAUNCH_EXTRA(CHANGED, true);
  } else if (extras) {
    if (bounded_scores(*extras)) LAUNCH_EXTRA(BOUNDED, false); else LAUNCH_EXTRA(CHANGED, false);
  }
#undef LAUNCH_EXTRA
  else if (sink)
    attention_mfma_kernel<D, 1, 4, true, 1, true><<<grid, block, 0, stream>>>(q, q_stride, k, vt, table, table_stride, table_rows, q_start, ctx, out, out_stride, part_o, part_ml, nh, nkv, page_size, page_shift_of(page_size), scale * 1.4426950408889634f, window, min_blocks, n_splits, sink);
  else
    attention_mfma_kernel<D, 1, 4, true, 1, false><<<grid, block, 0, stream>>>(q, q_stride, k, vt, table, table_stride, table_rows, q_start, ctx, out, out_stride, part_o, part_ml, nh, nkv, page_size, page_shift_of(page_size), scale * 1.4426950408889634f, window, min_blocks, n_splits, nullptr);
  attention_combine_kernel<D><<<dim3(n_requests * nh), dim3(D < 64 ? 64 : D), 0, stream>>>(part_o, part_ml, q_start, ctx, out, out_stride, nh, extras ? extras->value_dim : D, window, min_blocks, n_splits, extras ? extras->gate : nullptr, extras ? extras->gate_stride : 0, extras ? extras->gate_width : 1, extras ? extras->out_scale : 1.0f);
  return ms_launch_status();
}

}  // namespace

// Tuning knob: force the general shape's tile width (16 * nt columns), waves per tile and (narrow tiles) the
// number of blocks that share a tile's dims; 0 restores the choice by size.  Shapes outside the menu are
// refused at the call.
extern "C" void ms_attention_mfma_force(int nt, int waves, int dim_shares) {
  g_force_nt = nt;
  g_force_waves = waves;
  g_force_vs = dim_shares;
}

// Whether the matrix-core kernels take this geometry (else the caller uses the generic kernel).
// value_dim: the key size, or a smaller multiple of 16.
extern "C" int ms_attention_mfma_supported(int head_dim, int value_dim, int page_size) {
  return (head_dim == 32 || head_dim == 64 || head_dim == 128) && page_size > 0 && page_size % 16 == 0 &&
         value_dim > 0 && value_dim <= head_dim && value_dim % 16 == 0;
}

// A gate of one number per entry is read four entries at a time.
static bool gate_fits(const void* gate, long long gate_stride, int gate_width, int value_dim) {
  if (gate == nullptr || gate_width == 1) return true;
  return gate_width == value_dim && gate_stride % 4 == 0 && (uintptr_t)gate % 8 == 0;
}

// General shape.  q [N, >= nh*d] bfloat16 (row stride q_stride), k_pages [P, nkv, page_size, d],
// vt_pages [P, nkv, value_dim, page_size], block_table int32 [rows, table_stride], table_rows int32 [R] (the table's row
// of each request; null: request r has row r), q_start int32 [R + 1], context_lens int32 [R] (keys held after
// this step), out [N, nh*value_dim] (row stride out_stride).  n_tokens = q_start[R] or more, max_q_len the longest
// portion or more: the launch is sized by these two and n_requests alone, so tokens beyond q_start[R] and
// requests without tokens cost a block that leaves at once.
extern "C" int ms_paged_attention_mfma(const void* q, long long q_stride, const void* k_pages, const void* vt_pages,
                                       const int* block_table, int table_stride, const int* table_rows,
                                       const int* q_start, const int* context_lens, void* out, long long out_stride,
                                       int n_requests, int n_tokens, int max_q_len, int num_heads, int num_kv_heads,
                                       int head_dim, int value_dim, int page_size, float scale, int window, const float* sink,
                                       float softcap, const float* slopes, const void* gate, long long gate_stride,
                                       int gate_width, float out_scale, hipStream_t stream) {
  if (n_requests <= 0 || max_q_len <= 0 || n_tokens <= 0) return MS_OK;
  if (num_heads <= 0 || num_kv_heads <= 0 || num_heads % num_kv_heads || table_stride <= 0) return MS_BAD_ARG;
  if (!(scale > 0.f)) return MS_BAD_ARG;   // maxima are taken of the raw scores
  if (!ms_attention_mfma_supported(head_dim, value_dim, page_size)) return MS_UNSUPPORTED;
  if (!gate_fits(gate, gate_stride, gate_width, value_dim)) return MS_UNSUPPORTED;
  if (q_stride % 8 || out_stride % 4 || ((uintptr_t)q % 16) || ((uintptr_t)out % 8)) return MS_UNSUPPORTED;
  if (n_requests > 65535 || num_kv_heads > 65535) return MS_UNSUPPORTED;
  const bool changed = softcap > 0.f || slopes != nullptr || gate != nullptr || out_scale != 1.0f || value_dim != head_dim;
  const AttnExtras ex = {scale, softcap > 0.f ? softcap : 0.f, softcap > 0.f ? 2.0f * 1.4426950408889634f / softcap : 0.f,
                         slopes, (const bf16*)gate, (size_t)gate_stride, gate_width, out_scale, value_dim};
  const AttnExtras* extras = changed ? &ex : nullptr;
#define GO(D, NT, WV, VS) return launch_general<D, NT, WV, VS>((const bf16*)q, q_stride, (const bf16*)k_pages, (const bf16*)vt_pages, block_table, table_stride, table_rows, q_start, context_lens, (bf16*)out, out_stride, n_requests, n_tokens, max_q_len, num_heads, num_kv_heads, page_size, scale, window, sink, extras, stream)
  // Tile width (NT * 16 columns) and waves over a tile's keys.  Few columns (a decode step): one narrow tile
  // per request and many waves over its keys.
  const int cols = max_q_len * (num_heads / num_kv_heads);
  int nt = cols > 16 ? (head_dim == 128 ? 2 : 4) : 1;
  int waves = nt > 1 ? 4 : (head_dim == 128 ? 8 : 16);
  // narrow tiles, fewer of them than compute units: blocks share a tile's dims as far as there is a unit for
  // every block (measured at 200, 640 and 1,000 keys, head sizes 64 and 128: up to 64 tiles four ways, up to 128
  // two ways, e.g. 128 tiles at 640 keys 8.0 -> 7.0 us; with more blocks than units the keys' repeated reading
  // costs more than the shorter streams save).  Very many tiles of the large head size: four waves to a tile
  // (512 tiles at 640 keys: 32.2 -> 29.3 us).
  int vs = 1;
  if (nt == 1) {
    const long long per_request = (cols + 15) / 16;
    const long long tiles = num_kv_heads * std::min(per_request * n_requests, (long long)n_tokens * (num_heads / num_kv_heads) / 16 + n_requests);
    const int cus = ms_compute_units();
    while (vs < 4 && (head_dim / 16) % (vs * 2) == 0 && tiles * vs * 2 <= cus) vs *= 2;
    if (head_dim == 128 && tiles >= 2LL * cus) waves = 4;
  }
  // with a sink the widest tile at head size 64 has no register left for the softmax's other starting point
  if ((sink != nullptr || changed) && head_dim == 64 && nt == 4) nt = 2;
  if (changed && nt == 1) {     // the variants with changed scores: eight waves over a narrow tile's keys, four at 128 dims
    if (head_dim == 32 || value_dim != head_dim) vs = 1;
    waves = head_dim == 128 && vs == 1 ? 4 : 8;
  }
  if (g_force_nt) { nt = g_force_nt; waves = g_force_waves; }
  if (g_force_vs) vs = g_force_vs;
  if (nt > 1) vs = 1;
#define PICK(D, NT, WV) if (head_dim == D && nt == NT && waves == WV && vs == 1) GO(D, NT, WV, 1)
#define PICK_SHARED(D, WV, VS) if (head_dim == D && nt == 1 && waves == WV && vs == VS) GO(D, 1, WV, VS)
  PICK(32, 4, 4); PICK(32, 2, 4); PICK(32, 2, 8); PICK(32, 1, 8); PICK(32, 1, 16);
  PICK(64, 4, 4); PICK(64, 2, 4); PICK(64, 2, 8); PICK(64, 1, 4); PICK(64, 1, 8); PICK(64, 1, 16);
  PICK(128, 2, 4); PICK(128, 1, 4); PICK(128, 1, 8);
  PICK_SHARED(32, 16, 2);
  PICK_SHARED(64, 16, 2); PICK_SHARED(64, 16, 4); PICK_SHARED(64, 8, 2); PICK_SHARED(64, 8, 4);
  PICK_SHARED(128, 8, 2); PICK_SHARED(128, 8, 4);
#undef PICK_SHARED
#undef PICK
  return MS_UNSUPPORTED;
#undef GO
}

// Split shape, for long contexts in small batches: every request has exactly one token and the group
// (num_heads / num_kv_heads) is at most 16; the keys are spread over n_splits blocks and combined.
// part_o: float [R, nh, n_splits, value_dim], part_ml: float [R, nh, n_splits, 2].  Each request spreads its blocks of
// 32 keys evenly over the n_splits waves, at least min_blocks to a wave, so the launch does not depend on
// how long the contexts are.
extern "C" int ms_paged_attention_mfma_decode(const void* q, long long q_stride, const void* k_pages,
                                              const void* vt_pages, const int* block_table, int table_stride,
                                              const int* table_rows, const int* q_start, const int* context_lens, void* out,
                                              long long out_stride, void* part_o, void* part_ml, int n_requests,
                                              int num_heads, int num_kv_heads, int head_dim, int value_dim, int page_size,
                                              float scale, int window, int min_blocks, int n_splits, const float* sink,
                                              float softcap, const float* slopes, const void* gate, long long gate_stride,
                                              int gate_width, float out_scale, hipStream_t stream) {
  if (n_requests <= 0) return MS_OK;
  if (num_heads <= 0 || num_kv_heads <= 0 || num_heads % num_kv_heads || table_stride <= 0) return MS_BAD_ARG;
  if (num_heads / num_kv_heads > 16) return MS_UNSUPPORTED;
  if (!(scale > 0.f)) return MS_BAD_ARG;
  if (!ms_attention_mfma_supported(head_dim, value_dim, page_size)) return MS_UNSUPPORTED;
  if (!gate_fits(gate, gate_stride, gate_width, value_dim)) return MS_UNSUPPORTED;
  if (min_blocks <= 0 || n_splits <= 0 || n_splits > COMBINE_MAX_SPLITS) return MS_BAD_ARG;
  if (q_stride % 8 || out_stride % 4 || ((uintptr_t)q % 16) || ((uintptr_t)out % 8) || ((uintptr_t)part_o % 16)) return MS_UNSUPPORTED;
  if (n_requests > 65535 || num_kv_heads > 65535) return MS_UNSUPPORTED;
  const bool changed = softcap > 0.f || slopes != nullptr || gate != nullptr || out_scale != 1.0f || value_dim != head_dim;
  const AttnExtras ex = {scale, softcap > 0.f ? softcap : 0.f, softcap > 0.f ? 2.0f * 1.4426950408889634f / softcap : 0.f,
                         slopes, (const bf16*)gate, (size_t)gate_stride, gate_width, out_scale, value_dim};
  const AttnExtras* extras = changed ? &ex : nullptr;
#define GO(D) return launch_split<D>((const bf16*)q, q_stride, (const bf16*)k_pages, (const bf16*)vt_pages, block_table, table_stride, table_rows, q_start, context_lens, (bf16*)out, out_stride, (float*)part_o, (float*)part_ml, n_requests, num_heads, num_kv_heads, page_size, scale, window, min_blocks, n_splits, sink, extras, stream)
  if (head_dim == 32) GO(32);
  if (head_dim == 64) GO(64);
  GO(128);
#undef GO
}
