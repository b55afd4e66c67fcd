// Attention over cached latents on the matrix cores (v_mfma_f32_16x16x32_bf16), bfloat16 in, float softmax.
//
// All query heads read the same keys [c_j ; kr_j] and the same values c_j, so a *column* is a (token, head) pair
// and a wave owns 16 consecutive columns of one request (head running fastest): every key it loads serves 16
// heads, or several tokens' heads.  The waves of a block share one tile of 16 columns and take its key blocks in turn,
// each with its own running maximum, sum and accumulators, merged through LDS at the end in wave order: a single
// decoded token's keys are then walked by four waves at once.  Keys are walked in blocks of 32:
//
//   S^T[key, col]  = K[key, :] . Q^T[:, col]      A operand: 16 keys x 32 entries read in place from the pages (the
//                                                 latent's C entries, then the rotated part's R), B: the query
//   online softmax per column in float (log2 units); a column's own position and window mask its keys; the
//   sink joins the denominator at the end
//   O^T[i, col] += c^T[i, key] . P^T[key, col]    A operand: the latent pages' transposed copy [page][C][slot],
//                                                 B: P^T straight from the S^T accumulators
//
// The sums of the exponentials come from one more product with ones (the bfloat16 values that weigh the latents).
// Values past the last visible key are zeroed before use and pages past the context are never dereferenced.
// Launch: grid (column tiles of the longest portion, requests); a block without a tile leaves at once, so the launch
// depends on the step's number of requests and longest portion only.  A step of single tokens may spread a tile's key
// blocks over several blocks (grid z, SPLIT): each leaves its accumulators with their maximum and sum, and
// latent_combine_kernel adds a column's parts up in split order.
#include "common.h"
#include "api.h"

namespace {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

constexpr int LM_WAVES = 4;

template <int C, int R, bool SPLIT>
__global__ void __launch_bounds__(LM_WAVES * MS_WAVE)
latent_attention_mfma_kernel(const bf16* __restrict__ q, size_t q_tok, size_t q_head, const bf16* __restrict__ c_pages,
                             const bf16* __restrict__ r_pages, const bf16* __restrict__ ct_pages,
                             const int* __restrict__ block_table, int table_stride, const int* __restrict__ table_rows,
                             const int* __restrict__ q_start, const int* __restrict__ context_lens,
                             const float* __restrict__ sink, bf16* __restrict__ out, size_t out_tok, size_t out_head,
                             int H, int page_size, float scale_log2e, int window, float* __restrict__ part_o,
                             float* __restrict__ part_ml) {
  constexpr int KS_C = C / 32, KS_R = R / 32, CT = C / 16;
  __shared__ float sm_m[LM_WAVES][16], sm_l[LM_WAVES][16];
  __shared__ f32x4 sm_o[CT][MS_WAVE];
  const int lane = threadIdx.x & (MS_WAVE - 1);
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / MS_WAVE);
  const int col16 = lane & 15, kq = lane >> 4;
  const int r = blockIdx.y;
  const int q0 = q_start[r];
  const int qlen = q_start[r + 1] - q0;
  const int ncols = qlen * H;
  const int c0 = blockIdx.x * 16;
  if (c0 >= ncols) return;                         // the whole block
  const int start_pos = context_lens[r] - qlen;
  const int* table = block_table + (size_t)(table_rows ? table_rows[r] : r) * table_stride;

  const int last_col = min(ncols, c0 + 16) - 1;
  const int key_hi = start_pos + last_col / H;
  const int key_lo = window > 0 ? max(0, start_pos + c0 / H - window + 1) : 0;

  // this lane's column
  const int c = c0 + col16;
  const int cc = min(c, ncols - 1);
  const int tok = q0 + cc / H, head = cc % H;
  const int pos = c < ncols ? start_pos + cc / H : -1;     // -1: an idle column; it sees no key and writes nothing
  bf16x8 qv[KS_C + KS_R];
  {
    const bf16* qp = q + (size_t)tok * q_tok + (size_t)head * q_head + kq * 8;
#pragma unroll
    for (int s = 0; s < KS_C + KS_R; ++s) qv[s] = *reinterpret_cast<const bf16x8*>(qp + s * 32);
  }
  bf16x8 ones;
#pragma unroll
  for (int i = 0; i < 8; ++i) ones[i] = (__bf16)1.0f;

  float m = -INFINITY;
  f32x4 lsum = {0.f, 0.f, 0.f, 0.f};
  f32x4 o[CT];
#pragma unroll
  for (int t = 0; t < CT; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};

  // this block's key blocks of 32: all of the tile's, or (SPLIT) its share of them
  int b_lo = key_lo / 32, b_hi = key_hi / 32;
  if (SPLIT) {
    const int share = (b_hi - b_lo + (int)gridDim.z) / (int)gridDim.z;     // rounded up
    b_lo += (int)blockIdx.z * share;
    b_hi = min(b_hi, b_lo + share - 1);
  }
  for (int base = (b_lo + wave) * 32; base <= b_hi * 32; base += 32 * LM_WAVES) {
    // the two 16-key halves of the block: a half lies in one page (pages hold a multiple of 16 keys)
    size_t row0[2];     // first key's row in the pools (page * page_size + offset); the null page past the context
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int kb = base + u * 16;
      const int page = kb <= key_hi ? __builtin_amdgcn_readfirstlane(table[kb / page_size]) : 0;
      row0[u] = (size_t)page * page_size + (kb <= key_hi ? kb % page_size : 0);
    }
    // scores: s[u] holds keys base + u*16 + kq*4 + (0..3) of this lane's column.  All key fragments of the block are
    // asked for before the first product, so that a block costs one trip to memory for its keys, not one per fragment.
    f32x4 s[2];
    {
      bf16x8 kf[2][KS_C + KS_R];
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const bf16* kp = c_pages + (row0[u] + col16) * C + kq * 8;
        const bf16* rp = r_pages + (row0[u] + col16) * R + kq * 8;
#pragma unroll
        for (int ks = 0; ks < KS_C; ++ks) kf[u][ks] = *reinterpret_cast<const bf16x8*>(kp + ks * 32);
#pragma unroll
        for (int ks = 0; ks < KS_R; ++ks) kf[u][KS_C + ks] = *reinterpret_cast<const bf16x8*>(rp + ks * 32);
      }
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < KS_C + KS_R; ++ks) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[u][ks], qv[ks], acc, 0, 0, 0);
        s[u] = acc;
      }
    }
    // mask, block maximum
    float bm = -INFINITY;
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int key = base + u * 16 + kq * 4 + i;
        const bool see = key <= pos && (window <= 0 || key > pos - window);
        const float v = see ? s[u][i] * scale_log2e : -INFINITY;
        s[u][i] = v;
        bm = fmaxf(bm, v);
      }
    bm = fmaxf(bm, __shfl_xor(bm, 16, MS_WAVE));
    bm = fmaxf(bm, __shfl_xor(bm, 32, MS_WAVE));
    const float m_new = fmaxf(m, bm);
    const float m_safe = m_new == -INFINITY ? 0.f : m_new;
    const float corr = __builtin_amdgcn_exp2f(m - m_safe);     // m = -inf: 0
    m = m_new;
    bf16x8 p;
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int i = 0; i < 4; ++i) p[u * 4 + i] = (__bf16)__builtin_amdgcn_exp2f(s[u][i] - m_safe);
    if (__builtin_amdgcn_ballot_w64(corr != 1.0f) != 0) {
      lsum *= corr;
#pragma unroll
      for (int t = 0; t < CT; ++t) o[t] *= corr;
    }
    lsum = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, p, lsum, 0, 0, 0);
    // values: lane holds entry t*16 + col16 of the latent for keys u*16 + kq*4 + (0..3)
    const bool tail = base + 31 > key_hi;
    const bf16* vp0 = ct_pages + (row0[0] / page_size) * (size_t)page_size * C + row0[0] % page_size + kq * 4;
    const bf16* vp1 = ct_pages + (row0[1] / page_size) * (size_t)page_size * C + row0[1] % page_size + kq * 4;
    constexpr int VG = CT <= 16 ? CT : (CT % 16 ? 12 : 16);     // tiles of 16 entries whose values are asked for together
    static_assert(CT % VG == 0, "the latent's tiles come in whole groups");
#pragma unroll
    for (int t0 = 0; t0 < CT; t0 += VG) {
      bf16x4 va[VG], vb[VG];
#pragma unroll
      for (int j = 0; j < VG; ++j) {
        const size_t at = (size_t)((t0 + j) * 16 + col16) * page_size;
        va[j] = *reinterpret_cast<const bf16x4*>(vp0 + at);
        vb[j] = *reinterpret_cast<const bf16x4*>(vp1 + at);
      }
#pragma unroll
      for (int j = 0; j < VG; ++j) {
        bf16x8 vv;
#pragma unroll
        for (int i = 0; i < 4; ++i) { vv[i] = va[j][i]; vv[4 + i] = vb[j][i]; }
        if (tail) {      // what a reused page still holds past the last visible key must not meet the zero weights
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            if (base + kq * 4 + i > key_hi) vv[i] = (__bf16)0.0f;
            if (base + 16 + kq * 4 + i > key_hi) vv[4 + i] = (__bf16)0.0f;
          }
        }
        o[t0 + j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vv, p, o[t0 + j], 0, 0, 0);
      }
    }
  }
  float l = lsum[0];      // every row of the product with ones is the column's sum
  // merge the waves' shares (each relative to its own maximum) into wave 0, in wave order
  if (kq == 0) { sm_m[wave][col16] = m; sm_l[wave][col16] = l; }
  __syncthreads();
  {
    float big = sm_m[0][col16];
#pragma unroll
    for (int w = 1; w < LM_WAVES; ++w) big = fmaxf(big, sm_m[w][col16]);
    const float safe = big == -INFINITY ? 0.f : big;
    const float f = __builtin_amdgcn_exp2f(m - safe);      // a wave that saw no key: 0
#pragma unroll
    for (int t = 0; t < CT; ++t) o[t] *= f;
    l = 0.f;
#pragma unroll
    for (int w = 0; w < LM_WAVES; ++w) l += sm_l[w][col16] * __builtin_amdgcn_exp2f(sm_m[w][col16] - safe);
    m = big;
  }
  for (int w = 1; w < LM_WAVES; ++w) {
    if (wave == w) {
#pragma unroll
      for (int t = 0; t < CT; ++t) sm_o[t][lane] = o[t];
    }
    __syncthreads();
    if (wave == 0) {
#pragma unroll
      for (int t = 0; t < CT; ++t) o[t] += sm_o[t][lane];
    }
    __syncthreads();
  }
  if (wave != 0 || pos < 0) return;
  if (SPLIT) {            // (a share without keys leaves m = -inf, l = 0 and zeros)
    const size_t at = ((size_t)tok * H + head) * gridDim.z + blockIdx.z;
    float* po = part_o + at * C + kq * 4;
#pragma unroll
    for (int t = 0; t < CT; ++t) *reinterpret_cast<f32x4*>(po + t * 16) = o[t];
    if (kq == 0) { part_ml[2 * at] = m; part_ml[2 * at + 1] = l; }
    return;
  }
  if (sink) {             // the sink: one more term exp(sink) in the denominator, unscaled, with no value
    const float sk = sink[head] * 1.4426950408889634f;
    const float big = fmaxf(m, sk);
    const float f = __builtin_amdgcn_exp2f(m - big);
    l = l * f + __builtin_amdgcn_exp2f(sk - big);
#pragma unroll
    for (int t = 0; t < CT; ++t) o[t] *= f;
  }
  const float inv = 1.0f / l;
  bf16* op = out + (size_t)tok * out_tok + (size_t)head * out_head + kq * 4;
#pragma unroll
  for (int t = 0; t < CT; ++t) {
    bf16x4 w;
#pragma unroll
    for (int i = 0; i < 4; ++i) w[i] = (__bf16)(o[t][i] * inv);
    *reinterpret_cast<bf16x4*>(op + t * 16) = w;
  }
}

// out[column] = sum over the splits of a column's parts, brought to one maximum, divided by their sums (and the sink's
// term).  A block per (token, head); tokens of no request (from q_start[n_requests] on) are left alone.
__global__ void __launch_bounds__(128)
latent_combine_kernel(const float* __restrict__ part_o, const float* __restrict__ part_ml, const int* __restrict__ q_start,
                      int n_requests, const float* __restrict__ sink, bf16* __restrict__ out, size_t out_tok,
                      size_t out_head, int H, int C, int splits) {
  const int tok = blockIdx.x, head = blockIdx.y;
  if (tok >= q_start[n_requests]) return;
  const size_t at = ((size_t)tok * H + head) * splits;
  const float* ml = part_ml + 2 * at;
  const float sk = sink ? sink[head] * 1.4426950408889634f : -INFINITY;
  float big = sk;
  for (int s = 0; s < splits; ++s) big = fmaxf(big, ml[2 * s]);
  float l = sink ? __builtin_amdgcn_exp2f(sk - big) : 0.f;
  for (int s = 0; s < splits; ++s) l += ml[2 * s + 1] * __builtin_amdgcn_exp2f(ml[2 * s] - big);
  const float inv = 1.0f / l;
  const float* po = part_o + at * C;
  for (int i = threadIdx.x * 4; i < C; i += 128 * 4) {
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int s = 0; s < splits; ++s)
      acc += *reinterpret_cast<const f32x4*>(po + (size_t)s * C + i) * __builtin_amdgcn_exp2f(ml[2 * s] - big);
    bf16x4 w;
#pragma unroll
    for (int e = 0; e < 4; ++e) w[e] = (__bf16)(acc[e] * inv);
    *reinterpret_cast<bf16x4*>(out + (size_t)tok * out_tok + (size_t)head * out_head + i) = w;
  }
}

// The shape for long portions: the WAVES waves of a block own neighbouring tiles of 16 columns, whose key ranges all but
// coincide, and read every key block of 32 from LDS.  A key block goes from memory straight to LDS (global_load_lds, 16
// bytes a lane, no registers) into one of two buffers, one block ahead of the one that is multiplied, and its page ids are
// looked up one block before that; a step has one barrier.  In LDS a key is a row of C + R entries and a latent entry of the
// transposed copy a row of the block's 32 keys, both in pieces of 16 bytes whose places are permuted by the row so that
// fragment reads spread over the banks.  Blocks with the latest columns, which have the most keys, start first.
template <int C, int R> struct Staged {
  static constexpr int KP = (C + R) / 8;                                   // pieces of a key's row
  static constexpr int SHIFT = KP % 16 == 8 ? 1 : (KP % 16 == 0 ? 0 : 2);  // neighbouring rows start 32, 0 or 16 / 48 banks apart
  static constexpr int MASK = SHIFT == 2 ? 3 : 7;
  static_assert(C % 64 == 0 && (R / 8) % (MASK + 1) == 0, "pieces are permuted within whole groups");
  static constexpr int K_LOADS = 32 * KP / MS_WAVE, V_LOADS = C * 4 / MS_WAVE;    // loads of 64 pieces (1 KB)
  static constexpr size_t BUFFER = (size_t)(K_LOADS + V_LOADS) * MS_WAVE * 8;     // entries of one buffer
};

template <int C, int R, int WAVES>
__global__ void __launch_bounds__(WAVES * MS_WAVE)
latent_attention_mfma_staged_kernel(const bf16* __restrict__ q, size_t q_tok, size_t q_head,
                                    const bf16* __restrict__ c_pages, const bf16* __restrict__ r_pages,
                                    const bf16* __restrict__ ct_pages, const int* __restrict__ block_table,
                                    int table_stride, const int* __restrict__ table_rows,
                                    const int* __restrict__ q_start, const int* __restrict__ context_lens,
                                    const float* __restrict__ sink, bf16* __restrict__ out, size_t out_tok,
                                    size_t out_head, int H, int page_size, float scale_log2e, int window) {
  using L = Staged<C, R>;
  constexpr int KS_C = C / 32, KS_R = R / 32, CT = C / 16;
  constexpr int LOADS = (L::K_LOADS + L::V_LOADS + WAVES - 1) / WAVES;
  extern __shared__ __align__(16) bf16 ls[];       // two buffers: keys [32][C + R], then transposed latents [C][32]
  const int lane = threadIdx.x & (MS_WAVE - 1);
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / MS_WAVE);
  const int col16 = lane & 15, kq = lane >> 4;
  const int r = blockIdx.y;
  const int q0 = q_start[r];
  const int qlen = q_start[r + 1] - q0;
  const int ncols = qlen * H;
  const int b0 = (int)(gridDim.x - 1 - blockIdx.x) * 16 * WAVES;        // the block's first column
  if (b0 >= ncols) return;                         // the whole block
  const int start_pos = context_lens[r] - qlen;
  const int* table = block_table + (size_t)(table_rows ? table_rows[r] : r) * table_stride;
  // the block's keys: from the first column's window to the last column's own position
  const int blk_hi = start_pos + (min(ncols, b0 + 16 * WAVES) - 1) / H;
  const int blk_lo = window > 0 ? max(0, start_pos + b0 / H - window + 1) : 0;
  // this wave's tile and this lane's column
  const int c0 = b0 + wave * 16;
  const bool tile = c0 < ncols;
  const int key_hi = tile ? start_pos + (min(ncols, c0 + 16) - 1) / H : -1;
  const int key_lo = (tile && window > 0) ? max(0, start_pos + c0 / H - window + 1) : 0;
  const int c = c0 + col16;
  const int cc = min(c, ncols - 1);
  const int tok = q0 + cc / H, head = cc % H;
  const int pos = c < ncols ? start_pos + cc / H : -1;
  bf16x8 qv[KS_C + KS_R];
  {
    const bf16* qp = q + (size_t)tok * q_tok + (size_t)head * q_head + kq * 8;
#pragma unroll
    for (int s = 0; s < KS_C + KS_R; ++s) qv[s] = *reinterpret_cast<const bf16x8*>(qp + s * 32);
  }
  bf16x8 ones;
#pragma unroll
  for (int i = 0; i < 8; ++i) ones[i] = (__bf16)1.0f;
  float m = -INFINITY;
  f32x4 lsum = {0.f, 0.f, 0.f, 0.f};
  f32x4 o[CT];
#pragma unroll
  for (int t = 0; t < CT; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};

  typedef __attribute__((address_space(3))) void lds_void;
  typedef const __attribute__((address_space(1))) void global_void;
  int page0 = 0, page1 = 0;        // the pages of the two 16-key halves of the block to be asked for next
  auto lookup = [&](int base) __attribute__((always_inline)) {
    page0 = base <= blk_hi ? __builtin_amdgcn_readfirstlane(table[base / page_size]) : 0;
    page1 = base + 16 <= blk_hi ? __builtin_amdgcn_readfirstlane(table[(base + 16) / page_size]) : 0;
  };
  // Keys past the block's last one come from the null page or from what the page's last user left: their scores are
  // masked, and their latents zeroed in LDS before use.
  auto issue = [&](int base, bf16* buf) __attribute__((always_inline)) {
    const int off0 = base % page_size, off1 = base + 16 <= blk_hi ? (base + 16) % page_size : 0;
    const size_t row0 = (size_t)page0 * page_size + off0, row1 = (size_t)page1 * page_size + off1;
    const bf16* vt0 = ct_pages + (size_t)page0 * page_size * C + off0;
    const bf16* vt1 = ct_pages + (size_t)page1 * page_size * C + off1;
    int lane_now = lane;       // each load's place is worked out when it is asked for: kept across the loop the places of all
    asm volatile("" : "+v"(lane_now));     // loads would take the registers that the accumulators need
#pragma unroll
    for (int p = 0; p < LOADS; ++p) {
      const int load = wave + p * WAVES;
      if ((p + 1) * WAVES <= L::K_LOADS || (p * WAVES < L::K_LOADS && load < L::K_LOADS)) {
        const int at = load * MS_WAVE + lane_now, key = at / L::KP, place = at - key * L::KP;
        const int piece = place ^ ((key >> L::SHIFT) & L::MASK);   // (within its group: the latent's pieces stay the latent's)
        const size_t row = (key < 16 ? row0 : row1) + (key & 15);
        const bool latent = piece < C / 8;
        const bf16* from = latent ? c_pages : r_pages;
        const size_t off = row * (latent ? C : R) + (piece - (latent ? 0 : C / 8)) * 8;
        __builtin_amdgcn_global_load_lds((global_void*)(from + off), (lds_void*)(buf + (size_t)load * MS_WAVE * 8), 16, 0, 0);
      } else if ((p + 1) * WAVES <= L::K_LOADS + L::V_LOADS || load < L::K_LOADS + L::V_LOADS) {
        const int at = (load - L::K_LOADS) * MS_WAVE + lane_now, dim = at >> 2, piece = (at & 3) ^ ((dim >> 2) & 3);
        const bf16* from = piece < 2 ? vt0 : vt1;
        const size_t off = (size_t)dim * page_size + (piece & 1) * 8;
        __builtin_amdgcn_global_load_lds((global_void*)(from + off), (lds_void*)(buf + (size_t)load * MS_WAVE * 8), 16, 0, 0);
      }
    }
  };
  // this lane's fragment places: key rows of col16 (+ 16), latent rows of col16 (+ 16 t)
  const int swap = (col16 >> L::SHIFT) & L::MASK;
  const int k_even = (col16 * L::KP + (kq ^ swap)) * 8, k_odd = (col16 * L::KP + ((kq + 4) ^ swap)) * 8;
  const int v_swap = (col16 >> 2) & 3;
  const int v_at0 = 32 * L::KP * 8 + col16 * 32 + (((kq >> 1) ^ v_swap) * 8) + (kq & 1) * 4;
  const int v_at1 = 32 * L::KP * 8 + col16 * 32 + (((2 + (kq >> 1)) ^ v_swap) * 8) + (kq & 1) * 4;

  const int first = (blk_lo / 32) * 32;
  lookup(first);
  issue(first, ls);
  lookup(first + 32);
  int turn = 0;
  for (int base = first; base <= blk_hi; base += 32, turn ^= 1) {
    __builtin_amdgcn_s_waitcnt(0x0F70);   // vmcnt(0): this wave's share of the block has landed in LDS
    __syncthreads();                      // everybody's has, and nobody reads the other buffer any more
    bf16* buf = ls + (turn ? L::BUFFER : 0);
    if (base + 31 > blk_hi) {             // what a reused page still holds past the last key must not meet the zero weights
#pragma unroll 1
      for (int e = threadIdx.x; e < C * 32; e += WAVES * MS_WAVE) {
        const int dim = e >> 5, place = e & 31, key = (((place >> 3) ^ ((dim >> 2) & 3)) << 3) + (place & 7);
        if (base + key > blk_hi) buf[32 * L::KP * 8 + e] = from_float<bf16>(0.f);
      }
      __syncthreads();
    }
    if (base + 32 <= blk_hi) {
      issue(base + 32, ls + (turn ? 0 : L::BUFFER));
      lookup(base + 64);
    }
    if (!tile || base > key_hi || base + 31 < key_lo) continue;     // none of this block's keys is the tile's
    f32x4 s[2];
#pragma unroll
    for (int u = 0; u < 2; ++u) s[u] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < KS_C + KS_R; ++ks)
#pragma unroll
      for (int u = 0; u < 2; ++u) {
        const bf16* kp = buf + u * 16 * L::KP * 8 + (ks & 1 ? k_odd : k_even) + (ks >> 1) * 64;
        s[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(kp), qv[ks], s[u], 0, 0, 0);
      }
    float bm = -INFINITY;
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int key = base + u * 16 + kq * 4 + i;
        const bool see = key <= pos && (window <= 0 || key > pos - window);
        const float v = see ? s[u][i] * scale_log2e : -INFINITY;
        s[u][i] = v;
        bm = fmaxf(bm, v);
      }
    bm = fmaxf(bm, __shfl_xor(bm, 16, MS_WAVE));
    bm = fmaxf(bm, __shfl_xor(bm, 32, MS_WAVE));
    const float m_new = fmaxf(m, bm);
    const float m_safe = m_new == -INFINITY ? 0.f : m_new;
    const float corr = __builtin_amdgcn_exp2f(m - m_safe);
    m = m_new;
    bf16x8 p;
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
      for (int i = 0; i < 4; ++i) p[u * 4 + i] = (__bf16)__builtin_amdgcn_exp2f(s[u][i] - m_safe);
    if (__builtin_amdgcn_ballot_w64(corr != 1.0f) != 0) {
      lsum *= corr;
#pragma unroll
      for (int t = 0; t < CT; ++t) o[t] *= corr;
    }
    lsum = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ones, p, lsum, 0, 0, 0);
    auto value = [&](int t) __attribute__((always_inline)) {
      const bf16x4 a = *reinterpret_cast<const bf16x4*>(buf + v_at0 + t * 16 * 32);
      const bf16x4 b = *reinterpret_cast<const bf16x4*>(buf + v_at1 + t * 16 * 32);
      bf16x8 vv;
#pragma unroll
      for (int i = 0; i < 4; ++i) { vv[i] = a[i]; vv[4 + i] = b[i]; }
      return vv;
    };
#pragma unroll
    for (int t = 0; t < CT; ++t) o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(value(t), p, o[t], 0, 0, 0);
  }
  if (pos < 0) return;
  float l = lsum[0];
  if (sink) {
    const float sk = sink[head] * 1.4426950408889634f;
    const float big = fmaxf(m, sk);
    const float f = __builtin_amdgcn_exp2f(m - big);
    l = l * f + __builtin_amdgcn_exp2f(sk - big);
#pragma unroll
    for (int t = 0; t < CT; ++t) o[t] *= f;
  }
  const float inv = 1.0f / l;
  bf16* op = out + (size_t)tok * out_tok + (size_t)head * out_head + kq * 4;
#pragma unroll
  for (int t = 0; t < CT; ++t) {
    bf16x4 w;
#pragma unroll
    for (int i = 0; i < 4; ++i) w[i] = (__bf16)(o[t][i] * inv);
    *reinterpret_cast<bf16x4*>(op + t * 16) = w;
  }
}

}  // namespace

extern "C" int ms_latent_attention_mfma_supported(int C, int R, int page_size) {
  return (C == 64 || C == 128 || C == 192 || C == 256 || C == 384 || C == 512) && (R == 32 || R == 64) && page_size > 0 && page_size % 16 == 0;
}

// q [n, heads, C + R] (strides in elements, 16-byte aligned rows), c_pages [P, 1, page, C], r_pages [P, 1, page, R],
// ct_pages [P, 1, C, page] (the latents once more, transposed), out [n, heads, C].  Request r owns tokens
// q_start[r]..q_start[r+1]-1 and holds context_lens[r] keys once this step's are stored; max_q_len bounds its tokens.
// splits > 1 (max_q_len 1 only): a tile's keys over so many blocks; part_o float [n, heads, splits, C] and part_ml float
// [n, heads, splits, 2] for n_tokens tokens take their parts.
extern "C" int ms_latent_attention_mfma(const void* q, long long q_tok, long long q_head, const void* c_pages,
                                        const void* r_pages, const void* ct_pages, const int* block_table,
                                        int table_stride, const int* table_rows, const int* q_start,
                                        const int* context_lens, const float* sink, void* out, long long out_tok,
                                        long long out_head, int n_requests, int max_q_len, int heads, int C, int R,
                                        int page_size, long long num_pages, float scale, int window, int splits,
                                        int n_tokens, float* part_o, float* part_ml, hipStream_t stream) {
  if (n_requests <= 0 || max_q_len <= 0) return MS_OK;
  if (heads <= 0 || table_stride <= 0 || splits <= 0) return MS_BAD_ARG;
  if (splits > 1 && (max_q_len != 1 || !part_o || !part_ml || n_tokens <= 0 || splits > 1024)) return MS_BAD_ARG;
  if (!ms_latent_attention_mfma_supported(C, R, page_size)) return MS_UNSUPPORTED;
  if (q_tok % 8 || q_head % 8 || out_tok % 4 || out_head % 4) return MS_UNSUPPORTED;
  if (num_pages * page_size >= (1ll << 31) || n_requests > 65535) return MS_UNSUPPORTED;
  const long long tiles = ((long long)max_q_len * heads + 15) / 16;
  const float sl = scale * 1.4426950408889634f;
  // long portions: neighbouring tiles over key blocks staged in LDS (more than the 64 KB a launch may ask for without more
  // ado, so the kernel's limit is raised once), eight tiles a block where that still fills the chip; else a tile's keys over
  // the four waves of a block
  const bool staged = tiles >= 8 && splits == 1;
  const bool wide = staged && (tiles + 7) / 8 * n_requests >= ms_compute_units();
  const int per = wide ? 8 : (staged ? LM_WAVES : 1);
  dim3 grid((unsigned)((tiles + per - 1) / per), n_requests, splits), block((wide ? 8 : LM_WAVES) * MS_WAVE);
#define ARGS                                                                                                            \
      (const bf16*)q, (size_t)q_tok, (size_t)q_head, (const bf16*)c_pages, (const bf16*)r_pages, (const bf16*)ct_pages, \
      block_table, table_stride, table_rows, q_start, context_lens, sink, (bf16*)out, (size_t)out_tok,                  \
      (size_t)out_head, heads, page_size, sl, window
#define LAUNCH(CC, RR)                                                                                                  \
  do {                                                                                                                  \
    constexpr size_t lds = 2 * Staged<CC, RR>::BUFFER * sizeof(bf16);                                                   \
    if (staged) {                                                                                                       \
      static bool raised = false;                                                                                       \
      if (!raised) {                                                                                                    \
        if (hipFuncSetAttribute((const void*)latent_attention_mfma_staged_kernel<CC, RR, LM_WAVES>,                     \
                                hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess ||                  \
            hipFuncSetAttribute((const void*)latent_attention_mfma_staged_kernel<CC, RR, 8>,                            \
                                hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess)                    \
          return MS_LAUNCH_FAILED;                                                                                      \
        raised = true;                                                                                                  \
      }                                                                                                                 \
      if (wide) latent_attention_mfma_staged_kernel<CC, RR, 8><<<grid, block, lds, stream>>>(ARGS);                     \
      else latent_attention_mfma_staged_kernel<CC, RR, LM_WAVES><<<grid, block, lds, stream>>>(ARGS);                   \
    } else if (splits > 1) {                                                                                            \
      latent_attention_mfma_kernel<CC, RR, true><<<grid, block, 0, stream>>>(ARGS, part_o, part_ml);                    \
    } else {                                                                                                            \
      latent_attention_mfma_kernel<CC, RR, false><<<grid, block, 0, stream>>>(ARGS, nullptr, nullptr);                  \
    }                                                                                                                   \
  } while (0)
#define SIZES(CC)                          \
  case CC:                                 \
    if (R == 32) LAUNCH(CC, 32);           \
    else LAUNCH(CC, 64);                   \
    break
  switch (C) {
    SIZES(64); SIZES(128); SIZES(192); SIZES(256); SIZES(384); SIZES(512);
  }
#undef SIZES
#undef LAUNCH
#undef ARGS
  if (splits > 1) {
    dim3 cgrid(n_tokens, heads);
    latent_combine_kernel<<<cgrid, dim3(128), 0, stream>>>(part_o, part_ml, q_start, n_requests, sink, (bf16*)out,
                                                           (size_t)out_tok, (size_t)out_head, heads, C, splits);
  }
  return ms_launch_status();
}
