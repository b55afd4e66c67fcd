// out[n, h, :] = Mt[h] . in[n, h, :] (* sigmoid of a gate) for every head h on the matrix cores, bfloat16 in and out, float
// accumulation: the per-head maps of latent attention (v_mfma_f32_16x16x32_bf16).  Mt is [heads, J, I]: a head's output
// features are the A operand's rows (a lane reads 16 bytes of one), the tokens' slices of that head the B operand, so a lane
// ends with four neighbouring features of one token and writes them as one run.  A wave owns 16 * FT features by 16 * NT
// tokens, a block's four waves neighbouring features of the same tokens; each output sums over I in the same order whatever
// the batch.  Few tokens (a decode step) take NT = 1: many small blocks, each a short stream of its head's matrix; many
// tokens take NT = 4, FT = 2.
#include "common.h"
#include "api.h"

namespace {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) __bf16 bf16x4;
typedef __attribute__((ext_vector_type(4))) float f32x4;

constexpr int HW = 4;     // waves of a block

template <int NT, int FT>
__global__ void __launch_bounds__(HW * MS_WAVE)
head_matmul_mfma_kernel(const bf16* __restrict__ in, size_t in_tok, size_t in_head, const bf16* __restrict__ Mt,
                        bf16* __restrict__ out, size_t out_tok, size_t out_head, const bf16* __restrict__ gate,
                        size_t gate_tok, int gate_w, int N, int I, int J) {
  const int lane = threadIdx.x & (MS_WAVE - 1);
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / MS_WAVE);
  const int col = lane & 15, kq = lane >> 4;
  const int h = blockIdx.z;
  const int f0 = (blockIdx.x * HW + wave) * 16 * FT, n0 = blockIdx.y * 16 * NT;
  if (f0 >= J) return;                       // no barrier below
  const bf16* wrow[FT];
#pragma unroll
  for (int u = 0; u < FT; ++u) wrow[u] = Mt + ((size_t)h * J + min(f0 + u * 16 + col, J - 1)) * I + kq * 8;
  const bf16* arow[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) arow[t] = in + (size_t)min(n0 + t * 16 + col, N - 1) * in_tok + (size_t)h * in_head + kq * 8;
  f32x4 acc[FT][NT];
#pragma unroll
  for (int u = 0; u < FT; ++u)
#pragma unroll
    for (int t = 0; t < NT; ++t) acc[u][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  // what lies past the last feature or token is a repeated row whose results are not stored
#pragma unroll 4
  for (int k = 0; k < I; k += 32) {
    bf16x8 wv[FT], av[NT];
#pragma unroll
    for (int u = 0; u < FT; ++u) wv[u] = *reinterpret_cast<const bf16x8*>(wrow[u] + k);
#pragma unroll
    for (int t = 0; t < NT; ++t) av[t] = *reinterpret_cast<const bf16x8*>(arow[t] + k);
#pragma unroll
    for (int u = 0; u < FT; ++u)
#pragma unroll
      for (int t = 0; t < NT; ++t) acc[u][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wv[u], av[t], acc[u][t], 0, 0, 0);
  }
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int n = n0 + t * 16 + col;
    if (n >= N) continue;
    const bf16* gp = gate ? gate + (size_t)n * gate_tok + (size_t)h * gate_w : nullptr;
    const float one = gp && gate_w == 1 ? 1.0f / (1.0f + expf(-to_float(gp[0]))) : 1.0f;
#pragma unroll
    for (int u = 0; u < FT; ++u) {
      const int f = f0 + u * 16 + kq * 4;
      float v[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        v[i] = acc[u][t][i] * one;
        if (gp && gate_w != 1 && f + i < J) v[i] *= 1.0f / (1.0f + expf(-to_float(gp[f + i])));
      }
      bf16* op = out + (size_t)n * out_tok + (size_t)h * out_head + f;
      if (f + 3 < J && ((uintptr_t)op & 7) == 0) {
        bf16x4 p;
#pragma unroll
        for (int i = 0; i < 4; ++i) p[i] = (__bf16)v[i];
        *reinterpret_cast<bf16x4*>(op) = p;
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (f + i < J) op[i] = from_float<bf16>(v[i]);
      }
    }
  }
}

}  // namespace

// Rows of `in` are read in pieces of 16 bytes: I a multiple of 32, strides of 8, both operands 16-byte aligned.
extern "C" int ms_head_matmul_mfma(const void* in, long long in_tok, long long in_head, const void* Mt, void* out,
                                   long long out_tok, long long out_head, const void* gate, long long gate_tok, int gate_w,
                                   int n_tokens, int heads, int I, int J, hipStream_t stream) {
  if (n_tokens <= 0) return MS_OK;
  if (heads <= 0 || I <= 0 || J <= 0 || (gate && gate_w != 1 && gate_w != J)) return MS_BAD_ARG;
  if (I % 32 || in_tok % 8 || in_head % 8 || (((uintptr_t)in | (uintptr_t)Mt) & 15) || heads > 65535) return MS_UNSUPPORTED;
#define GO(NT, FT)                                                                                                     \
  do {                                                                                                                 \
    dim3 grid((J + HW * 16 * FT - 1) / (HW * 16 * FT), (n_tokens + 16 * NT - 1) / (16 * NT), heads), block(HW * MS_WAVE); \
    if (grid.y > 65535) return MS_UNSUPPORTED;                                                                         \
    head_matmul_mfma_kernel<NT, FT><<<grid, block, 0, stream>>>((const bf16*)in, (size_t)in_tok, (size_t)in_head,       \
        (const bf16*)Mt, (bf16*)out, (size_t)out_tok, (size_t)out_head, (const bf16*)gate, (size_t)gate_tok, gate_w,    \
        n_tokens, I, J);                                                                                               \
  } while (0)
  if (n_tokens <= 16) GO(1, 1);
  else if (n_tokens <= 128) GO(2, 1);
  else GO(4, 2);
#undef GO
  return ms_launch_status();
}
