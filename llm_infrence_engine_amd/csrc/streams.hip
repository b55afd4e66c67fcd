// A residual stream made of S copies ("streams") that every sublayer reads and writes through numbers of its own:
//   write   X[t] <- sum_s M[s, t] X[s] + b[t] y      (all t at once from the old X; M is indexed [from, to])
//   read    u = sum_s a[s] X[s];   out = norm(u)
// with X float [N, S, W].  One pass over X does both: the write of the sublayer that has just run and the read of the one
// that comes next, with its norm, so X goes over the memory's wires once each way per sublayer.
// The addend y is a sublayer's output (float or bfloat16) and / or the weighted rows that a token's routed experts left:
//   y[n] = base[n] + sum_j weight[n, j] part[n * top + j]
// Norms (float, the row u held in LDS): 0 none (out = u), 1 RMS, 2 layer norm, with a weight and an optional bias.
//   streams_kernel<S, V>   S streams in registers, V neighbouring values a lane
//   streams_any_kernel     any number of streams, the old values of a column in LDS
#include "common.h"
#include "api.h"

namespace {

struct StreamsArgs {
  float* x;                // [N, S, W]
  const void* base;        // [N, W] or null
  int base_bf16;
  const float* part;       // [N * top, W] or null
  const float* part_w;     // [N, top]
  int top;
  const float* mix;        // [S, S], [from, to]; with b null: no write
  const float* b;          // [S]
  const float* a;          // [S]; null: no read
  int norm;
  const float* w;          // [W]
  const float* bias;       // [W] or null
  const int* rows;         // [n_rows] or null
  void* out;               // [n_rows, W]
  int out_bf16;
  int W;
  float eps;
  int write_back;
};

template <int V> struct Vals { float v[V]; };

template <int V> __device__ __forceinline__ Vals<V> load_f32(const float* p) {
  Vals<V> r;
  if (V == 4) {
    const float4 q = *reinterpret_cast<const float4*>(p);
    r.v[0] = q.x; r.v[1 % V] = q.y; r.v[2 % V] = q.z; r.v[3 % V] = q.w;
  } else {
    r.v[0] = p[0];
  }
  return r;
}

template <int V> __device__ __forceinline__ void store_f32(float* p, const Vals<V>& r) {
  if (V == 4) *reinterpret_cast<float4*>(p) = make_float4(r.v[0], r.v[1 % V], r.v[2 % V], r.v[3 % V]);
  else p[0] = r.v[0];
}

template <int V> __device__ __forceinline__ Vals<V> load_bf16(const bf16* p) {
  Vals<V> r;
  struct alignas(2 * V) Pack { bf16 v[V]; };
  const Pack q = *reinterpret_cast<const Pack*>(p);
#pragma unroll
  for (int e = 0; e < V; ++e) r.v[e] = to_float(q.v[e]);
  return r;
}

// the addend of row n at column i
template <int V> __device__ __forceinline__ Vals<V> addend(const StreamsArgs& A, size_t n, int i) {
  Vals<V> y;
  if (A.base) {
    y = A.base_bf16 ? load_bf16<V>((const bf16*)A.base + n * A.W + i) : load_f32<V>((const float*)A.base + n * A.W + i);
  } else {
#pragma unroll
    for (int e = 0; e < V; ++e) y.v[e] = 0.f;
  }
  if (A.part) {
    for (int j = 0; j < A.top; ++j) {
      const float g = A.part_w[n * A.top + j];
      const Vals<V> p = load_f32<V>(A.part + (n * A.top + j) * (size_t)A.W + i);
#pragma unroll
      for (int e = 0; e < V; ++e) y.v[e] = fmaf(g, p.v[e], y.v[e]);
    }
  }
  return y;
}

// out = norm of the row u that the block's threads have left in LDS (every thread reads back what it wrote itself)
template <int V> __device__ __forceinline__ void norm_row(const StreamsArgs& A, const float* u, float first_sum, float* red) {
  float mean = 0.f, inv = 1.f;
  const int step = blockDim.x * V;
  if (A.norm == 2) {
    mean = block_sum(first_sum, red) / (float)A.W;
    float q = 0.f;
    for (int i = threadIdx.x * V; i < A.W; i += step)
#pragma unroll
      for (int e = 0; e < V; ++e) { const float d = u[i + e] - mean; q = fmaf(d, d, q); }
    inv = 1.0f / sqrtf(block_sum(q, red) / (float)A.W + A.eps);
  } else if (A.norm == 1) {
    inv = 1.0f / sqrtf(block_sum(first_sum, red) / (float)A.W + A.eps);
  }
  const size_t at = (size_t)blockIdx.x * A.W;
  for (int i = threadIdx.x * V; i < A.W; i += step) {
    float o[V];
#pragma unroll
    for (int e = 0; e < V; ++e) {
      o[e] = (u[i + e] - mean) * inv;
      if (A.norm) o[e] *= A.w[i + e];
      if (A.norm && A.bias) o[e] += A.bias[i + e];
    }
    if (A.out_bf16) {
      struct alignas(2 * V) Pack { bf16 v[V]; } p;
#pragma unroll
      for (int e = 0; e < V; ++e) p.v[e] = from_float<bf16>(o[e]);
      *reinterpret_cast<Pack*>((bf16*)A.out + at + i) = p;
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) ((float*)A.out)[at + i + e] = o[e];
    }
  }
}

template <int S, int V>
__global__ void __launch_bounds__(1024) streams_kernel(const StreamsArgs A) {
  extern __shared__ __align__(16) float u_row[];
  __shared__ float red[16];
  const size_t n = A.rows ? (size_t)A.rows[blockIdx.x] : (size_t)blockIdx.x;
  float* xr = A.x + n * S * A.W;
  float sum = 0.f;
  for (int i = threadIdx.x * V; i < A.W; i += blockDim.x * V) {
    Vals<V> old[S];
#pragma unroll
    for (int s = 0; s < S; ++s) old[s] = load_f32<V>(xr + (size_t)s * A.W + i);
    if (A.b) {
      const Vals<V> y = addend<V>(A, n, i);
      Vals<V> now[S];
#pragma unroll
      for (int t = 0; t < S; ++t) {
        const float bt = A.b[t];
#pragma unroll
        for (int e = 0; e < V; ++e) now[t].v[e] = bt * y.v[e];
#pragma unroll
        for (int s = 0; s < S; ++s) {
          const float m = A.mix[s * S + t];
#pragma unroll
          for (int e = 0; e < V; ++e) now[t].v[e] = fmaf(m, old[s].v[e], now[t].v[e]);
        }
      }
#pragma unroll
      for (int t = 0; t < S; ++t) {
        if (A.write_back) store_f32<V>(xr + (size_t)t * A.W + i, now[t]);
        old[t] = now[t];
      }
    }
    if (A.a) {
      float u[V];
#pragma unroll
      for (int e = 0; e < V; ++e) u[e] = 0.f;
#pragma unroll
      for (int s = 0; s < S; ++s) {
        const float as = A.a[s];
#pragma unroll
        for (int e = 0; e < V; ++e) u[e] = fmaf(as, old[s].v[e], u[e]);
      }
#pragma unroll
      for (int e = 0; e < V; ++e) {
        u_row[i + e] = u[e];
        sum = A.norm == 1 ? fmaf(u[e], u[e], sum) : sum + u[e];
      }
    }
  }
  if (A.a) norm_row<V>(A, u_row, sum, red);
}

constexpr int ANY_THREADS = 256;

__global__ void __launch_bounds__(ANY_THREADS) streams_any_kernel(const StreamsArgs A, int S) {
  extern __shared__ __align__(16) float sh[];      // [S][ANY_THREADS] old values, then the row u
  __shared__ float red[16];
  float* old = sh + threadIdx.x;
  float* u_row = sh + (size_t)S * ANY_THREADS;
  const size_t n = A.rows ? (size_t)A.rows[blockIdx.x] : (size_t)blockIdx.x;
  float* xr = A.x + n * S * A.W;
  float sum = 0.f;
  for (int i = threadIdx.x; i < A.W; i += ANY_THREADS) {
    for (int s = 0; s < S; ++s) old[s * ANY_THREADS] = xr[(size_t)s * A.W + i];
    const float y = A.b ? addend<1>(A, n, i).v[0] : 0.f;
    float u = 0.f;
    for (int t = 0; t < S; ++t) {
      float now = old[t * ANY_THREADS];
      if (A.b) {
        now = A.b[t] * y;
        for (int s = 0; s < S; ++s) now = fmaf(A.mix[s * S + t], old[s * ANY_THREADS], now);
        if (A.write_back) xr[(size_t)t * A.W + i] = now;
      }
      if (A.a) u = fmaf(A.a[t], now, u);
    }
    if (A.a) {
      u_row[i] = u;
      sum = A.norm == 1 ? fmaf(u, u, sum) : sum + u;
    }
  }
  if (A.a) norm_row<1>(A, u_row, sum, red);
}

}  // namespace

extern "C" int ms_streams_max() { return 32; }

// x float [N, S, W].  b null: nothing is written; a null: nothing is read.  base (may be null) [N, W] of base_dtype, part
// (may be null) float [N * top, W] with part_w float [N, top]; rows (may be null) int32 [n_rows]: which rows of x; out
// [n_rows, W] of out_dtype; norm 0, 1, 2 as above; write_back 0: the written streams are only read, not kept.
extern "C" int ms_streams(float* x, const void* base, int base_dtype, const float* part, const float* part_w, int top,
                          const float* mix, const float* b, const float* a, int norm, const float* w, const float* bias,
                          float eps, const int* rows, void* out, int out_dtype, int n_rows, int S, int W, int write_back,
                          hipStream_t stream) {
  if (n_rows <= 0) return MS_OK;
  if (S <= 0 || W <= 0 || norm < 0 || norm > 2 || (norm && !w) || (a && !out) || (!a && !b) || (b && !mix)) return MS_BAD_ARG;
  if (part && (!part_w || top <= 0)) return MS_BAD_ARG;
  if ((base_dtype != MS_F32 && base_dtype != MS_BF16) || (out_dtype != MS_F32 && out_dtype != MS_BF16)) return MS_BAD_ARG;
  if (S > ms_streams_max()) return MS_UNSUPPORTED;
  const StreamsArgs A{x, base, base_dtype == MS_BF16, part, part_w, top, mix, b, a, norm, w, bias, rows, out,
                      out_dtype == MS_BF16, W, eps, write_back};
  const bool vec = W % 4 == 0 && (((uintptr_t)x | (uintptr_t)base | (uintptr_t)part | (uintptr_t)out) & 15) == 0;
  const size_t row = a ? (size_t)W * sizeof(float) : 0, any_lds = row + (size_t)S * ANY_THREADS * sizeof(float);
  if (row > 65024 || (S > 8 && any_lds > 65024)) return MS_UNSUPPORTED;     // a block's LDS, with its few words of its own
  const int lanes = vec ? W / 4 : W;
  const int threads = lanes >= 1024 ? 1024 : ((lanes + MS_WAVE - 1) / MS_WAVE) * MS_WAVE;
#define GO(S_)                                                                              \
  case S_:                                                                                  \
    if (vec) streams_kernel<S_, 4><<<dim3(n_rows), dim3(threads), row, stream>>>(A);        \
    else streams_kernel<S_, 1><<<dim3(n_rows), dim3(threads), row, stream>>>(A);            \
    break
  switch (S) {
    GO(1); GO(2); GO(3); GO(4); GO(5); GO(6); GO(7); GO(8);
    default:
      streams_any_kernel<<<dim3(n_rows), dim3(ANY_THREADS), any_lds, stream>>>(A, S);
  }
#undef GO
  return ms_launch_status();
}
