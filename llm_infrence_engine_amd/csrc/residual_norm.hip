// Kernels of layers that normalise a sublayer's output before it joins the residual stream:
//   x <- x + w_post * y / sqrt(mean(y^2) + eps)        (y: the sublayer's output, x: the float residual stream)
// fused, when asked, with what the next sublayer reads: the norm h = w_next * x / sqrt(mean(x^2) + eps_next), or, where
// sublayers read the stream as it is, x rounded to the activations' type.  y may come with the routed experts' last sum left to
// do: y[n] = base[n] (if given) + sum_j weight[n, j] part[n top + j].  Without w_post nothing is added: h alone.
// And the small sum that opens a pass over a looped stretch of layers: x <- x (+ kept) (+ vec).
// Everything is float; activations are rounded once on store.
#include "common.h"
#include "api.h"

namespace {

constexpr int MAX_PARTS = 32;     // rows one token's sum is made of, beside the base

template <typename T, int V> struct alignas(sizeof(T) * V) Pack { T v[V]; };

// One block per row, V neighbouring columns to a thread and step.  The row of y (then of x) is kept in LDS when it fits
// (`staged`), else worked out again from memory.
template <typename TY, typename TO, int V>
__global__ void __launch_bounds__(1024)
rms_norm_add_kernel(const TY* __restrict__ y, size_t y_stride, const float* __restrict__ parts,
                    const float* __restrict__ part_weights, int top, const float* __restrict__ w_post, float eps_post,
                    float* __restrict__ x, const float* __restrict__ w_next, float eps_next, TO* __restrict__ out, int H,
                    int staged) {
  __shared__ float red[16];
  __shared__ float s_w[MAX_PARTS];
  extern __shared__ __align__(16) float buf[];
  const int r = blockIdx.x;
  const TY* yr = y ? y + (size_t)r * y_stride : nullptr;
  const float* pr = parts ? parts + (size_t)r * top * H : nullptr;
  float* xr = x + (size_t)r * H;
  typedef Pack<float, V> F;
  if (pr) {
    if ((int)threadIdx.x < top) s_w[threadIdx.x] = part_weights[(size_t)r * top + threadIdx.x];
    __syncthreads();
  }
  auto y_at = [&](int i) {
    F v;
    if (yr) {
      const Pack<TY, V> p = *reinterpret_cast<const Pack<TY, V>*>(yr + i);
#pragma unroll
      for (int j = 0; j < V; ++j) v.v[j] = to_float(p.v[j]);
    } else {
#pragma unroll
      for (int j = 0; j < V; ++j) v.v[j] = 0.f;
    }
    if (pr)
      for (int k = 0; k < top; ++k) {
        const F p = *reinterpret_cast<const F*>(pr + (size_t)k * H + i);
        const float w = s_w[k];
#pragma unroll
        for (int j = 0; j < V; ++j) v.v[j] = fmaf(w, p.v[j], v.v[j]);
      }
    return v;
  };
  const int step = blockDim.x * V;
  float s2 = 0.f;
  if (w_post) {
    float ss = 0.f;
    for (int i = threadIdx.x * V; i < H; i += step) {
      const F v = y_at(i);
      if (staged) *reinterpret_cast<F*>(buf + i) = v;
#pragma unroll
      for (int j = 0; j < V; ++j) ss = fmaf(v.v[j], v.v[j], ss);
    }
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)H + eps_post);
    const bool plain = out != nullptr && w_next == nullptr;
    for (int i = threadIdx.x * V; i < H; i += step) {
      const F v = staged ? *reinterpret_cast<const F*>(buf + i) : y_at(i);
      const F w = *reinterpret_cast<const F*>(w_post + i);
      F nx = *reinterpret_cast<const F*>(xr + i);
      Pack<TO, V> o;
#pragma unroll
      for (int j = 0; j < V; ++j) {
        nx.v[j] += w.v[j] * (v.v[j] * inv);
        s2 = fmaf(nx.v[j], nx.v[j], s2);
        o.v[j] = from_float<TO>(nx.v[j]);
      }
      *reinterpret_cast<F*>(xr + i) = nx;
      if (plain) *reinterpret_cast<Pack<TO, V>*>(out + (size_t)r * H + i) = o;
      else if (staged) *reinterpret_cast<F*>(buf + i) = nx;
    }
    if (out == nullptr || plain) return;
  } else {
    for (int i = threadIdx.x * V; i < H; i += step) {
      const F nx = *reinterpret_cast<const F*>(xr + i);
      if (w_next == nullptr) {
        Pack<TO, V> o;
#pragma unroll
        for (int j = 0; j < V; ++j) o.v[j] = from_float<TO>(nx.v[j]);
        *reinterpret_cast<Pack<TO, V>*>(out + (size_t)r * H + i) = o;
        continue;
      }
      if (staged) *reinterpret_cast<F*>(buf + i) = nx;
#pragma unroll
      for (int j = 0; j < V; ++j) s2 = fmaf(nx.v[j], nx.v[j], s2);
    }
    if (w_next == nullptr) return;
  }
  s2 = block_sum(s2, red);
  const float inv2 = 1.0f / sqrtf(s2 / (float)H + eps_next);
  for (int i = threadIdx.x * V; i < H; i += step) {
    const F v = staged ? *reinterpret_cast<const F*>(buf + i) : *reinterpret_cast<const F*>(xr + i);
    const F w = *reinterpret_cast<const F*>(w_next + i);
    Pack<TO, V> o;
#pragma unroll
    for (int j = 0; j < V; ++j) o.v[j] = from_float<TO>(w.v[j] * (v.v[j] * inv2));
    *reinterpret_cast<Pack<TO, V>*>(out + (size_t)r * H + i) = o;
  }
}

__global__ void add_rows_kernel(float* __restrict__ x, const float* __restrict__ kept, const float* __restrict__ vec,
                                size_t total, int H) {
  const size_t stride = (size_t)gridDim.x * blockDim.x;
  for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += stride) {
    float v = x[i];
    if (kept) v += kept[i];
    if (vec) v += vec[i % H];
    x[i] = v;
  }
}

}  // namespace

extern "C" int ms_rms_norm_add(const void* y, long long y_stride, int y_dtype, const float* parts, const float* part_weights,
                               int top, const float* w_post, float eps_post, float* x, const float* w_next, float eps_next,
                               void* out, int out_dtype, int n_rows, int hidden, hipStream_t stream) {
  if (n_rows <= 0) return MS_OK;
  if (hidden <= 0 || x == nullptr) return MS_BAD_ARG;
  if (w_post != nullptr ? (y == nullptr && parts == nullptr) : (y != nullptr || parts != nullptr || out == nullptr)) return MS_BAD_ARG;
  if (parts != nullptr && (part_weights == nullptr || top <= 0)) return MS_BAD_ARG;
  if (parts != nullptr && top > MAX_PARTS) return MS_UNSUPPORTED;
  const int staged = hidden <= 12288;
  const size_t lds = staged ? (size_t)hidden * sizeof(float) : 0;
  const uintptr_t all = (uintptr_t)y | (uintptr_t)parts | (uintptr_t)w_post | (uintptr_t)x | (uintptr_t)w_next | (uintptr_t)out;
  const bool wide = hidden % 4 == 0 && all % 16 == 0 && (y == nullptr || y_stride % 4 == 0);
  // few rows: more threads to a row, as there are units to spare
  dim3 grid(n_rows), block(wide && n_rows <= 128 && hidden >= 2048 ? 512 : 256);
#define LAUNCH(TY, TO, V)                                                                                            \
  rms_norm_add_kernel<TY, TO, V><<<grid, block, lds, stream>>>((const TY*)y, (size_t)y_stride, parts, part_weights, top, \
                                                               w_post, eps_post, x, w_next, eps_next, (TO*)out, hidden, staged)
#define LAUNCH_V(TY, TO) do { if (wide) LAUNCH(TY, TO, 4); else LAUNCH(TY, TO, 1); } while (0)
  if (y_dtype == MS_F32 && out_dtype == MS_F32) LAUNCH_V(float, float);
  else if (y_dtype == MS_F32 && out_dtype == MS_BF16) LAUNCH_V(float, bf16);
  else if (y_dtype == MS_BF16 && out_dtype == MS_F32) LAUNCH_V(bf16, float);
  else if (y_dtype == MS_BF16 && out_dtype == MS_BF16) LAUNCH_V(bf16, bf16);
  else return MS_BAD_ARG;
#undef LAUNCH_V
#undef LAUNCH
  return ms_launch_status();
}

extern "C" int ms_add_rows(float* x, const float* kept, const float* vec, int n_rows, int hidden, hipStream_t stream) {
  if (n_rows <= 0) return MS_OK;
  if (hidden <= 0) return MS_BAD_ARG;
  const size_t total = (size_t)n_rows * hidden;
  int blocks = (int)((total + 1023) / 1024);
  if (blocks > 4096) blocks = 4096;
  add_rows_kernel<<<blocks, 256, 0, stream>>>(x, kept, vec, total, hidden);
  return ms_launch_status();
}
