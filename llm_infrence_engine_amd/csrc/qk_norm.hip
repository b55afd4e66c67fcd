// What lies between the packed q/k/v projection and attention for heads that are normalised instead of rotated:
// the RMS norm of every query and key head (one weight per entry, shared by the heads), a query temperature that
// grows with the logarithm of the position,
//   q <- q * (1 + coef * ln(floor((p + 1) / every) + 1)),
// optionally a rotation of the first rot_dim entries of every q and k head (entry i with entry i + rot_dim / 2, by the
// angle position * inv_freq[i], after the norm), and the store of k and v into the cache pages.  `unit_norm`: heads are
// divided by their root mean square even where no weight is given.  Keys and values may have different sizes.
// qkv [N, nh * d + nkv * d + nkv * dv]; q and k are rewritten in place.  Norms, logarithm, temperature, angles, sines
// and cosines are float.
//
// ms_qk_span_norm_store: the same place for norms that run over the whole projection: all q heads of a token are divided by
// one root mean square and multiplied by one weight per entry of the projection, all k heads by another; then the rotation
// and the store.  Values may be blended on their way into the pages, v <- (1 - lambda) v + lambda first, with another
// matrix's row of the same token (`first`) and one stored number lambda; the projection's own v stays as it is.
#include "common.h"
#include "api.h"

namespace {

constexpr int MAX_HEAD = 256;   // the longest head the rotation can hold in LDS (the attention kernels' own limit)

template <typename T>
__global__ void __launch_bounds__(256)
qk_norm_store_kernel(T* __restrict__ qkv, size_t stride, const float* __restrict__ q_w, const float* __restrict__ k_w,
                     float eps, const int* __restrict__ positions, float coef, int every,
                     const int* __restrict__ slots, T* __restrict__ k_pages, T* __restrict__ v_pages, long long items,
                     int nh, int nkv, int d, int dv, int page_size, int v_transposed, int unit_norm,
                     const float* __restrict__ inv_freq, int rot_dim) {
  __shared__ float head[4][MAX_HEAD];
  const int wave = threadIdx.x / MS_WAVE;
  const int lane = threadIdx.x & (MS_WAVE - 1);
  const long long item = (long long)blockIdx.x * (blockDim.x / MS_WAVE) + threadIdx.x / MS_WAVE;
  if (item >= items) return;
  const int per_token = nh + 2 * nkv;
  const long long n = item / per_token;
  const int h = (int)(item - n * per_token);
  T* row = qkv + (size_t)n * stride;
  const int slot = slots ? slots[n] : -1;
  if (h < nh + nkv) {
    const bool is_q = h < nh;
    T* p = row + (size_t)h * d;   // k heads follow the q heads at the same width
    const float* w = is_q ? q_w : k_w;
    float mult = 1.f;
    if (w || unit_norm) {
      float ss = 0.f;
      for (int i = lane; i < d; i += MS_WAVE) { const float v = to_float(p[i]); ss = fmaf(v, v, ss); }
      ss = wave_sum(ss);
      mult = 1.0f / sqrtf(ss / (float)d + eps);
    }
    float temp = 1.f;
    if (is_q && coef != 0.f) temp = 1.0f + coef * logf((float)((positions[n] + 1) / every + 1));
    T* kp = nullptr;
    if (!is_q && k_pages && slot >= 0) {
      const int page = slot / page_size, off = slot % page_size;
      kp = k_pages + (((size_t)page * nkv + (h - nh)) * page_size + off) * d;
    }
    if (rot_dim > 0) {
      // the normed head waits in LDS: the two entries of a pair may belong to different lanes
      for (int i = lane; i < d; i += MS_WAVE) {
        float v = to_float(p[i]) * mult;
        if (w) v *= w[i];
        head[wave][i] = v * temp;
      }
      __builtin_amdgcn_wave_barrier();
      const int half = rot_dim / 2;
      const float pos = (float)positions[n];
      for (int i = lane; i < d; i += MS_WAVE) {
        float v = head[wave][i];
        if (i < rot_dim) {
          const int j = i < half ? i : i - half;
          float sn, cs;
          sincosf(pos * inv_freq[j], &sn, &cs);
          v = i < half ? head[wave][i] * cs - head[wave][i + half] * sn : head[wave][i] * cs + head[wave][i - half] * sn;
        }
        const T r = from_float<T>(v);
        p[i] = r;
        if (kp) kp[i] = r;
      }
    } else {
      for (int i = lane; i < d; i += MS_WAVE) {
        float v = to_float(p[i]) * mult;
        if (w) v *= w[i];
        const T r = from_float<T>(v * temp);
        p[i] = r;
        if (kp) kp[i] = r;
      }
    }
  } else if (v_pages && slot >= 0) {
    const int g = h - nh - nkv;
    const T* p = row + (size_t)(nh + nkv) * d + (size_t)g * dv;
    const int page = slot / page_size, off = slot % page_size;
    if (v_transposed) {
      T* vp = v_pages + ((size_t)page * nkv + g) * dv * page_size + off;
      for (int i = lane; i < dv; i += MS_WAVE) vp[(size_t)i * page_size] = p[i];
    } else {
      T* vp = v_pages + (((size_t)page * nkv + g) * page_size + off) * dv;
      for (int i = lane; i < dv; i += MS_WAVE) vp[i] = p[i];
    }
  }
}

// One block per token, V neighbouring entries of a head to a thread and step (V = 8: heads, halves of the rotated part and
// rows are whole pieces of 16 bytes in bfloat16).  q and k wait in LDS, as floats, between the sums and the rotation.
template <typename T, int V> struct alignas(sizeof(T) * V < 16 ? sizeof(T) * V : 16) Piece { T v[V]; };

template <typename T, int V>
__global__ void __launch_bounds__(512)
qk_span_norm_store_kernel(T* __restrict__ qkv, size_t stride, const float* __restrict__ q_w, const float* __restrict__ k_w,
                          float eps, const int* __restrict__ positions, const float* __restrict__ inv_freq, int rot_dim,
                          const T* __restrict__ first, size_t first_stride, const float* __restrict__ lambda,
                          const int* __restrict__ slots, T* __restrict__ k_pages, T* __restrict__ v_pages, int nh, int nkv,
                          int d, int dv, int page_size, int v_transposed) {
  extern __shared__ __align__(16) float s_mem[];     // [rot_dim] cosines, sines; then q and k, [(nh + nkv) * d]
  __shared__ float red[16];
  float* cs = s_mem;
  float* sn = s_mem + rot_dim / 2;
  float* row_f = s_mem + rot_dim + (4 - rot_dim % 4) % 4;
  const int n = blockIdx.x, tid = threadIdx.x;
  T* row = qkv + (size_t)n * stride;
  const int nq = nh * d, nk = nkv * d, half = rot_dim / 2;
  typedef Piece<T, V> P;
  typedef Piece<float, V> F;
  if (rot_dim > 0) {
    const float pos = (float)positions[n];
    for (int i = tid; i < half; i += blockDim.x) sincosf(pos * inv_freq[i], &sn[i], &cs[i]);
  }
  float sq = 0.f, sk = 0.f;
  for (int i = tid * V; i < nq + nk; i += blockDim.x * V) {
    const P p = *reinterpret_cast<const P*>(row + i);
    F f;
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < V; ++j) { f.v[j] = to_float(p.v[j]); ss = fmaf(f.v[j], f.v[j], ss); }
#pragma unroll
    for (int j = 0; j < V; ++j) row_f[i + j] = f.v[j];
    if (i < nq) sq += ss; else sk += ss;
  }
  sq = block_sum(sq, red);
  sk = block_sum(sk, red);       // (its barriers also stand between the rows' writes to LDS and their reads)
  const float iq = 1.0f / sqrtf(sq / (float)nq + eps), ik = 1.0f / sqrtf(sk / (float)nk + eps);
  const int slot = slots ? slots[n] : -1;
  const int page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
  for (int i = tid * V; i < nq + nk; i += blockDim.x * V) {
    const bool is_q = i < nq;
    const int at = is_q ? i : i - nq;       // entry of its projection, head and entry of its head
    const int head = at / d, e = at - head * d;
    const float inv = is_q ? iq : ik;
    const float* w = (is_q ? q_w : k_w) + at;
    F v;
#pragma unroll
    for (int j = 0; j < V; ++j) v.v[j] = row_f[i + j] * inv * w[j];
    if (e < rot_dim) {                      // (V > 1: a piece lies in one half)
      const bool low = e < half;
      const int other = low ? half : -half, pair = low ? e : e - half;
#pragma unroll
      for (int j = 0; j < V; ++j) {
        const float o = row_f[i + other + j] * inv * w[other + j];
        const float c = cs[pair + j], s = sn[pair + j];
        v.v[j] = low ? v.v[j] * c - o * s : v.v[j] * c + o * s;
      }
    }
    P p;
#pragma unroll
    for (int j = 0; j < V; ++j) p.v[j] = from_float<T>(v.v[j]);
    *reinterpret_cast<P*>(row + i) = p;
    if (!is_q && k_pages && slot >= 0)
      *reinterpret_cast<P*>(k_pages + (((size_t)page * nkv + head) * page_size + off) * d + e) = p;
  }
  if (v_pages && slot >= 0) {
    const T* vr = row + nq + nk;
    const T* fr = first ? first + (size_t)n * first_stride : nullptr;
    const float lam = first ? *lambda : 0.f;
    for (int i = tid; i < nkv * dv; i += blockDim.x) {
      T v = vr[i];
      if (fr) v = from_float<T>(fmaf(lam, to_float(fr[i]), (1.0f - lam) * to_float(v)));
      const int g = i / dv, e = i - g * dv;
      if (v_transposed) v_pages[(((size_t)page * nkv + g) * dv + e) * page_size + off] = v;
      else v_pages[(((size_t)page * nkv + g) * page_size + off) * dv + e] = v;
    }
  }
}

}  // namespace

extern "C" int ms_qk_norm_store(void* qkv, long long stride, const float* q_weight, const float* k_weight, float eps,
                                const int* positions, float coef, int every, const int* slots, void* k_pages,
                                void* v_pages, int n_tokens, int num_heads, int num_kv_heads, int head_dim, int value_dim,
                                int page_size, int v_transposed, int unit_norm, const float* inv_freq, int rot_dim, int dtype,
                                hipStream_t stream) {
  if (n_tokens <= 0) return MS_OK;
  if (num_heads <= 0 || num_kv_heads <= 0 || head_dim <= 0 || value_dim <= 0) return MS_BAD_ARG;
  if (coef != 0.f && (positions == nullptr || every <= 0)) return MS_BAD_ARG;
  if (rot_dim < 0 || rot_dim % 2 || rot_dim > head_dim || (rot_dim > 0 && (positions == nullptr || inv_freq == nullptr)))
    return MS_BAD_ARG;
  if (rot_dim > 0 && head_dim > MAX_HEAD) return MS_UNSUPPORTED;
  if ((k_pages != nullptr) != (v_pages != nullptr) || (k_pages != nullptr && (slots == nullptr || page_size <= 0)))
    return MS_BAD_ARG;
  const long long items = (long long)n_tokens * (num_heads + 2 * num_kv_heads);
  const int waves = 4;
  dim3 grid((unsigned)((items + waves - 1) / waves)), block(waves * MS_WAVE);
#define LAUNCH(T)                                                                                                    \
  qk_norm_store_kernel<T><<<grid, block, 0, stream>>>((T*)qkv, (size_t)stride, q_weight, k_weight, eps, positions,  \
                                                      coef, every, slots, (T*)k_pages, (T*)v_pages, items, num_heads, \
                                                      num_kv_heads, head_dim, value_dim, page_size, v_transposed, unit_norm, \
                                                      inv_freq, rot_dim)
  if (dtype == MS_F32) LAUNCH(float);
  else if (dtype == MS_BF16) LAUNCH(bf16);
  else return MS_BAD_ARG;
#undef LAUNCH
  return ms_launch_status();
}

// q_weight float [nh * d], k_weight float [nkv * d]; first: rows of [nkv * dv] (first_stride apart) and lambda a float on the
// device, or null.  q and k of one token must fit in LDS as floats.
extern "C" int ms_qk_span_norm_store(void* qkv, long long stride, const float* q_weight, const float* k_weight, float eps,
                                     const int* positions, const float* inv_freq, int rot_dim, const void* first,
                                     long long first_stride, const float* lambda, const int* slots, void* k_pages,
                                     void* v_pages, int n_tokens, int num_heads, int num_kv_heads, int head_dim,
                                     int value_dim, int page_size, int v_transposed, int dtype, hipStream_t stream) {
  if (n_tokens <= 0) return MS_OK;
  if (num_heads <= 0 || num_kv_heads <= 0 || head_dim <= 0 || value_dim <= 0 || !q_weight || !k_weight) return MS_BAD_ARG;
  if (rot_dim < 0 || rot_dim % 2 || rot_dim > head_dim || (rot_dim > 0 && (positions == nullptr || inv_freq == nullptr)))
    return MS_BAD_ARG;
  if ((first != nullptr) != (lambda != nullptr)) return MS_BAD_ARG;
  if ((k_pages != nullptr) != (v_pages != nullptr) || (k_pages != nullptr && (slots == nullptr || page_size <= 0)))
    return MS_BAD_ARG;
  const size_t lds = ((size_t)(num_heads + num_kv_heads) * head_dim + rot_dim + 4) * sizeof(float);
  if (lds > 60 * 1024) return MS_UNSUPPORTED;
  const uintptr_t all = (uintptr_t)qkv | (uintptr_t)k_pages;
  const bool wide = head_dim % 8 == 0 && (rot_dim / 2) % 8 == 0 && stride % 8 == 0 && all % 16 == 0;
  dim3 grid(n_tokens), block(n_tokens <= 256 ? 512 : 256);
#define LAUNCH(T, V)                                                                                                      \
  qk_span_norm_store_kernel<T, V><<<grid, block, lds, stream>>>((T*)qkv, (size_t)stride, q_weight, k_weight, eps,       \
                                                                positions, inv_freq, rot_dim, (const T*)first,          \
                                                                (size_t)first_stride, lambda, slots, (T*)k_pages,       \
                                                                (T*)v_pages, num_heads, num_kv_heads, head_dim,         \
                                                                value_dim, page_size, v_transposed)
  if (dtype == MS_F32) { if (wide) LAUNCH(float, 8); else LAUNCH(float, 1); }
  else if (dtype == MS_BF16) { if (wide) LAUNCH(bf16, 8); else LAUNCH(bf16, 1); }
  else return MS_BAD_ARG;
#undef LAUNCH
  return ms_launch_status();
}
