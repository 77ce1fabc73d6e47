// Hyper-connections (ops/hyper.py): a residual state of several float32 streams X [T, S, W].
//
//   hc_embed_kernel   every stream = table[id] * scale
//   hc_step_kernel    one launch between two sublayers, a workgroup per token:
//       write   y = coef * (f(o, w1) + f(o2, w2)), f(o, w) = o / sqrt(mean(o^2) + eps) * w when w is given and o
//               itself otherwise (o2 null: one term);  x_t <- sum_s mix[s, t] x_s + out[t] y, all streams at
//               once from the old ones
//       read    u = sum_s in[s] x_s;  h = u / sqrt(mean(u^2) + eps) * gain (a scalar), the next sublayer's input
//     either half may be left out.  A lane owns V consecutive columns of every stream: the S old values sit in
//     its registers, the new ones leave as they are made and u waits in LDS for the row's mean square, so the
//     streams are read and written once (2 x 4 S W bytes per token, the bound of the kernel).
//
// Templates over the activation type T (bf16 or float), the columns per lane V and the streams: exact builds for
// 1 .. 4, guarded ones for up to 8 and 16.
#include <math.h>

#include "common.h"
#include "launchers.h"
#include "stream_common.h"

namespace dllm {

template <typename T, int V>
__global__ void __launch_bounds__(256) hc_embed_kernel(float* __restrict__ x, const int32_t* __restrict__ ids,
                                                       const void* __restrict__ table_, int streams, int width, int vocab,
                                                       float scale) {
  int id = ids[blockIdx.x];
  id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
  const T* src = (const T*)table_ + (size_t)id * width;
  float* dst = x + (size_t)blockIdx.x * streams * width;
  for (int i = threadIdx.x * V; i < width; i += 256 * V) {
    float v[V];
    ldv<V>(src + i, v);
#pragma unroll
    for (int j = 0; j < V; ++j) v[j] *= scale;
    for (int s = 0; s < streams; ++s) stv<V>(dst + (size_t)s * width + i, v);
  }
}

void hc_embed(uintptr_t x, uintptr_t ids, uintptr_t table, int tokens, int streams, int width, int vocab, float scale,
              int f32, uintptr_t stream) {
  if (tokens <= 0) return;
  DLLM_HOST_CHECK(streams > 0 && width > 0 && vocab > 0 && x && ids && table, "hyper-connection embedding arguments");
  const bool vec = width % 4 == 0 && x % 16 == 0 && table % (f32 ? 16 : 8) == 0;
#define HC_EMBED(T, V)                                                                                               \
  hipLaunchKernelGGL(HIP_KERNEL_NAME(hc_embed_kernel<T, V>), dim3(tokens), dim3(256), 0, (hipStream_t)stream, (float*)x, \
                     (const int32_t*)ids, (const void*)table, streams, width, vocab, scale)
  if (f32) { if (vec) HC_EMBED(float, 4); else HC_EMBED(float, 1); }
  else { if (vec) HC_EMBED(bf16, 4); else HC_EMBED(bf16, 1); }
#undef HC_EMBED
  DLLM_HIP_CHECK(hipGetLastError());
}

template <typename T, int V, int S, bool EXACT>
__global__ void __launch_bounds__(256) hc_step_kernel(float* __restrict__ x, const float* __restrict__ mix,
                                                      const float* __restrict__ out_w, const void* __restrict__ o_,
                                                      const void* __restrict__ w1_, const void* __restrict__ o2_,
                                                      const void* __restrict__ w2_, float coef,
                                                      const float* __restrict__ in_w, float gain, void* __restrict__ h_,
                                                      int streams, int width, float eps) {
  __shared__ float red[16];
  extern __shared__ float us[];                     // u of the row [width]
  const int ns = EXACT ? S : streams;
  const size_t row = blockIdx.x;
  const T* o = o_ ? (const T*)o_ + row * width : nullptr;
  const T* o2 = o2_ ? (const T*)o2_ + row * width : nullptr;
  const T* w1 = (const T*)w1_;
  const T* w2 = (const T*)w2_;
  float* xr = x + row * ns * width;
  float inv1 = 1.f, inv2 = 1.f;
  if (w1 || (o2 && w2)) {
    float s1 = 0.f, s2 = 0.f;
    for (int i = threadIdx.x * V; i < width; i += 256 * V) {
      float v[V];
      if (w1) {
        ldv<V>(o + i, v);
#pragma unroll
        for (int j = 0; j < V; ++j) s1 += v[j] * v[j];
      }
      if (o2 && w2) {
        ldv<V>(o2 + i, v);
#pragma unroll
        for (int j = 0; j < V; ++j) s2 += v[j] * v[j];
      }
    }
    if (w1) inv1 = 1.0f / sqrtf(block_sum(s1, red) / (float)width + eps);
    if (o2 && w2) inv2 = 1.0f / sqrtf(block_sum(s2, red) / (float)width + eps);
  }
  float mx[S * S], ow[S], iw[S];                    // uniform over the launch
#pragma unroll
  for (int s = 0; s < S; ++s) {
    if (!EXACT && s >= ns) continue;
    if (o) {
      ow[s] = out_w[s];
      if constexpr (S <= 4) {
#pragma unroll
        for (int t = 0; t < S; ++t) mx[s * S + t] = mix[s * S + t];
      }
    }
    if (h_) iw[s] = in_w[s];
  }
  float sq = 0.f;
  for (int i = threadIdx.x * V; i < width; i += 256 * V) {
    float xv[S][V], u[V];
#pragma unroll
    for (int s = 0; s < S; ++s)
      if (EXACT || s < ns) ldv<V>(xr + (size_t)s * width + i, xv[s]);
#pragma unroll
    for (int j = 0; j < V; ++j) u[j] = 0.f;
    if (o) {
      float y[V], v[V], g[V];
      ldv<V>(o + i, y);
      if (w1) {
        ldv<V>(w1 + i, g);
#pragma unroll
        for (int j = 0; j < V; ++j) y[j] *= inv1 * g[j];
      }
      if (o2) {
        ldv<V>(o2 + i, v);
        if (w2) {
          ldv<V>(w2 + i, g);
#pragma unroll
          for (int j = 0; j < V; ++j) v[j] *= inv2 * g[j];
        }
#pragma unroll
        for (int j = 0; j < V; ++j) y[j] += v[j];
      }
#pragma unroll
      for (int j = 0; j < V; ++j) y[j] *= coef;
#pragma unroll
      for (int t = 0; t < S; ++t) {
        if (!EXACT && t >= ns) continue;
        float n[V];
#pragma unroll
        for (int j = 0; j < V; ++j) n[j] = ow[t] * y[j];
#pragma unroll
        for (int s = 0; s < S; ++s) {
          if (!EXACT && s >= ns) continue;
          float m;
          if constexpr (S <= 4) m = EXACT ? mx[s * S + t] : mix[s * ns + t];
          else m = mix[s * ns + t];
#pragma unroll
          for (int j = 0; j < V; ++j) n[j] = fmaf(m, xv[s][j], n[j]);
        }
        stv<V>(xr + (size_t)t * width + i, n);
        if (h_) {
#pragma unroll
          for (int j = 0; j < V; ++j) u[j] = fmaf(iw[t], n[j], u[j]);
        }
      }
    } else {
#pragma unroll
      for (int s = 0; s < S; ++s) {
        if (!EXACT && s >= ns) continue;
#pragma unroll
        for (int j = 0; j < V; ++j) u[j] = fmaf(iw[s], xv[s][j], u[j]);
      }
    }
    if (h_) {
#pragma unroll
      for (int j = 0; j < V; ++j) sq += u[j] * u[j];
      stv<V>(us + i, u);
    }
  }
  if (!h_) return;
  sq = block_sum(sq, red);
  const float inv = gain / sqrtf(sq / (float)width + eps);
  T* h = (T*)h_ + row * width;
  for (int i = threadIdx.x * V; i < width; i += 256 * V) {      // each lane re-reads what it put into LDS itself
    float u[V];
    ldv<V>(us + i, u);
#pragma unroll
    for (int j = 0; j < V; ++j) u[j] *= inv;
    stv<V>(h + i, u);
  }
}

// x [rows, streams, width] float32 in place; mix [streams, streams] (from, to), out_w / in_w [streams] float32; o, o2, w1,
// w2 and h of the activation type (o null: nothing is written back; h null: nothing is read out).
void hc_step(uintptr_t x, uintptr_t mix, uintptr_t out_w, uintptr_t o, uintptr_t w1, uintptr_t o2, uintptr_t w2, float coef,
             uintptr_t in_w, float gain, uintptr_t h, int rows, int streams, int width, float eps, int f32,
             uintptr_t stream) {
  if (rows <= 0) return;
  DLLM_HOST_CHECK(x && (!o || (mix && out_w)) && (!h || in_w) && (o || h) && (!w1 || o) && (!w2 || o2) && (!o2 || o),
                  "hyper-connection arguments");
  DLLM_HOST_CHECK(streams >= 1 && streams <= 16 && width > 0 && width <= 16384, "hyper-connections: 1 <= streams <= 16, width <= 16384");
  const size_t lds = h ? sizeof(float) * (size_t)width : 0;
  const int esz = f32 ? 4 : 2;
  const bool vec = width % 4 == 0 && x % 16 == 0 && o % (4 * esz) == 0 && o2 % (4 * esz) == 0 && w1 % (4 * esz) == 0 &&
                   w2 % (4 * esz) == 0 && h % (4 * esz) == 0;
  hipStream_t s = (hipStream_t)stream;
#define HC_GO(T, V, S, EXACT)                                                                                          \
  hipLaunchKernelGGL(HIP_KERNEL_NAME(hc_step_kernel<T, V, S, EXACT>), dim3(rows), dim3(256), lds, s, (float*)x,        \
                     (const float*)mix, (const float*)out_w, (const void*)o, (const void*)w1, (const void*)o2,         \
                     (const void*)w2, coef, (const float*)in_w, gain, (void*)h, streams, width, eps)
#define HC_BY_STREAMS(T, V)                           \
  do {                                                \
    if (streams == 1) HC_GO(T, V, 1, true);           \
    else if (streams == 2) HC_GO(T, V, 2, true);      \
    else if (streams == 3) HC_GO(T, V, 3, true);      \
    else if (streams == 4) HC_GO(T, V, 4, true);      \
    else if (streams <= 8) HC_GO(T, V, 8, false);     \
    else HC_GO(T, V, 16, false);                      \
  } while (0)
  if (f32) { if (vec) HC_BY_STREAMS(float, 4); else HC_BY_STREAMS(float, 1); }
  else { if (vec) HC_BY_STREAMS(bf16, 4); else HC_BY_STREAMS(bf16, 1); }
#undef HC_BY_STREAMS
#undef HC_GO
  DLLM_HIP_CHECK(hipGetLastError());
}

}  // namespace dllm
