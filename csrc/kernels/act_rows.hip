// Activations over strided rows (the producer's and the consumer's buffers are column slices of wider ones).
// MODE 0: y = gelu(x), exact (erf) form; 1: y = silu(g) * u * s with [g | u] side by side in a row and an
// optional number s per row; 2: y = gelu_tanh(g) * u; 3: y = tanh(x); 4: y = max(x, 0)^2;
// 5: y = cap tanh(x / cap). An optional bias per input column. x and y may be the same.
#include "common.h"

namespace {

template <typename E> __device__ __forceinline__ float to_f(E v);
template <> __device__ __forceinline__ float to_f<float>(float v) { return v; }
template <> __device__ __forceinline__ float to_f<bf16_t>(bf16_t v) { return bf2f(v); }
template <typename E> __device__ __forceinline__ E from_f(float v);
template <> __device__ __forceinline__ float from_f<float>(float v) { return v; }
template <> __device__ __forceinline__ bf16_t from_f<bf16_t>(float v) { return f2bf(v); }

template <typename E, int V>
struct alignas(sizeof(E) * V) Pack { E v[V]; };

template <typename E>
__device__ __forceinline__ float tanh_t(float u) {
  if constexpr (sizeof(E) == 4) return tanhf(u);
  else return fast_tanh(u);
}

template <typename E, int V, int MODE>
__global__ void __launch_bounds__(256) act_rows_kernel(const E* x, long long ldx, const float* rs, const E* bias, E* y,
                                                       long long ldy, int T, int F, float cap) {
  constexpr bool GATED = MODE == 1 || MODE == 2;
  const int per = F / V;
  const long long n = (long long)T * per;
  for (long long i = (long long)blockIdx.x * 256 + threadIdx.x; i < n; i += (long long)gridDim.x * 256) {
    const int t = (int)(i / per), c = (int)(i - (long long)t * per) * V;
    const E* src = x + t * ldx + c;
    const Pack<E, V> a = *reinterpret_cast<const Pack<E, V>*>(src);
    Pack<E, V> o;
    float g[V], u[V];
#pragma unroll
    for (int e = 0; e < V; ++e) g[e] = to_f<E>(a.v[e]);
    if constexpr (GATED) {
      const Pack<E, V> w = *reinterpret_cast<const Pack<E, V>*>(src + F);
#pragma unroll
      for (int e = 0; e < V; ++e) u[e] = to_f<E>(w.v[e]);
    }
    if (bias) {
      const Pack<E, V> b = *reinterpret_cast<const Pack<E, V>*>(bias + c);
#pragma unroll
      for (int e = 0; e < V; ++e) g[e] += to_f<E>(b.v[e]);
      if constexpr (GATED) {
        const Pack<E, V> w = *reinterpret_cast<const Pack<E, V>*>(bias + F + c);
#pragma unroll
        for (int e = 0; e < V; ++e) u[e] += to_f<E>(w.v[e]);
      }
    }
    const float s = GATED && rs ? rs[t] : 1.f;
#pragma unroll
    for (int e = 0; e < V; ++e) {
      float v;
      if constexpr (MODE == 0) v = 0.5f * g[e] * (1.f + erff(g[e] * 0.70710678118654752f));
      else if constexpr (MODE == 1) v = g[e] / (1.f + (sizeof(E) == 4 ? expf(-g[e]) : __expf(-g[e]))) * u[e] * s;
      else if constexpr (MODE == 2)
        v = 0.5f * g[e] * (1.f + tanh_t<E>(0.7978845608028654f * (g[e] + 0.044715f * g[e] * g[e] * g[e]))) * u[e] * s;
      else if constexpr (MODE == 3) v = tanh_t<E>(g[e]);
      else if constexpr (MODE == 4) v = fmaxf(g[e], 0.f) * fmaxf(g[e], 0.f);
      else v = cap * tanh_t<E>(g[e] / cap);
      o.v[e] = from_f<E>(v);
    }
    *reinterpret_cast<Pack<E, V>*>(y + t * ldy + c) = o;
  }
}

template <typename E, int V>
void go(int mode, const void* x, long long ldx, const void* rs, const void* bias, void* y, long long ldy, int T, int F,
        float cap, hipStream_t s) {
  const int g = kca_grid((long long)T * (F / V), 256);
#define GO(M)                                                                                                          \
  hipLaunchKernelGGL((act_rows_kernel<E, V, M>), dim3(g), dim3(256), 0, s, (const E*)x, ldx, (const float*)rs,         \
                     (const E*)bias, (E*)y, ldy, T, F, cap)
  if (mode == 0) GO(0);
  else if (mode == 1) GO(1);
  else if (mode == 2) GO(2);
  else if (mode == 3) GO(3);
  else if (mode == 4) GO(4);
  else GO(5);
#undef GO
}

}  // namespace

// dtype: 0 fp32, 1 bf16
KCA_API int kca_act_rows(int dtype, int mode, const void* x, long long ldx, const void* rs, const void* bias, void* y,
                         long long ldy, int T, int F, float cap, hipStream_t s) {
  if (mode < 0 || mode > 5 || (mode == 5 && !(cap > 0.f))) return 1;
  const bool gated = mode == 1 || mode == 2;
  if (T < 1 || F < 1 || !x || !y || ldx < (gated ? 2LL : 1LL) * F || ldy < F) return 1;
  const int V = dtype == 0 ? 4 : 8;
  const bool v = F % V == 0 && ldx % V == 0 && ldy % V == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)y % 16 == 0 &&
                 (uintptr_t)bias % 16 == 0;
  if (dtype == 0) v ? go<float, 4>(mode, x, ldx, rs, bias, y, ldy, T, F, cap, s) : go<float, 1>(mode, x, ldx, rs, bias, y, ldy, T, F, cap, s);
  else if (dtype == 1)
    v ? go<bf16_t, 8>(mode, x, ldx, rs, bias, y, ldy, T, F, cap, s) : go<bf16_t, 1>(mode, x, ldx, rs, bias, y, ldy, T, F, cap, s);
  else return 3;
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
