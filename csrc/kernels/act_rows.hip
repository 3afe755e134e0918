// Feed-forward activations over strided rows (the producer's and the consumer's buffers are column slices
// of wider ones): y = gelu(u), exact (erf) form, or y = silu(g) * u * s with [g | u] side by side in a row
// and an optional number s per row.
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

template <typename E, int V, bool GATED>
__global__ void __launch_bounds__(256) act_rows_kernel(const E* x, long long ldx, const float* rs, E* y, long long ldy,
                                                       int T, int F) {
  const int per = F / V;
  const long long n = (long long)T * per;
  for (long long i = (long long)blockIdx.x * 256 + threadIdx.x; i < n; i += (long long)gridDim.x * 256) {
    const int t = (int)(i / per), c = (int)(i - (long long)t * per) * V;
    const E* src = x + t * ldx + c;
    const Pack<E, V> a = *reinterpret_cast<const Pack<E, V>*>(src);
    Pack<E, V> o;
    if constexpr (GATED) {
      const Pack<E, V> u = *reinterpret_cast<const Pack<E, V>*>(src + F);
      const float s = rs ? rs[t] : 1.f;
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float g = to_f<E>(a.v[e]);
        o.v[e] = from_f<E>(g / (1.f + (sizeof(E) == 4 ? expf(-g) : __expf(-g))) * to_f<E>(u.v[e]) * s);
      }
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float g = to_f<E>(a.v[e]);
        o.v[e] = from_f<E>(0.5f * g * (1.f + erff(g * 0.70710678118654752f)));
      }
    }
    *reinterpret_cast<Pack<E, V>*>(y + t * ldy + c) = o;
  }
}

template <typename E, int V>
void go(int gated, const void* x, long long ldx, const void* rs, void* y, long long ldy, int T, int F, hipStream_t s) {
  const int g = kca_grid((long long)T * (F / V), 256);
  if (gated)
    hipLaunchKernelGGL((act_rows_kernel<E, V, true>), dim3(g), dim3(256), 0, s, (const E*)x, ldx, (const float*)rs,
                       (E*)y, ldy, T, F);
  else
    hipLaunchKernelGGL((act_rows_kernel<E, V, false>), dim3(g), dim3(256), 0, s, (const E*)x, ldx, (const float*)rs,
                       (E*)y, ldy, T, F);
}

}  // namespace

// dtype: 0 fp32, 1 bf16
KCA_API int kca_act_rows(int dtype, int gated, const void* x, long long ldx, const void* rs, void* y, long long ldy,
                         int T, int F, hipStream_t s) {
  if (T < 1 || F < 1 || !x || !y || ldx < (gated ? 2LL : 1LL) * F || ldy < F) return 1;
  const int V = dtype == 0 ? 4 : 8;
  const bool v = F % V == 0 && ldx % V == 0 && ldy % V == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)y % 16 == 0;
  if (dtype == 0) v ? go<float, 4>(gated, x, ldx, rs, y, ldy, T, F, s) : go<float, 1>(gated, x, ldx, rs, y, ldy, T, F, s);
  else if (dtype == 1)
    v ? go<bf16_t, 8>(gated, x, ldx, rs, y, ldy, T, F, s) : go<bf16_t, 1>(gated, x, ldx, rs, y, ldy, T, F, s);
  else return 3;
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
