// Element access shared by the one-query-per-row attention kernels over the paged cache (diff_attn.hip,
// biased_attn.hip): fp32 or bf16, eight elements a lane.
#pragma once
#include "attn_tile.h"

namespace {

template <typename E> struct El;
template <> struct El<bf16_t> {
  static __device__ __forceinline__ float ld(const bf16_t* p) { return bf2f(*p); }
  static __device__ __forceinline__ void st(bf16_t* p, float v) { *p = f2bf(v); }
  static __device__ __forceinline__ float ex(float x) { return __expf(x); }
};
template <> struct El<float> {
  static __device__ __forceinline__ float ld(const float* p) { return *p; }
  static __device__ __forceinline__ void st(float* p, float v) { *p = v; }
  static __device__ __forceinline__ float ex(float x) { return expf(x); }
};

// eight elements as loaded (converted where they are used); `left` of them exist
template <typename E>
struct Raw8 {
  E v[8];
  __device__ __forceinline__ float f(int i) const { return El<E>::ld(v + i); }
};
template <typename E, bool VEC>
__device__ __forceinline__ void ld8g(const E* p, int left, Raw8<E>& x) {
  if constexpr (VEC) {
    u32x4* d = reinterpret_cast<u32x4*>(x.v);
#pragma unroll
    for (int i = 0; i < (int)sizeof(E) / 2; ++i)
      d[i] = left > 0 ? reinterpret_cast<const u32x4*>(p)[i] : u32x4{0u, 0u, 0u, 0u};
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i) x.v[i] = i < left ? p[i] : (E)0;
  }
}

static inline int lanes_for(int n) {  // lanes of 8 elements, a power of two
  int l = 8;
  while (l * 8 < n) l *= 2;
  return l;
}

}  // namespace
