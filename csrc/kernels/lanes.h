// Reductions over groups of consecutive lanes, and the ordering of one wave's LDS traffic.
#pragma once
#include "common.h"

// sum / maximum over N consecutive lanes (all of them get it): DPP steps within a row of 16
template <int CTRL>
__device__ __forceinline__ float dpp(float x) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), CTRL, 0xf, 0xf, true));
}
template <int N, typename F>
__device__ __forceinline__ float lanes_reduce(float x, F f) {
  static_assert(N == 4 || N == 8 || N == 16 || N == 32 || N == 64, "lanes");
  x = f(x, dpp<0xB1>(x));  // lane ^ 1
  x = f(x, dpp<0x4E>(x));  // lane ^ 2
  if constexpr (N >= 8) x = f(x, dpp<0x141>(x));   // mirrored in 8: the other four
  if constexpr (N >= 16) x = f(x, dpp<0x140>(x));  // mirrored in 16: the other eight
  if constexpr (N >= 32) x = f(x, __shfl_xor(x, 16, 64));
  if constexpr (N >= 64) x = f(x, __shfl_xor(x, 32, 64));
  return x;
}
__device__ __forceinline__ void wave_sync() {  // orders one wave's LDS writes before its later reads
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}
