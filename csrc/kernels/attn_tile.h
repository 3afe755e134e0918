// LDS tile image and fragment reads shared by the matrix-core attention kernels (attention_tiled.hip,
// diff_attn.hip): a 32-row x D bf16 tile as 8-row x 32-column sub-tiles of 512 B, conflict-free for both
// the ds_read_b128 row reads of S^T = K.Q^T and the ds_read_b64_tr_b16 reads of O^T += V^T.P^T.
#pragma once
#include "common.h"

constexpr float kLog2e = 1.4426950408889634f;
constexpr float kLn2 = 0.6931471805599453f;
constexpr float kRescaleThr = 8.0f;

typedef __attribute__((address_space(3))) bf16x4 lds_bf16x4_t;
typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ bf16x4 lds_tr4(const char* base, int byte_off) {
  return __builtin_amdgcn_ds_read_tr16_b64_v4bf16(
      (lds_bf16x4_t*)(reinterpret_cast<uintptr_t>(base + byte_off)));
}

__device__ __forceinline__ bf16x8 lds_b128(const char* base, int byte_off) {
  return *reinterpret_cast<const bf16x8*>(base + byte_off);
}

// byte offset of 16-B chunk `ch` of row `row` in a [32][D] image (see header)
template <int D>
__device__ __forceinline__ int img_off(int row, int ch) {
  return (row >> 3) * 16 * D + 512 * (ch >> 2) + 64 * (row & 7) + 16 * ((ch & 3) ^ ((row >> 2) & 3));
}

__device__ __forceinline__ bf16x8 cat8(bf16x4 a, bf16x4 b) {
  return __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7);
}

__device__ __forceinline__ uint32_t pk_bf16(float lo, float hi) {
  return pack_bf16x2(lo, hi);
}
