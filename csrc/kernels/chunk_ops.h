// Matrix-core pieces shared by the chunked recurrences over prompt portions (delta_chunk.hip, ssd_chunk.hip).
#pragma once
#include "attn_tile.h"

namespace {

constexpr int CT = 64;   // tokens of a chunk

__device__ __forceinline__ f32x4 mm32(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
// 16 x 16 x 16 in fp32: a = four consecutive elements of row lane & 15 from column 4 (lane >> 4), b in the
// accumulators' layout (rows 4 (lane >> 4) + r of column lane & 15)
__device__ __forceinline__ f32x4 mm16f(float4 a, f32x4 b, f32x4 c) {
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b[0], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b[1], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b[2], c, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b[3], c, 0, 0, 0);
}
typedef float f32x2 __attribute__((ext_vector_type(2)));
typedef __bf16 bf16x2v __attribute__((ext_vector_type(2)));
__device__ __forceinline__ uint32_t pk2(float lo, float hi) {  // one v_cvt_pk
  return __builtin_bit_cast(uint32_t, __builtin_convertvector(f32x2{lo, hi}, bf16x2v));
}
__device__ __forceinline__ s16x4 pk4(f32x4 v) {
  const uint2 u = make_uint2(pk2(v[0], v[1]), pk2(v[2], v[3]));
  return __builtin_bit_cast(s16x4, u);
}
// operands of two token blocks side by side: the matrix instruction's 8 slots of a lane group hold its four
// tokens of either block, on both sides alike
__device__ __forceinline__ bf16x8 two(s16x4 a, s16x4 b) {
  return __builtin_bit_cast(bf16x8, __builtin_shufflevector(a, b, 0, 1, 2, 3, 4, 5, 6, 7));
}
// one block: the other half of the slots zero. (Not the 16-deep instruction: a sum that passes from one bf16 matrix
// instruction to another kind of them, into other registers, came out wrong; one kind throughout does not.)
__device__ __forceinline__ f32x4 mm16(s16x4 a, s16x4 b, f32x4 c) { return mm32(two(a, s16x4{0, 0, 0, 0}), two(b, s16x4{0, 0, 0, 0}), c); }
__device__ __forceinline__ s16x4 neg4(s16x4 v) {
  uint2 u = __builtin_bit_cast(uint2, v);
  u.x ^= 0x80008000u;
  u.y ^= 0x80008000u;
  return __builtin_bit_cast(s16x4, u);
}
// operand of four tokens (rows 4 (lane >> 4) of the block) at column lane & 15 of a row-major LDS image
template <int LD>
__device__ __forceinline__ s16x4 tok4(const bf16_t* img, int row, int col) {
  const int lane = threadIdx.x & 63, gi = lane & 15;
  const bf16_t* p = img + (row + 4 * (lane >> 4) + (gi >> 2)) * LD + col + 4 * (gi & 3);
  return __builtin_bit_cast(s16x4, lds_tr4(reinterpret_cast<const char*>(p), 0));
}
__device__ __forceinline__ s16x4 row4(const bf16_t* p) { return *reinterpret_cast<const s16x4*>(p); }
__device__ __forceinline__ f32x4 up4(s16x4 v) {
  const uint2 u = __builtin_bit_cast(uint2, v);
  return f32x4{__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
               __uint_as_float(u.y & 0xffff0000u)};
}

}  // namespace
