// Latent attention: every head's keys and values come from one cached latent row per token,
//   row j = [c_j (C, normed) | r_j (R, rotated key part shared by all heads)]
// so that a score is (W_uk^T q)_h . c_j + rot(q_h) . r_j, and a head's output W_uv (sum_j weight_j c_j).
// The softmax's denominator also holds exp(sink_h). Scores, weights, angles and norms are fp32.
#pragma once
#include "common.h"

struct LatentArgs {
  const void* x;            // projection rows [query latent Q at o_q | C + R at o_kv], row stride ld
  long long ld;
  int o_q, o_kv;
  int H, D, R, E, C, Q, nr; // heads, unrotated / rotated query dims, value dims, latent, query latent; nr of R rotate
  const void* gq;           // [Q] gain of the query latent's norm
  const void* gk;           // [C]
  float eps, scale;
  void* cq;                 // [T][Q] normed query latents (out)
  void* kc;                 // pages [n][PS][C + R]
  long long k_sp;
  const int* table;
  int tstride, shift;
  const int* pos;           // [T]
  const int* slot;          // [T]
  const float* freq;        // [nr / 2] radians per position
  const void* q;            // [T][H][D + R]
  const void* qa;           // [T][H][C] absorbed queries W_uk^T q
  const void* sink;         // [H]
  float* part;              // partial softmaxes [rows][H][nsplit][C + 4]: m, l, -, -, sum of weighted latents
  int nsplit, chunk;        // keys per split
  const int* row_of;        // rows kernel: token row of block b (nullable: b)
  const void* wuv;          // [H][E][C]
  void* out;                // [T][H E], row stride ldo
  long long ldo;
  // prompt tiles
  const void* kv;           // expanded keys and values of the contexts [n][H D | H E], row stride ldkv
  long long ldkv;
  const void* kr;           // their cached rows [n][C + R] (the rotated part is read)
  const int* tiles;         // [ntiles][4]: first row, rows, position of the first row, context row of position 0
};

namespace latent {
template <typename E> __device__ __forceinline__ float ld(const E* p);
template <> __device__ __forceinline__ float ld<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ld<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <typename E> __device__ __forceinline__ void st(E* p, float v);
template <> __device__ __forceinline__ void st<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void st<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }

// rotated element i of a vector at position pos (pairs 2i, 2i + 1 below nr)
template <typename E>
__device__ __forceinline__ float rot(const E* x, int i, int pos, const float* freq, int nr) {
  const float v = ld<E>(x + i);
  if (i >= nr) return v;
  float s, c;
  sincosf((float)pos * freq[i >> 1], &s, &c);
  const float o = ld<E>(x + (i ^ 1));
  return (i & 1) ? v * c + o * s : v * c - o * s;
}
}  // namespace latent

static inline bool latent_args_ok(const LatentArgs& a) {
  return a.H > 0 && a.D > 0 && a.R >= 0 && a.E > 0 && a.C > 0 && a.Q > 0 && a.nr >= 0 && a.nr <= a.R && a.nr % 2 == 0 &&
         a.table && a.pos && a.slot && a.kc && a.shift >= 4 && (a.nr == 0 || a.freq);
}
