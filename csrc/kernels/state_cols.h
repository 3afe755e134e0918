// A head's recurrent state [dk][dv] spread over waves, for the token-by-token recurrences (delta_rule.hip,
// matrix_memory.hip).
#pragma once
#include "common.h"
#include "lanes.h"

namespace {

// A wave's part of the state: CW columns from 4 column groups (lane >> 4), rows lane & 15 + 16 i.
template <int R, int CW>
struct Cols {
  float s[R][CW];
  __device__ __forceinline__ void load(const float* S, int dk, int dv, int rg, int col, bool live) {
#pragma unroll
    for (int i = 0; i < R; ++i) {
      const int r = rg + 16 * i;
#pragma unroll
      for (int e = 0; e < CW; ++e) s[i][e] = 0.f;
      if (live && r < dk && col < dv) {
        const float* q = S + (long long)r * dv + col;
        if constexpr (CW == 4) {
          const float4 v = *reinterpret_cast<const float4*>(q);
          s[i][0] = v.x; s[i][1] = v.y; s[i][2] = v.z; s[i][3] = v.w;
        } else {
          s[i][0] = *q;
        }
      }
    }
  }
  __device__ __forceinline__ void store(float* S, int dk, int dv, int rg, int col) const {
#pragma unroll
    for (int i = 0; i < R; ++i) {
      const int r = rg + 16 * i;
      if (r < dk && col < dv) {
        float* q = S + (long long)r * dv + col;
        if constexpr (CW == 4) *reinterpret_cast<float4*>(q) = make_float4(s[i][0], s[i][1], s[i][2], s[i][3]);
        else *q = s[i][0];
      }
    }
  }
  // one token: the vectors at rows rg + 16 i (zero past dk), v at the lane's columns -> read-out
  template <bool DELTA = true>
  __device__ __forceinline__ void token(const float (&w)[R], const float (&z)[R], const float (&p)[R], const float (&k)[R],
                                        const float (&q)[R], const float (&v)[CW], float qp, float qk, float (&o)[CW]) {
    float zs[CW], qs[CW];
#pragma unroll
    for (int e = 0; e < CW; ++e) zs[e] = qs[e] = 0.f;
#pragma unroll
    for (int i = 0; i < R; ++i) {
      const float qw = q[i] * w[i];
#pragma unroll
      for (int e = 0; e < CW; ++e) {
        if (DELTA) zs[e] = fmaf(z[i], s[i][e], zs[e]);
        qs[e] = fmaf(qw, s[i][e], qs[e]);
      }
    }
    auto add = [](float x, float y) { return x + y; };
#pragma unroll
    for (int e = 0; e < CW; ++e) {
      if (DELTA) zs[e] = lanes_reduce<16>(zs[e], add);
      qs[e] = lanes_reduce<16>(qs[e], add);
      o[e] = qs[e] + qp * zs[e] + qk * v[e];  // q^T (w S + p s + k v)
    }
#pragma unroll
    for (int i = 0; i < R; ++i)
#pragma unroll
      for (int e = 0; e < CW; ++e) s[i][e] = fmaf(w[i], s[i][e], DELTA ? fmaf(p[i], zs[e], k[i] * v[e]) : k[i] * v[e]);
  }
  // one token of a state with one decay: S <- w S + k v^T -> read-out q^T S, with qk = q . k
  __device__ __forceinline__ void decayed(float w, const float (&k)[R], const float (&q)[R], const float (&v)[CW], float qk,
                                          float (&o)[CW]) {
#pragma unroll
    for (int e = 0; e < CW; ++e) o[e] = 0.f;
#pragma unroll
    for (int i = 0; i < R; ++i)
#pragma unroll
      for (int e = 0; e < CW; ++e) o[e] = fmaf(q[i], s[i][e], o[e]);
#pragma unroll
    for (int e = 0; e < CW; ++e) o[e] = fmaf(w, lanes_reduce<16>(o[e], [](float x, float y) { return x + y; }), qk * v[e]);
#pragma unroll
    for (int i = 0; i < R; ++i)
#pragma unroll
      for (int e = 0; e < CW; ++e) s[i][e] = fmaf(w, s[i][e], k[i] * v[e]);
  }
};

template <int R>
__device__ __forceinline__ void rows_of(const float* src, int dk, int rg, float (&x)[R]) {
#pragma unroll
  for (int i = 0; i < R; ++i) x[i] = rg + 16 * i < dk ? src[rg + 16 * i] : 0.f;
}

static inline int state_rows(int dk) {  // rows a lane holds: 16 row groups
  const int n = (dk + 15) / 16;
  return n <= 1 ? 1 : n <= 2 ? 2 : n <= 3 ? 3 : n <= 4 ? 4 : n <= 6 ? 6 : n <= 8 ? 8 : n <= 12 ? 12 : 16;
}

#define KCA_STATE_ROWS(DK, F)        \
  switch (state_rows(DK)) {         \
    case 1: return F(1);            \
    case 2: return F(2);            \
    case 3: return F(3);            \
    case 4: return F(4);            \
    case 6: return F(6);            \
    case 8: return F(8);            \
    case 12: return F(12);          \
    default: return F(16);          \
  }

}  // namespace
