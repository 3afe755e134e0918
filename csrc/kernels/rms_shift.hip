// Residual add + RMS norm + token shift in one pass over the residual stream.
//
// Per token t of a flat batch of sequence portions ("entries"):
//   x_t   = x_in_t (or the embedding row of its token) + m * (a_t + sum_k y[inv[t][k]])
//   h_t   = x_t / sqrt(mean(x_t^2) + eps) * g          g: one number, or one per coordinate
//   hs_t  = h_t + (h_(t-1) - h_t) * mu                 the shifted copy a mixer reads
// The residual stream x is fp32 and double buffered (x_in -> x_out), so a workgroup may recompute its
// left neighbour's row; h / hs are written in the compute type, rounded once from fp32. h_(t-1) of an
// entry's first token is the carried row of its sequence (zeros at position 0), and an entry's last
// h is written to the sequence's slot. The carry is read from `prev` -- the slots themselves when every
// entry is one token (each thread reads its elements before it writes them), a gathered copy
// otherwise, since an entry's first and last rows may belong to different workgroups.
// `inv` / `y`: outputs of routed experts, `top` rows per token (moe.hip).
#include "common.h"

namespace {

struct RmsShiftArgs {
  const float* x_in;
  const void* embed;          // x_in null: embedding rows
  const long long* tokens;
  const void* a;              // branch output rows (nullable)
  long long lda;
  const void* y;              // expert output rows (nullable), row stride d
  const int* inv;             // [T][top]
  int top;
  float m;
  const void* gain;
  int gain_vec;               // 0: one number
  float eps;
  const void* mu;             // [d] (nullable: no shift)
  const float* prev;          // carried rows, stride d
  const int* prev_idx;        // [T] row of prev of an entry-first token
  const int* pos;             // [T]
  const int* flags;           // [T] bit 0: first of its entry, bit 1: last (null: every row is both)
  float* state;               // [slots][d]
  const int* slot;            // [T]
  const int* rows;            // output row i reads token rows[i] (nullable; no shift, no x_out)
  float* x_out;
  void* h;
  void* hs;
  int T, d, R;
};

template <typename E> __device__ __forceinline__ float ldf(const E* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <typename E> __device__ __forceinline__ void stf(E* p, float v);
template <> __device__ __forceinline__ void stf<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void stf<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }

template <int VEC>
__device__ __forceinline__ void ldv(const float* p, float (&v)[VEC]) {
  if constexpr (VEC == 4) {
    const float4 q = *reinterpret_cast<const float4*>(p);
    v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = p[i];
  }
}
template <int VEC>
__device__ __forceinline__ void ldv(const bf16_t* p, float (&v)[VEC]) {
  if constexpr (VEC == 4) {
    const U16x4 q = *reinterpret_cast<const U16x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = bf2f(q.v[i]);
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = bf2f(p[i]);
  }
}
template <int VEC>
__device__ __forceinline__ void stv(float* p, const float (&v)[VEC]) {
  if constexpr (VEC == 4) *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  else
#pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = v[i];
}
template <int VEC>
__device__ __forceinline__ void stv(bf16_t* p, const float (&v)[VEC]) {
  if constexpr (VEC == 4)
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
  else
#pragma unroll
    for (int i = 0; i < VEC; ++i) p[i] = f2bf(v[i]);
}

// E: compute type, VEC elements per access (4: d % 4 == 0), NCH accesses per thread
template <typename E, int VEC, int NCH>
__global__ void __launch_bounds__(256) rms_shift_kernel(RmsShiftArgs p) {
  __shared__ float red[4];
  const int tid = threadIdx.x, d = p.d;
  const E* a = reinterpret_cast<const E*>(p.a);
  const E* y = reinterpret_cast<const E*>(p.y);
  const E* gain = reinterpret_cast<const E*>(p.gain);
  const E* mu = reinterpret_cast<const E*>(p.mu);
  const int r0 = blockIdx.x * p.R, r1 = min(p.T, r0 + p.R);

  // row t -> h (registers); x_out written where `out` >= 0
  auto row = [&](int t, float (&h)[NCH][VEC], bool write_x) {
    float ss = 0.f;
    const long long tok = p.x_in ? 0 : p.tokens[t];
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * 256 + tid) * VEC;
      if (i >= d) continue;
      float x[VEC];
      if (p.x_in) ldv<VEC>(p.x_in + (long long)t * d + i, x);
      else ldv<VEC>(reinterpret_cast<const E*>(p.embed) + tok * d + i, x);
      float add[VEC];
#pragma unroll
      for (int e = 0; e < VEC; ++e) add[e] = 0.f;
      if (a) ldv<VEC>(a + (long long)t * p.lda + i, add);
      if (y)
        for (int k = 0; k < p.top; ++k) {
          float w[VEC];
          ldv<VEC>(y + (long long)p.inv[(long long)t * p.top + k] * d + i, w);
#pragma unroll
          for (int e = 0; e < VEC; ++e) add[e] += w[e];
        }
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        x[e] = fmaf(p.m, add[e], x[e]);
        ss = fmaf(x[e], x[e], ss);
        h[c][e] = x[e];
      }
      if (write_x) stv<VEC>(p.x_out + (long long)t * d + i, x);
    }
    const float rstd = 1.f / sqrtf(block_sum(ss, red) / (float)d + p.eps);
    const float g0 = p.gain_vec ? 1.f : ldf(gain);
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * 256 + tid) * VEC;
      if (i >= d) continue;
#pragma unroll
      for (int e = 0; e < VEC; ++e) h[c][e] = h[c][e] * rstd * (p.gain_vec ? ldf(gain + i + e) : g0);
    }
  };

  float pv[NCH][VEC];
  bool have = false;
  for (int r = r0; r < r1; ++r) {
    const int t = p.rows ? p.rows[r] : r;
    const int fl = p.flags ? p.flags[t] : 3;
    if (mu) {
      if (fl & 1) {
        const bool zero = p.pos[t] == 0;
        const float* src = p.prev + (long long)p.prev_idx[t] * d;
#pragma unroll
        for (int c = 0; c < NCH; ++c) {
          const int i = (c * 256 + tid) * VEC;
          if (i >= d) continue;
          if (zero) {
#pragma unroll
            for (int e = 0; e < VEC; ++e) pv[c][e] = 0.f;
          } else {
            ldv<VEC>(src + i, pv[c]);
          }
        }
      } else if (!have) {
        row(t - 1, pv, false);
      }
    }
    float h[NCH][VEC];
    row(t, h, p.x_out != nullptr);
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * 256 + tid) * VEC;
      if (i >= d) continue;
      if (p.h) stv<VEC>(reinterpret_cast<E*>(p.h) + (long long)r * d + i, h[c]);
      if (mu) {
        float m4[VEC], s[VEC];
        ldv<VEC>(mu + i, m4);
#pragma unroll
        for (int e = 0; e < VEC; ++e) s[e] = fmaf(pv[c][e] - h[c][e], m4[e], h[c][e]);
        stv<VEC>(reinterpret_cast<E*>(p.hs) + (long long)r * d + i, s);
        if (fl & 2) stv<VEC>(p.state + (long long)p.slot[t] * d + i, h[c]);
#pragma unroll
        for (int e = 0; e < VEC; ++e) pv[c][e] = h[c][e];
      }
    }
    have = true;
  }
}

template <typename E>
int launch(const RmsShiftArgs& a, hipStream_t s) {
  const dim3 g((a.T + a.R - 1) / a.R);
  const bool v4 = a.d % 4 == 0 && a.lda % 4 == 0;
  const int per = v4 ? 1024 : 256, n = (a.d + per - 1) / per;
#define GO(V, N) hipLaunchKernelGGL((rms_shift_kernel<E, V, N>), g, dim3(256), 0, s, a)
  if (v4) {
    if (n <= 1) GO(4, 1);
    else if (n <= 2) GO(4, 2);
    else if (n <= 4) GO(4, 4);
    else if (n <= 8) GO(4, 8);
    else if (n <= 16) GO(4, 16);
    else return 10;
  } else {
    if (n <= 1) GO(1, 1);
    else if (n <= 4) GO(1, 4);
    else if (n <= 16) GO(1, 16);
    else return 10;
  }
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

}  // namespace

// dtype: 0 fp32, 1 bf16 (of embed, a, y, gain, mu, h, hs)
KCA_API int kca_rms_shift(int dtype, const void* x_in, const void* embed, const void* tokens, const void* a,
                          long long lda, const void* y, const void* inv, int top, float m, const void* gain,
                          int gain_vec, float eps, const void* mu, const void* prev, const void* prev_idx,
                          const void* pos, const void* flags, void* state, const void* slot, const void* rows,
                          void* x_out, void* h, void* hs, int T, int d, int R, hipStream_t s) {
  if (T < 1 || d < 1 || R < 1 || (!x_in && (!embed || !tokens)) || !gain || (y && (!inv || top < 1))) return 1;
  if (mu && (!prev || !prev_idx || !pos || !state || !slot || !hs || rows)) return 1;
  if (x_in && x_in == x_out) return 2;
  if (rows && x_out) return 2;
  RmsShiftArgs p{(const float*)x_in, embed, (const long long*)tokens, a, lda, y, (const int*)inv, top, m, gain,
                 gain_vec, eps, mu, (const float*)prev, (const int*)prev_idx, (const int*)pos, (const int*)flags,
                 (float*)state, (const int*)slot, (const int*)rows, (float*)x_out, h, hs, T, d, R};
  if (dtype == 0) return launch<float>(p, s);
  if (dtype == 1) return launch<bf16_t>(p, s);
  return 3;
}
