// Sandwich norms around a sublayer, in one pass over the residual stream. Per token t:
//   x_t = x_in_t (or the embedding row of its token) + ls * N(a_t + b; gb)
//   h_t = N(x_t; g)
// N(v; g) is a layer norm (v - mean) / sqrt(var + eps) * g or an RMS norm v / sqrt(mean v^2 + eps) * g.
// a: the sublayer's output rows, b its bias (optional), ls a per-coordinate scale. The stream x is fp32 and
// double buffered; h is rounded once. Statistics are fp32 and two-pass within a wave; the waves of a row merge
// theirs by counts (one barrier a norm). Few rows load gains and scales ahead of the statistics (AHEAD).
//
// Pre-norms (prenorm_kernel), RMS throughout:
//   x_t = src_t + a_t     or   x_t = src_t + mul * (N(a_t; ga) + N(b_t; gb))
//   h_t = x_t / sqrt(mean x_t^2 + eps) * (1 + g),   raw_t = x_t rounded (a column block of a wider buffer)
// src: the stream, scaled embedding rows, or rows of a product plus one vector.
//
// Post-norms (postnorm_kernel): RMS norms of what a sublayer adds, gains of one number
//   u_t = a_t + sum_k y[inv[t][k]] + (sum of wts[t][k] with inv -1) src_t      routed rows (moe.hip), identity experts
//   x_t = src_t + ga u_t / sqrt(mean u_t^2 + eps)
//   h_t = x_t rounded, or hmul g x_t / sqrt(mean x_t^2 + eps)
#include "common.h"
#include "lanes.h"

namespace {

struct NormArgs {
  const float* x_in;
  const void* embed;          // x_in null: embedding rows
  const long long* tokens;
  const void* a;              // sublayer output (nullable)
  long long lda;
  const void* bias;           // [d] (nullable)
  const void* gb;             // [d] gain of the output norm
  const void* ls;             // [d] layer scale (nullable: 1)
  const void* g;              // [d] gain of the next norm
  float eps;
  const int* rows;            // output row i reads token rows[i] (nullable)
  float* x_out;               // nullable
  void* h;                    // nullable
  int T, d, layer;            // layer: 1 layer norm, 0 RMS norm
};

template <typename E> __device__ __forceinline__ float ldf(const E* p);
template <> __device__ __forceinline__ float ldf<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ldf<bf16_t>(const bf16_t* p) { return bf2f(*p); }

template <typename E, int VEC>
__device__ __forceinline__ void ldv(const E* p, float (&v)[VEC]) {
  if constexpr (VEC == 4 && sizeof(E) == 4) {
    const float4 q = *reinterpret_cast<const float4*>(p);
    v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
  } else if constexpr (VEC == 4) {
    const U16x4 q = *reinterpret_cast<const U16x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = bf2f(q.v[i]);
  } else {
#pragma unroll
    for (int i = 0; i < VEC; ++i) v[i] = ldf<E>(p + i);
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

// a vector of parameters as loaded
template <typename E, int VEC>
struct alignas(VEC * sizeof(E)) Pack {
  E v[VEC];
  __device__ __forceinline__ float at(int i) const { return ldf<E>(v + i); }
};

template <typename E, int VEC, int NCH, int NT, bool AHEAD>
__global__ void __launch_bounds__(256) norm_residual_kernel(NormArgs p) {
  constexpr int RPB = 256 / NT;  // rows of a workgroup (one wave each when NT == 64)
  static_assert(RPB == 1 || NT == 64, "a row is a wave or the workgroup");
  __shared__ float2 red[2][NT / 64];  // a norm each
  const int tid = threadIdx.x % NT, d = p.d;
  const int r = blockIdx.x * RPB + threadIdx.x / NT;
  if (r >= p.T) return;  // (whole waves; RPB == 1: never)
  const int t = p.rows ? p.rows[r] : r;
  const float inv = 1.f / (float)d;
  float x[NCH][VEC], v[NCH][VEC];
  const E* a = reinterpret_cast<const E*>(p.a);
  const long long tok = p.x_in ? 0 : p.tokens[t];
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = (c * NT + tid) * VEC;
    if (i < d) {
      if (p.x_in) ldv<float, VEC>(p.x_in + (long long)t * d + i, x[c]);
      else ldv<E, VEC>(reinterpret_cast<const E*>(p.embed) + tok * d + i, x[c]);
      if (a) ldv<E, VEC>(a + (long long)t * p.lda + i, v[c]);
    } else {
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[c][e] = 0.f;
    }
  }
  using P = Pack<E, VEC>;
  auto par = [&](const void* q, int c) { return *reinterpret_cast<const P*>(reinterpret_cast<const E*>(q) + min((c * NT + tid) * VEC, d - VEC)); };
  P pgb[AHEAD ? NCH : 1], pls[AHEAD ? NCH : 1], pg[AHEAD ? NCH : 1];
  if constexpr (AHEAD) {
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      if (a) pgb[c] = par(p.gb, c);
      if (a && p.ls) pls[c] = par(p.ls, c);
      if (p.h) pg[c] = par(p.g, c);
    }
  }
  auto get = [&](const P* ahead, const void* q, int c) {
    if constexpr (AHEAD) return ahead[c];
    else return par(q, c);
  };
  auto add = [](float u, float w) { return u + w; };
  // mean and 1 / deviation of a row
  auto stats = [&](float (&q)[NCH][VEC], float2* rd, float& mean, float& rstd) {
    auto count = [&](int w) {  // elements of the row's wave w
      int n = 0;
#pragma unroll
      for (int c = 0; c < NCH; ++c) n += min(max(d - (c * NT + 64 * w) * VEC, 0), 64 * VEC);
      return (float)n;
    };
    const int wv = NT == 64 ? 0 : threadIdx.x >> 6;
    float s = 0.f, ss = 0.f, mw = 0.f;
    if (p.layer) {
#pragma unroll
      for (int c = 0; c < NCH; ++c)
#pragma unroll
        for (int e = 0; e < VEC; ++e) s += (c * NT + tid) * VEC < d ? q[c][e] : 0.f;
      s = lanes_reduce<64>(s, add);
      mw = s * __builtin_amdgcn_rcpf(fmaxf(count(wv), 1.f));
    }
#pragma unroll
    for (int c = 0; c < NCH; ++c)
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        const float y = (c * NT + tid) * VEC < d ? q[c][e] - mw : 0.f;
        ss = fmaf(y, y, ss);
      }
    ss = lanes_reduce<64>(ss, add);
    mean = mw;
    if constexpr (NT > 64) {
      if ((threadIdx.x & 63) == 0) rd[wv] = make_float2(s, ss);
      __syncthreads();
      float2 o[NT / 64];
      s = ss = 0.f;
#pragma unroll
      for (int i = 0; i < NT / 64; ++i) {
        o[i] = rd[i];
        s += o[i].x;
        ss += o[i].y;
      }
      mean = s * inv;  // (RMS norm: 0)
      if (p.layer)
#pragma unroll
        for (int i = 0; i < NT / 64; ++i) {
          const float n = count(i), off = o[i].x - n * mean;
          ss = fmaf(off, off * __builtin_amdgcn_rcpf(fmaxf(n, 1.f)), ss);
        }
    }
    rstd = 1.f / sqrtf(ss * inv + p.eps);
  };
  if (a) {
    if (p.bias) {
#pragma unroll
      for (int c = 0; c < NCH; ++c) {
        const P b = par(p.bias, c);
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[c][e] += b.at(e);
      }
    }
    float mean, rstd;
    stats(v, red[0], mean, rstd);
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      if ((c * NT + tid) * VEC >= d) continue;
      const P g = get(pgb, p.gb, c);
      P s;
      if (p.ls) s = get(pls, p.ls, c);
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        const float n = (v[c][e] - mean) * rstd * g.at(e);
        x[c][e] = p.ls ? fmaf(s.at(e), n, x[c][e]) : x[c][e] + n;
      }
    }
  }
  if (p.x_out) {
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      const int i = (c * NT + tid) * VEC;
      if (i < d) stv<VEC>(p.x_out + (long long)r * d + i, x[c]);
    }
  }
  if (!p.h) return;
  float mean, rstd;
  stats(x, red[1], mean, rstd);
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = (c * NT + tid) * VEC;
    if (i >= d) continue;
    const P g = get(pg, p.g, c);
    float y[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = (x[c][e] - mean) * rstd * g.at(e);
    stv<VEC>(reinterpret_cast<E*>(p.h) + (long long)r * d + i, y);
  }
}

template <typename E>
int launch(const NormArgs& a, hipStream_t s) {
  const bool v4 = a.d % 4 == 0 && a.lda % 4 == 0;
#define GO(V, N, NT, AHEAD)                                                                                          \
  hipLaunchKernelGGL((norm_residual_kernel<E, V, N, NT, AHEAD>), dim3((a.T + 256 / NT - 1) / (256 / NT)), dim3(256), 0, s, a)
  const bool few = a.T <= 256;
  if (v4 && a.T >= 512 && a.d <= 1024) {  // many short rows: a wave each, no barriers
    if (a.d <= 256) GO(4, 1, 64, false);
    else if (a.d <= 512) GO(4, 2, 64, false);
    else GO(4, 4, 64, false);
  } else if (v4) {
    const int n = (a.d + 1023) / 1024;
    if (n <= 1) GO(4, 1, 256, true);
    else if (n <= 2) GO(4, 2, 256, true);
    else if (n <= 4 && few) GO(4, 4, 256, true);
    else if (n <= 4) GO(4, 4, 256, false);
    else if (n <= 8) GO(4, 8, 256, false);
    else if (n <= 16) GO(4, 16, 256, false);
    else return 10;
  } else {
    const int n = (a.d + 255) / 256;
    if (n <= 1) GO(1, 1, 256, false);
    else if (n <= 4) GO(1, 4, 256, false);
    else if (n <= 16) GO(1, 16, 256, false);
    else return 10;
  }
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

struct PreArgs {
  const float* x_in;          // one source: the stream,
  const void* embed;          // embedding rows (times escale),
  const long long* tokens;
  float escale;
  const void* base;           // or rows (stride ldbase) plus vec
  long long ldbase;
  const void* vec;
  const void* a;              // sublayer output (nullable)
  long long lda;
  const void* ga;             // gain of its norm (nullable: added as it is)
  const void* b;              // a second one, normed too (nullable)
  long long ldb;
  const void* gb;
  float mul;                  // of the normed outputs
  const void* g;              // the next norm's gain minus one
  float eps;
  const int* rows;            // output row i reads token rows[i] (nullable)
  float* x_out;               // nullable
  void* raw;                  // nullable, row stride ldr
  long long ldr;
  void* h;                    // nullable
  int T, d;
};

template <typename E, int VEC, int NCH, int NT, bool AHEAD>
__global__ void __launch_bounds__(256) prenorm_kernel(PreArgs p) {
  constexpr int RPB = 256 / NT;  // rows of a workgroup (one wave each when NT == 64)
  static_assert(RPB == 1 || NT == 64, "a row is a wave or the workgroup");
  __shared__ float2 red[2][NT / 64];
  const int tid = threadIdx.x % NT, d = p.d;
  const int r = blockIdx.x * RPB + threadIdx.x / NT;
  if (r >= p.T) return;  // (whole waves; RPB == 1: never)
  const int t = p.rows ? p.rows[r] : r;
  const float inv = 1.f / (float)d;
  using P = Pack<E, VEC>;
  float x[NCH][VEC], u[NCH][VEC], v[NCH][VEC];
  auto at = [&](int c) { return (c * NT + tid) * VEC; };
  auto par = [&](const void* q, int c) { return *reinterpret_cast<const P*>(reinterpret_cast<const E*>(q) + min(at(c), d - VEC)); };
  const long long tok = p.embed ? p.tokens[t] : 0;
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = at(c);
#pragma unroll
    for (int e = 0; e < VEC; ++e) x[c][e] = u[c][e] = v[c][e] = 0.f;
    if (i < d) {
      if (p.x_in) ldv<float, VEC>(p.x_in + (long long)t * d + i, x[c]);
      else if (p.embed) ldv<E, VEC>(reinterpret_cast<const E*>(p.embed) + tok * d + i, x[c]);
      else ldv<E, VEC>(reinterpret_cast<const E*>(p.base) + (long long)t * p.ldbase + i, x[c]);
      if (p.a) ldv<E, VEC>(reinterpret_cast<const E*>(p.a) + (long long)t * p.lda + i, u[c]);
      if (p.b) ldv<E, VEC>(reinterpret_cast<const E*>(p.b) + (long long)t * p.ldb + i, v[c]);
    }
  }
  P pa[AHEAD ? NCH : 1], pb[AHEAD ? NCH : 1], pg[AHEAD ? NCH : 1];
  if constexpr (AHEAD) {
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      if (p.ga) pa[c] = par(p.ga, c);
      if (p.gb) pb[c] = par(p.gb, c);
      if (p.h) pg[c] = par(p.g, c);
    }
  }
  auto get = [&](const P* ahead, const void* q, int c) {
    if constexpr (AHEAD) return ahead[c];
    else return par(q, c);
  };
  auto add = [](float y, float z) { return y + z; };
  // sums of squares of two rows (elements past d are zero)
  auto sums = [&](const float (&y)[NCH][VEC], const float (&z)[NCH][VEC], bool both, float2* rd) {
    float2 s = make_float2(0.f, 0.f);
#pragma unroll
    for (int c = 0; c < NCH; ++c)
#pragma unroll
      for (int e = 0; e < VEC; ++e) {
        s.x = fmaf(y[c][e], y[c][e], s.x);
        if (both) s.y = fmaf(z[c][e], z[c][e], s.y);
      }
    s.x = lanes_reduce<64>(s.x, add);
    if (both) s.y = lanes_reduce<64>(s.y, add);
    if constexpr (NT > 64) {
      if ((threadIdx.x & 63) == 0) rd[threadIdx.x >> 6] = s;
      __syncthreads();
      s = make_float2(0.f, 0.f);
#pragma unroll
      for (int i = 0; i < NT / 64; ++i) s.x += rd[i].x, s.y += rd[i].y;
    }
    return s;
  };
  if (p.embed) {
#pragma unroll
    for (int c = 0; c < NCH; ++c)
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[c][e] *= p.escale;
  } else if (p.vec && !p.x_in) {
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      if (at(c) >= d) continue;
      const P w = par(p.vec, c);
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[c][e] += w.at(e);
    }
  }
  if (p.ga) {
    const float2 s = sums(u, v, p.b != nullptr, red[0]);
    const float na = p.mul / sqrtf(s.x * inv + p.eps), nb = p.mul / sqrtf(s.y * inv + p.eps);
#pragma unroll
    for (int c = 0; c < NCH; ++c) {
      if (at(c) >= d) continue;
      const P ga = get(pa, p.ga, c);
#pragma unroll
      for (int e = 0; e < VEC; ++e) u[c][e] *= na * ga.at(e);
      if (p.b) {
        const P gb = get(pb, p.gb, c);
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[c][e] = fmaf(v[c][e], nb * gb.at(e), u[c][e]);
      }
    }
  }
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = at(c);
    if (p.a)
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[c][e] += u[c][e];
    if (i < d) {
      if (p.x_out) stv<VEC>(p.x_out + (long long)r * d + i, x[c]);
      if (p.raw) stv<VEC>(reinterpret_cast<E*>(p.raw) + (long long)r * p.ldr + i, x[c]);
    }
  }
  if (!p.h) return;
  const float n = 1.f / sqrtf(sums(x, x, false, red[1]).x * inv + p.eps);
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = at(c);
    if (i >= d) continue;
    const P g = get(pg, p.g, c);
    float y[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = x[c][e] * n * (1.f + g.at(e));
    stv<VEC>(reinterpret_cast<E*>(p.h) + (long long)r * d + i, y);
  }
}

struct PostArgs {
  const float* x_in;          // one source: the stream,
  const void* embed;          // embedding rows (times escale)
  const long long* tokens;
  float escale;
  const void* a;              // sublayer output (nullable)
  long long lda;
  const void* y;              // routed rows (nullable), row stride d
  const int* inv;             // [T][top] row of y; -1: the source itself, times
  const float* wts;           // [T][top]
  int top;
  const void* ga;             // gain of their norm (nullable: nothing is added)
  const void* g;              // gain of the closing norm (nullable: none)
  float hmul, eps;
  const int* rows;            // output row i reads token rows[i] (nullable)
  float* x_out;               // nullable
  void* h;                    // nullable
  int T, d;
};

template <typename E, int VEC, int NCH, int NT>
__global__ void __launch_bounds__(256) postnorm_kernel(PostArgs p) {
  constexpr int RPB = 256 / NT;  // rows of a workgroup (one wave each when NT == 64)
  static_assert(RPB == 1 || NT == 64, "a row is a wave or the workgroup");
  __shared__ float red[2][NT / 64];
  const int tid = threadIdx.x % NT, d = p.d;
  const int r = blockIdx.x * RPB + threadIdx.x / NT;
  if (r >= p.T) return;  // (whole waves; RPB == 1: never)
  const int t = p.rows ? p.rows[r] : r;
  const float inv = 1.f / (float)d;
  float x[NCH][VEC], u[NCH][VEC];
  auto at = [&](int c) { return (c * NT + tid) * VEC; };
  const long long tok = p.embed ? p.tokens[t] : 0;
  const float ga = p.ga ? ldf<E>(reinterpret_cast<const E*>(p.ga)) : 0.f, g = p.g ? ldf<E>(reinterpret_cast<const E*>(p.g)) : 0.f;
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    const int i = at(c);
#pragma unroll
    for (int e = 0; e < VEC; ++e) x[c][e] = u[c][e] = 0.f;
    if (i < d) {
      if (p.x_in) ldv<float, VEC>(p.x_in + (long long)t * d + i, x[c]);
      else ldv<E, VEC>(reinterpret_cast<const E*>(p.embed) + tok * d + i, x[c]);
      if (p.a) ldv<E, VEC>(reinterpret_cast<const E*>(p.a) + (long long)t * p.lda + i, u[c]);
    }
  }
  if (p.embed)
#pragma unroll
    for (int c = 0; c < NCH; ++c)
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[c][e] *= p.escale;
  if (p.y) {
    const int* iv = p.inv + (long long)t * p.top;
    const float* wt = p.wts + (long long)t * p.top;
    float pass = 0.f;
    for (int k0 = 0; k0 < p.top; k0 += 4) {  // four rows' loads together; past the end and identity experts: row 0 times zero
      float v[4][NCH][VEC], on[4];
#pragma unroll
      for (int k = 0; k < 4; ++k) {
        const bool in = k0 + k < p.top;
        const int row = in ? iv[k0 + k] : 0;
        on[k] = in && row >= 0 ? 1.f : 0.f;
        if (in && row < 0) pass += wt[k0 + k];
#pragma unroll
        for (int c = 0; c < NCH; ++c) {
#pragma unroll
          for (int e = 0; e < VEC; ++e) v[k][c][e] = 0.f;
          if (at(c) < d && on[k] != 0.f) ldv<E, VEC>(reinterpret_cast<const E*>(p.y) + (long long)row * d + at(c), v[k][c]);
        }
      }
#pragma unroll
      for (int k = 0; k < 4; ++k)
#pragma unroll
        for (int c = 0; c < NCH; ++c)
#pragma unroll
          for (int e = 0; e < VEC; ++e) u[c][e] += v[k][c][e];
    }
#pragma unroll
    for (int c = 0; c < NCH; ++c)
#pragma unroll
      for (int e = 0; e < VEC; ++e) u[c][e] = fmaf(pass, x[c][e], u[c][e]);
  }
  auto rstd = [&](const float (&y)[NCH][VEC], float* rd) {  // (elements past d are zero)
    float s = 0.f;
#pragma unroll
    for (int c = 0; c < NCH; ++c)
#pragma unroll
      for (int e = 0; e < VEC; ++e) s = fmaf(y[c][e], y[c][e], s);
    s = lanes_reduce<64>(s, [](float a, float b) { return a + b; });
    if constexpr (NT > 64) {
      if ((threadIdx.x & 63) == 0) rd[threadIdx.x >> 6] = s;
      __syncthreads();
      s = 0.f;
#pragma unroll
      for (int i = 0; i < NT / 64; ++i) s += rd[i];
    }
    return 1.f / sqrtf(s * inv + p.eps);
  };
  if (p.ga) {
    const float n = ga * rstd(u, red[0]);
#pragma unroll
    for (int c = 0; c < NCH; ++c)
#pragma unroll
      for (int e = 0; e < VEC; ++e) x[c][e] = fmaf(n, u[c][e], x[c][e]);
  }
  if (p.x_out) {
#pragma unroll
    for (int c = 0; c < NCH; ++c)
      if (at(c) < d) stv<VEC>(p.x_out + (long long)r * d + at(c), x[c]);
  }
  if (!p.h) return;
  const float n = p.g ? p.hmul * g * rstd(x, red[1]) : 1.f;
#pragma unroll
  for (int c = 0; c < NCH; ++c) {
    float y[VEC];
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = x[c][e] * n;
    if (at(c) < d) stv<VEC>(reinterpret_cast<E*>(p.h) + (long long)r * d + at(c), y);
  }
}

template <typename E>
int launch_post(const PostArgs& a, hipStream_t s) {
  const bool v4 = a.d % 4 == 0 && a.lda % 4 == 0;
#define GO(V, N, NT) \
  hipLaunchKernelGGL((postnorm_kernel<E, V, N, NT>), dim3((a.T + 256 / NT - 1) / (256 / NT)), dim3(256), 0, s, a)
  if (v4 && a.T >= 512 && a.d <= 1024) {  // many short rows: a wave each, no barriers
    if (a.d <= 256) GO(4, 1, 64);
    else if (a.d <= 512) GO(4, 2, 64);
    else GO(4, 4, 64);
  } else if (v4) {
    const int n = (a.d + 1023) / 1024;
    if (n <= 1) GO(4, 1, 256);
    else if (n <= 2) GO(4, 2, 256);
    else if (n <= 4) GO(4, 4, 256);
    else if (n <= 8) GO(4, 8, 256);
    else if (n <= 16) GO(4, 16, 256);
    else return 10;
  } else {
    const int n = (a.d + 255) / 256;
    if (n <= 1) GO(1, 1, 256);
    else if (n <= 4) GO(1, 4, 256);
    else if (n <= 16) GO(1, 16, 256);
    else return 10;
  }
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

template <typename E>
int launch_pre(const PreArgs& a, hipStream_t s) {
  const bool v4 = a.d % 4 == 0 && a.lda % 4 == 0 && a.ldb % 4 == 0 && a.ldbase % 4 == 0 && a.ldr % 4 == 0 &&
                  (uintptr_t)a.raw % (4 * sizeof(E)) == 0;
#define GO(V, N, NT, AHEAD)                                                                                          \
  hipLaunchKernelGGL((prenorm_kernel<E, V, N, NT, AHEAD>), dim3((a.T + 256 / NT - 1) / (256 / NT)), dim3(256), 0, s, a)
  const bool few = a.T <= 256;
  if (v4 && a.T >= 512 && a.d <= 1024) {  // many short rows: a wave each, no barriers
    if (a.d <= 256) GO(4, 1, 64, false);
    else if (a.d <= 512) GO(4, 2, 64, false);
    else GO(4, 4, 64, false);
  } else if (v4) {
    const int n = (a.d + 1023) / 1024;
    if (n <= 1) GO(4, 1, 256, true);
    else if (n <= 2) GO(4, 2, 256, true);
    else if (n <= 4 && few) GO(4, 4, 256, true);
    else if (n <= 4) GO(4, 4, 256, false);
    else if (n <= 8) GO(4, 8, 256, false);
    else if (n <= 16) GO(4, 16, 256, false);
    else return 10;
  } else {
    const int n = (a.d + 255) / 256;
    if (n <= 1) GO(1, 1, 256, false);
    else if (n <= 4) GO(1, 4, 256, false);
    else if (n <= 16) GO(1, 16, 256, false);
    else return 10;
  }
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

}  // namespace

// dtype: 0 fp32, 1 bf16 (of embed, a, bias, gains, ls, h)
KCA_API int kca_norm_residual(int dtype, const void* x_in, const void* embed, const void* tokens, const void* a,
                              long long lda, const void* bias, const void* gb, const void* ls, const void* g,
                              float eps, const void* rows, void* x_out, void* h, int T, int d, int layer,
                              hipStream_t s) {
  if (T < 1 || d < 1 || (!x_in && (!embed || !tokens)) || (a && !gb) || (h && !g) || (!h && !x_out)) return 1;
  if (x_in && x_in == x_out && rows) return 2;
  const NormArgs p{(const float*)x_in, embed, (const long long*)tokens, a, lda, bias, gb, ls, g, eps, (const int*)rows,
                   (float*)x_out, h, T, d, layer};
  if (dtype == 0) return launch<float>(p, s);
  if (dtype == 1) return launch<bf16_t>(p, s);
  return 3;
}

// Mirrored by ops/norm_residual.py
KCA_API int kca_prenorm_abi() { return (int)sizeof(PreArgs); }

// dtype: 0 fp32, 1 bf16 (of every tensor but the stream)
KCA_API int kca_prenorm(const PreArgs* in, int dtype, hipStream_t s) {
  const PreArgs& p = *in;
  const int src = (p.x_in != nullptr) + (p.embed != nullptr) + (p.base != nullptr);
  if (p.T < 1 || p.d < 1 || src != 1 || (p.embed && !p.tokens) || (!p.a && (p.ga || p.b)) || (p.b && (!p.ga || !p.gb)) ||
      (p.h && !p.g) || (!p.h && !p.x_out && !p.raw))
    return 1;
  if (p.x_in && p.x_in == p.x_out && p.rows) return 2;
  if (dtype == 0) return launch_pre<float>(p, s);
  if (dtype == 1) return launch_pre<bf16_t>(p, s);
  return 3;
}

KCA_API int kca_postnorm_abi() { return (int)sizeof(PostArgs); }

// dtype: 0 fp32, 1 bf16 (of every tensor but the stream and the router's weights)
KCA_API int kca_postnorm(const PostArgs* in, int dtype, hipStream_t s) {
  const PostArgs& p = *in;
  if (p.T < 1 || p.d < 1 || (p.x_in != nullptr) == (p.embed != nullptr) || (p.embed && !p.tokens) || (p.ga && !p.a && !p.y) ||
      (!p.ga && (p.a || p.y)) || (p.y && (!p.inv || !p.wts || p.top < 1)) || (!p.h && (!p.x_out || p.g)))
    return 1;
  if (p.x_in && p.x_in == p.x_out && p.rows) return 2;
  if (dtype == 0) return launch_post<float>(p, s);
  if (dtype == 1) return launch_post<bf16_t>(p, s);
  return 3;
}
