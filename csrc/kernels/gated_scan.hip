// Gated linear recurrence (minGRU form) over a flat batch of sequence portions.
//
//   z = sigmoid(zx + bz), u = ux + bx, c = u + 1/2 (u >= 0) or sigmoid(u) (u < 0)
//   S_t = (1 - z) S_(t-1) + z c,   y_t = S_t * silu(g_t)
// with [z | x | g] the three projections of one GEMM, side by side per row. Gates and state are fp32.
//
// The recurrence is an affine map per element, so a portion is cut in chunks: scan_sum_kernel folds
// every chunk that has a successor into one (A, B) with S_end = A S_0 + B (all chunks at once), and
// scan_run_kernel starts each chunk from its predecessors' maps applied to the carried state and
// writes y. The carried state of a sequence lives in its slot; a chunk-0 workgroup of a portion with
// several chunks takes it from the copy scan_sum_kernel made, since the last chunk overwrites it.
#include "common.h"

namespace {

struct ScanArgs {
  const void* zxg;        // [T][3W] (row stride ld)
  long long ld;
  const void* bz;         // [W]
  const void* bx;
  void* y;                // row stride ldy
  long long ldy;
  float* state;           // [slots][W]
  float* ws;              // [nchunk][3][W]: A, B, S_0 (of chunk 0)
  const int* chunks;      // [nchunk][6]: row0, rows, index in entry, chunks in entry, position of row0, slot
  int W, nchunk;
};

template <typename E> struct Vec;
template <> struct Vec<bf16_t> {
  static constexpr bool fast = true;
  static __device__ __forceinline__ float ld(const bf16_t* p) { return bf2f(*p); }
  static __device__ __forceinline__ void st(bf16_t* p, float v) { *p = f2bf(v); }
  static __device__ __forceinline__ float sig(float x) { return __builtin_amdgcn_rcpf(1.f + __expf(-x)); }
};
template <> struct Vec<float> {
  static constexpr bool fast = false;
  static __device__ __forceinline__ float ld(const float* p) { return *p; }
  static __device__ __forceinline__ void st(float* p, float v) { *p = v; }
  static __device__ __forceinline__ float sig(float x) { return 1.f / (1.f + expf(-x)); }
};

// V elements as loaded (converted at use), so that the next tokens' loads stay in flight in few registers
template <typename E, int V>
struct alignas(sizeof(E) * V) Raw {
  E v[V];
  __device__ __forceinline__ float f(int i) const { return Vec<E>::ld(v + i); }
};

template <typename E, int V>
__device__ __forceinline__ void ldn(const E* p, float (&v)[V]) {
  if constexpr (V == 4 && sizeof(E) == 2) {
    const U16x4 q = *reinterpret_cast<const U16x4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = bf2f(q.v[i]);
  } else if constexpr (V == 4) {
    const float4 q = *reinterpret_cast<const float4*>(p);
    v[0] = q.x; v[1] = q.y; v[2] = q.z; v[3] = q.w;
  } else {
#pragma unroll
    for (int i = 0; i < V; ++i) v[i] = Vec<E>::ld(p + i);
  }
}
template <typename E, int V>
__device__ __forceinline__ void stn(E* p, const float (&v)[V]) {
  if constexpr (V == 4 && sizeof(E) == 2)
    *reinterpret_cast<uint2*>(p) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
  else if constexpr (V == 2 && sizeof(E) == 2)
    *reinterpret_cast<uint32_t*>(p) = pack_bf16x2(v[0], v[1]);
  else if constexpr (V == 4)
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
  else
#pragma unroll
    for (int i = 0; i < V; ++i) Vec<E>::st(p + i, v[i]);
}

// one element's gate and candidate
template <typename E>
__device__ __forceinline__ void gate(float zx, float ux, float& z, float& zc) {
  if constexpr (Vec<E>::fast) {
    const float ez = 1.f + __expf(fminf(-zx, 28.f)), eu = 1.f + __expf(fminf(-ux, 28.f));
    const float r = __builtin_amdgcn_rcpf(ez * eu);
    z = r * eu;
    zc = z * (ux >= 0.f ? ux + 0.5f : r * ez);
    return;
  }
  z = Vec<E>::sig(zx);
  const float c = ux >= 0.f ? ux + 0.5f : Vec<E>::sig(ux);
  zc = z * c;
}

// ... and with the output gate's silu: fp32 as written; bf16 shares one reciprocal between the sigmoids
// (inputs clamped at -28, where a sigmoid is below 1e-12), since the scan is bound by these as much as by memory
template <typename E>
__device__ __forceinline__ void gate_out(float zx, float ux, float g, float& z, float& zc, float& sg) {
  if constexpr (Vec<E>::fast) {
    const float ez = 1.f + __expf(fminf(-zx, 28.f)), eu = 1.f + __expf(fminf(-ux, 28.f)), eg = 1.f + __expf(fminf(-g, 28.f));
    const float zu = ez * eu, r = __builtin_amdgcn_rcpf(zu * eg);
    z = r * eu * eg;
    zc = z * (ux >= 0.f ? ux + 0.5f : r * ez * eg);
    sg = g * r * zu;
  } else {
    gate<E>(zx, ux, z, zc);
    sg = g * Vec<E>::sig(g);
  }
}

constexpr int UN = 8;  // tokens whose loads are in flight together

template <typename E, int V>
__global__ void __launch_bounds__(64) scan_sum_kernel(ScanArgs p) {
  const int* ck = p.chunks + blockIdx.y * 6;
  const int row0 = ck[0], n = ck[1], ci = ck[2], nc = ck[3], pos = ck[4], slot = ck[5];
  const int w = (blockIdx.x * 64 + threadIdx.x) * V, W = p.W;
  if (nc == 1 || ci == nc - 1 || w >= W) return;
  float* ws = p.ws + (long long)blockIdx.y * 3 * W + w;
  if (ci == 0) {
    float s0[V];
#pragma unroll
    for (int e = 0; e < V; ++e) s0[e] = 0.f;
    if (pos > 0) ldn<float, V>(p.state + (long long)slot * W + w, s0);
    stn<float, V>(ws + 2 * W, s0);
  }
  float bz[V], bx[V], A[V], B[V];
  ldn<E, V>(reinterpret_cast<const E*>(p.bz) + w, bz);
  ldn<E, V>(reinterpret_cast<const E*>(p.bx) + w, bx);
#pragma unroll
  for (int e = 0; e < V; ++e) A[e] = 1.f, B[e] = 0.f;
  const E* base = reinterpret_cast<const E*>(p.zxg) + (long long)row0 * p.ld + w;
  Raw<E, V> zv[UN], uv[UN];
  auto load = [&](int t0, Raw<E, V>(&z)[UN], Raw<E, V>(&u)[UN]) {
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      const E* q = base + min(t0 + i, n - 1) * p.ld;
      z[i] = *reinterpret_cast<const Raw<E, V>*>(q);
      u[i] = *reinterpret_cast<const Raw<E, V>*>(q + W);
    }
  };
  load(0, zv, uv);
  for (int t0 = 0; t0 < n; t0 += UN) {
    Raw<E, V> zn[UN], un[UN];
    load(t0 + UN, zn, un);
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      if (t0 + i >= n) break;
#pragma unroll
      for (int e = 0; e < V; ++e) {
        float z, zc;
        gate<E>(zv[i].f(e) + bz[e], uv[i].f(e) + bx[e], z, zc);
        A[e] *= 1.f - z;
        B[e] = fmaf(1.f - z, B[e], zc);
      }
    }
#pragma unroll
    for (int i = 0; i < UN; ++i) zv[i] = zn[i], uv[i] = un[i];
  }
  stn<float, V>(ws, A);
  stn<float, V>(ws + W, B);
}

template <typename E, int V>
__global__ void __launch_bounds__(64) scan_run_kernel(ScanArgs p) {
  const int* ck = p.chunks + blockIdx.y * 6;
  const int row0 = ck[0], n = ck[1], ci = ck[2], nc = ck[3], pos = ck[4], slot = ck[5];
  const int w = (blockIdx.x * 64 + threadIdx.x) * V, W = p.W;
  if (w >= W) return;
  float S[V];
#pragma unroll
  for (int e = 0; e < V; ++e) S[e] = 0.f;
  if (nc == 1) {
    if (pos > 0) ldn<float, V>(p.state + (long long)slot * W + w, S);
  } else {
    const float* ws = p.ws + (long long)(blockIdx.y - ci) * 3 * W + w;
    ldn<float, V>(ws + 2 * W, S);
    for (int c0 = 0; c0 < ci; c0 += 4) {
      float A[4][V], B[4][V];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float* q = ws + (long long)min(c0 + i, ci - 1) * 3 * W;
        ldn<float, V>(q, A[i]);
        ldn<float, V>(q + W, B[i]);
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (c0 + i < ci)
#pragma unroll
          for (int e = 0; e < V; ++e) S[e] = fmaf(A[i][e], S[e], B[i][e]);
    }
  }
  float bz[V], bx[V];
  ldn<E, V>(reinterpret_cast<const E*>(p.bz) + w, bz);
  ldn<E, V>(reinterpret_cast<const E*>(p.bx) + w, bx);
  const E* base = reinterpret_cast<const E*>(p.zxg) + (long long)row0 * p.ld + w;
  E* y = reinterpret_cast<E*>(p.y) + (long long)row0 * p.ldy + w;
  Raw<E, V> zv[UN], uv[UN], gv[UN];
  auto load = [&](int t0, Raw<E, V>(&z)[UN], Raw<E, V>(&u)[UN], Raw<E, V>(&g)[UN]) {
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      const E* q = base + min(t0 + i, n - 1) * p.ld;
      z[i] = *reinterpret_cast<const Raw<E, V>*>(q);
      u[i] = *reinterpret_cast<const Raw<E, V>*>(q + W);
      g[i] = *reinterpret_cast<const Raw<E, V>*>(q + 2 * W);
    }
  };
  load(0, zv, uv, gv);
  for (int t0 = 0; t0 < n; t0 += UN) {
    Raw<E, V> zn[UN], un[UN], gn[UN];
    load(t0 + UN, zn, un, gn);
#pragma unroll
    for (int i = 0; i < UN; ++i) {
      if (t0 + i >= n) break;
      float o[V];
#pragma unroll
      for (int e = 0; e < V; ++e) {
        float z, zc, sg;
        gate_out<E>(zv[i].f(e) + bz[e], uv[i].f(e) + bx[e], gv[i].f(e), z, zc, sg);
        S[e] = fmaf(1.f - z, S[e], zc);
        o[e] = S[e] * sg;
      }
      stn<E, V>(y + (t0 + i) * p.ldy, o);
    }
#pragma unroll
    for (int i = 0; i < UN; ++i) zv[i] = zn[i], uv[i] = un[i], gv[i] = gn[i];
  }
  if (ci == nc - 1) stn<float, V>(p.state + (long long)slot * W + w, S);
}

// one token per row (row b of slot[b] at pos[b]): the decode step
template <typename E, int V>
__global__ void __launch_bounds__(64) scan_step_kernel(ScanArgs p, const int* pos, const int* slots) {
  const int b = blockIdx.y, w = (blockIdx.x * 64 + threadIdx.x) * V, W = p.W;
  if (w >= W) return;
  float S[V], z4[V], u4[V], g4[V], bz[V], bx[V], o[V];
  const E* q = reinterpret_cast<const E*>(p.zxg) + (long long)b * p.ld + w;
  ldn<E, V>(q, z4);
  ldn<E, V>(q + W, u4);
  ldn<E, V>(q + 2 * W, g4);
  ldn<E, V>(reinterpret_cast<const E*>(p.bz) + w, bz);
  ldn<E, V>(reinterpret_cast<const E*>(p.bx) + w, bx);
  float* st = p.state + (long long)slots[b] * W + w;
#pragma unroll
  for (int e = 0; e < V; ++e) S[e] = 0.f;
  if (pos[b] > 0) ldn<float, V>(st, S);
#pragma unroll
  for (int e = 0; e < V; ++e) {
    float z, zc, sg;
    gate_out<E>(z4[e] + bz[e], u4[e] + bx[e], g4[e], z, zc, sg);
    S[e] = fmaf(1.f - z, S[e], zc);
    o[e] = S[e] * sg;
  }
  stn<float, V>(st, S);
  stn<E, V>(reinterpret_cast<E*>(p.y) + (long long)b * p.ldy + w, o);
}

template <typename E, int V>
int launch(const ScanArgs& a, int multi, hipStream_t s) {
  const dim3 g((a.W + 64 * V - 1) / (64 * V), a.nchunk);
  if (multi) hipLaunchKernelGGL((scan_sum_kernel<E, V>), g, dim3(64), 0, s, a);
  hipLaunchKernelGGL((scan_run_kernel<E, V>), g, dim3(64), 0, s, a);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

template <typename E, int V>
int launch_step(const ScanArgs& a, const int* pos, const int* slots, hipStream_t s) {
  hipLaunchKernelGGL((scan_step_kernel<E, V>), dim3((a.W + 64 * V - 1) / (64 * V), a.nchunk), dim3(64), 0, s, a, pos,
                     slots);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

}  // namespace

// dtype: 0 fp32, 1 bf16. multi: some portion has more than one chunk (ws: nchunk * 3 * W floats).
KCA_API int kca_gated_scan(int dtype, const void* zxg, long long ld, const void* bz, const void* bx, void* y,
                           long long ldy, void* state, void* ws, long long ws_floats, const void* chunks, int nchunk,
                           int multi, int W, hipStream_t s) {
  if (nchunk < 1 || nchunk > 65535 || W < 1 || !zxg || !bz || !bx || !y || !state || !chunks) return 1;
  if (multi && (!ws || ws_floats < (long long)nchunk * 3 * W)) return 2;
  const ScanArgs a{zxg, ld, bz, bx, y, ldy, (float*)state, (float*)ws, (const int*)chunks, W, nchunk};
  // two channels a thread: the scan's waves are few, four would halve them again
  const bool v2 = W % 2 == 0 && ld % 2 == 0 && ldy % 2 == 0 && (uintptr_t)y % 8 == 0 && (uintptr_t)zxg % 8 == 0;
  if (dtype == 0) return v2 ? launch<float, 2>(a, multi, s) : launch<float, 1>(a, multi, s);
  if (dtype == 1) return v2 ? launch<bf16_t, 2>(a, multi, s) : launch<bf16_t, 1>(a, multi, s);
  return 3;
}

KCA_API int kca_gated_step(int dtype, const void* zxg, long long ld, const void* bz, const void* bx, void* y,
                           long long ldy, void* state, const void* pos, const void* slots, int B, int W,
                           hipStream_t s) {
  if (B < 1 || B > 65535 || W < 1 || !zxg || !bz || !bx || !y || !state || !pos || !slots) return 1;
  const ScanArgs a{zxg, ld, bz, bx, y, ldy, (float*)state, nullptr, nullptr, W, B};
  const int *ps = (const int*)pos, *sl = (const int*)slots;
  const bool v4 = W % 4 == 0 && ld % 4 == 0 && ldy % 4 == 0 && (uintptr_t)y % 16 == 0;
  if (dtype == 0) return v4 ? launch_step<float, 4>(a, ps, sl, s) : launch_step<float, 1>(a, ps, sl, s);
  if (dtype == 1) return v4 ? launch_step<bf16_t, 4>(a, ps, sl, s) : launch_step<bf16_t, 1>(a, ps, sl, s);
  return 3;
}
