// Delta-rule token mixers: per head a state S [dk][dv] of a sequence follows
//   S_t = diag(w_t) S_(t-1) + p_t (z_t^T S_(t-1)) + k_t v_t^T,     o_t = S_t^T q_t
// KIND 0 (general): w = exp(-e^(-1/2) sigmoid(lw + w0)), u = k / sqrt(|k|^2 + 1e-6), z = u, p = -(a u),
//   a = sigmoid(.. + ab); q, k, v are projections; lw a two-step projection with a tanh between.
// KIND 1 (channel): q, k, v pass a short causal convolution and silu; q (times qscale) and k become unit
//   vectors, shared by the H / G heads of a group; w = exp(-exp(A) softplus(lw + dt)), z = w k,
//   p = -beta k, k <- beta k.
// The read-out is RMS-normed per head, times a gain, times sigmoid(gate).
// Everything after the projections is fp32. `prep_head` derives one head's vectors of one token in LDS.
#pragma once
#include "common.h"
#include "lanes.h"

struct DeltaArgs {
  const void* x;            // projection rows, row stride ld; column offsets below
  long long ld;
  int o_q, o_k, o_v, o_a, o_g, o_w;  // a: removal logits | beta logits; g: gate logits | its inner; w: decay inner
  int H, G, dk, dv, taps, rank_w, rank_g;
  const void* lo_w;         // [H dk][rank_w] second step of the decay projection
  const void* lo_g;         // [H dv][rank_g] ... of the gate (KIND 1)
  const void* dw;           // its result rows [T][H dk] where a GEMM made them (row stride ldw)
  long long ldw;
  const void* dg;           // [T][H dv]
  long long ldg;
  const void* w0;           // [H dk]: w0 | dt bias
  const void* ab;           // a's bias [H dk] | A [H]
  const void* conv;         // [2 G dk + H dv][taps], last column the current token's
  const void* gain;         // [H dv] | [dv]
  float eps, qscale;
  float* state;             // [slots][H][dk][dv]
  float* ring;              // [slots][taps][2 G dk + H dv]: convolution inputs, position p in row p % taps
  const int* pos;           // [T]
  const int* slot;          // [T]
  const int* e0;            // [T] first row of the token's entry in this batch (nullable: the row itself)
  const int* e1;            // [T] one past its last row
  void* out;                // rows [H dv], row stride ldo
  long long ldo;
  const int* rows;          // prep kernel: token row of prepared row b (nullable: b)
  float* pk;                // prepared vectors [rows][H][pk_stride]: w z p k q [dk], v [dv], q.p, q.k
  float* o;                 // read-outs [T][H dv]
  const int* ent;           // scan kernel: [n][5]: first row, rows, position of the first row, slot, first prepared row
};

namespace delta {

template <typename E> __device__ __forceinline__ float ld(const E* p);
template <> __device__ __forceinline__ float ld<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ld<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <typename E> __device__ __forceinline__ void st(E* p, float v);
template <> __device__ __forceinline__ void st<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void st<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }
template <typename E>
__device__ __forceinline__ float tanh_t(float v) {
  if constexpr (sizeof(E) == 4) return tanhf(v);
  else return fast_tanh(v);
}

__device__ __forceinline__ float sigmoid(float v) { return 1.f / (1.f + expf(-v)); }
__device__ __forceinline__ float softplus(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }
__host__ __device__ __forceinline__ int pk_stride(int dk, int dv) { return (5 * dk + dv + 2 + 3) & ~3; }

// log decay of one (head, key channel) from the second step's result
template <int KIND>
__device__ __forceinline__ float log_decay(float lw, float w0, float A) {
  if constexpr (KIND == 0) return -0.60653065971263342f * sigmoid(lw + w0);
  else return -expf(A) * softplus(lw + w0);
}

// silu(convolution) of input column `col` (convolution channel ch) at row t
template <typename E>
__device__ __forceinline__ float conv_silu(const DeltaArgs& a, int t, int col, int ch) {
  const int pos = a.pos[t], back = a.e0 ? t - a.e0[t] : 0, C = 2 * a.G * a.dk + a.H * a.dv;
  const E* x = reinterpret_cast<const E*>(a.x) + (long long)t * a.ld + col;
  const E* w = reinterpret_cast<const E*>(a.conv) + (long long)ch * a.taps + a.taps - 1;
  float y = 0.f;
  for (int i = 0; i < a.taps && i <= pos; ++i) {
    const float v = i <= back ? ld<E>(x - i * a.ld)
                              : a.ring[((long long)a.slot[t] * a.taps + (pos - i) % a.taps) * C + ch];
    y = fmaf(ld<E>(w - i), v, y);
  }
  return y / (1.f + expf(-y));
}

// what position t leaves for the convolution of later tokens; `lane` of `n` threads
template <typename E>
__device__ __forceinline__ void ring_store(const DeltaArgs& a, int t, int h, int lane, int n) {
  const int C = 2 * a.G * a.dk + a.H * a.dv, per = a.H / a.G, g = h / per;
  float* r = a.ring + ((long long)a.slot[t] * a.taps + a.pos[t] % a.taps) * C;
  const E* x = reinterpret_cast<const E*>(a.x) + (long long)t * a.ld;
  for (int c = lane; c < a.dv; c += n) r[2 * a.G * a.dk + h * a.dv + c] = ld<E>(x + a.o_v + h * a.dv + c);
  if (h % per == 0)
    for (int c = lane; c < a.dk; c += n) {
      r[g * a.dk + c] = ld<E>(x + a.o_q + g * a.dk + c);
      r[(a.G + g) * a.dk + c] = ld<E>(x + a.o_k + g * a.dk + c);
    }
}

// LDS of one head: floats
__host__ __device__ __forceinline__ int prep_floats(int dk, int dv, int rw, int rg) { return 5 * dk + 2 * dv + rw + rg + 32; }

struct Head {
  float *w, *z, *p, *k, *q, *v, *gate, *tw, *tg, *red;
  float qp, qk;
  __device__ __forceinline__ Head(float* m, int dk, int dv, int rw, int rg) {
    w = m; z = w + dk; p = z + dk; k = p + dk; q = k + dk; v = q + dk; gate = v + dv; tw = gate + dv; tg = tw + rw;
    red = tg + rg;
  }
};

// dot of a low-rank row with an LDS vector, 4 consecutive lanes each; all of them get it
template <typename E>
__device__ __forceinline__ float dot4(const E* row, const float* v, int n, int sub) {
  float s = 0.f;
  if (n % 8 == 0 && ((uintptr_t)row & 15) == 0 && sizeof(E) == 2) {
    for (int i = sub * 8; i < n; i += 32) {
      const U16x8 u = *reinterpret_cast<const U16x8*>(row + i);
#pragma unroll
      for (int e = 0; e < 8; ++e) s = fmaf(bf2f(u.v[e]), v[i + e], s);
    }
  } else {
    for (int i = sub; i < n; i += 4) s = fmaf(ld<E>(row + i), v[i], s);
  }
  return lanes_reduce<4>(s, [](float x, float y) { return x + y; });
}

// vectors of (token row t, head h) in LDS, by the whole workgroup of NT threads
template <typename E, int KIND>
__device__ __forceinline__ void prep_head(const DeltaArgs& a, int t, int h, Head& s) {
  const int tid = threadIdx.x, NT = blockDim.x, dk = a.dk, dv = a.dv, sub = tid & 3;
  const E* x = reinterpret_cast<const E*>(a.x) + (long long)t * a.ld;
  const int g = h / (a.H / a.G), nqk = a.G * dk;
  if (!a.dw)
    for (int i = tid; i < a.rank_w; i += NT) {
      const float v = ld<E>(x + a.o_w + i);
      s.tw[i] = KIND == 0 ? tanh_t<E>(v) : v;
    }
  if (KIND == 1 && !a.dg)
    for (int i = tid; i < a.rank_g; i += NT) s.tg[i] = ld<E>(x + a.o_g + i);
  float sk = 0.f, sq = 0.f;
  for (int c = tid; c < dk; c += NT) {
    float q, k;
    if constexpr (KIND == 0) {
      q = ld<E>(x + a.o_q + h * dk + c);
      k = ld<E>(x + a.o_k + h * dk + c);
    } else {
      q = conv_silu<E>(a, t, a.o_q + g * dk + c, g * dk + c);
      k = conv_silu<E>(a, t, a.o_k + g * dk + c, nqk + g * dk + c);
    }
    s.q[c] = q;
    s.k[c] = k;
    sk = fmaf(k, k, sk);
    sq = fmaf(q, q, sq);
  }
  for (int c = tid; c < dv; c += NT) {
    if constexpr (KIND == 0) s.v[c] = ld<E>(x + a.o_v + h * dv + c);
    else s.v[c] = conv_silu<E>(a, t, a.o_v + h * dv + c, 2 * nqk + h * dv + c);
  }
  const float ik = 1.f / sqrtf(block_sum(sk, s.red) + 1e-6f);  // (its barriers also publish tw, tg)
  const float iq = KIND == 1 ? a.qscale / sqrtf(block_sum(sq, s.red + 16) + 1e-6f) : 1.f;
  float A = 0.f, beta = 0.f;
  if constexpr (KIND == 1) {
    A = ld<E>(reinterpret_cast<const E*>(a.ab) + h);
    beta = sigmoid(ld<E>(x + a.o_a + h));
  }
  // decays (and, channel, gates): four lanes a dot
  const int ndot = a.dw ? 0 : dk, ng = (KIND == 1 && !a.dg) ? dv : 0;
  for (int i0 = 0; i0 < ndot + ng; i0 += NT / 4) {
    const int i = i0 + tid / 4;
    if (i < ndot) {
      const float d = dot4<E>(reinterpret_cast<const E*>(a.lo_w) + (long long)(h * dk + i) * a.rank_w, s.tw, a.rank_w, sub);
      if (sub == 0) s.w[i] = d;
    } else if (i < ndot + ng) {
      const int c = i - ndot;
      const float d = dot4<E>(reinterpret_cast<const E*>(a.lo_g) + (long long)(h * dv + c) * a.rank_g, s.tg, a.rank_g, sub);
      if (sub == 0) s.gate[c] = sigmoid(d);
    }
  }
  __syncthreads();
  float qp = 0.f, qk = 0.f;
  for (int c = tid; c < dk; c += NT) {
    const float lw = a.dw ? ld<E>(reinterpret_cast<const E*>(a.dw) + (long long)t * a.ldw + h * dk + c) : s.w[c];
    const float w = expf(log_decay<KIND>(lw, ld<E>(reinterpret_cast<const E*>(a.w0) + h * dk + c), A));
    const float k = s.k[c], u = k * ik, q = s.q[c] * iq;
    float p, kw = k;
    if constexpr (KIND == 0) {
      p = -u * sigmoid(ld<E>(x + a.o_a + h * dk + c) + ld<E>(reinterpret_cast<const E*>(a.ab) + h * dk + c));
      s.z[c] = u;
    } else {
      kw = beta * u;
      p = -kw;
      s.z[c] = w * u;
    }
    s.w[c] = w;
    s.p[c] = p;
    s.k[c] = kw;
    s.q[c] = q;
    qp = fmaf(q, p, qp);
    qk = fmaf(q, kw, qk);
  }
  for (int c = tid; c < dv; c += NT) {
    if constexpr (KIND == 0) s.gate[c] = sigmoid(ld<E>(x + a.o_g + h * dv + c));
    else if (a.dg) s.gate[c] = sigmoid(ld<E>(reinterpret_cast<const E*>(a.dg) + (long long)t * a.ldg + h * dv + c));
  }
  s.qp = block_sum(qp, s.red);
  s.qk = block_sum(qk, s.red + 16);  // (and the vectors are visible to the workgroup)
}

}  // namespace delta

static inline bool delta_args_ok(const DeltaArgs& a, int kind) {
  if ((kind != 0 && kind != 1) || a.H < 1 || a.G < 1 || a.H % a.G || a.dk < 1 || a.dv < 1 || a.dk > 256 || a.dv > 1024) return false;
  if (!a.x || !a.w0 || !a.ab || !a.gain || !a.state || !a.pos || !a.slot || !a.out) return false;
  if (a.rank_w < 1 || (!a.dw && !a.lo_w)) return false;
  if (kind == 0) return a.G == a.H && a.dk == a.dv;
  return a.conv && a.ring && a.taps >= 1 && a.rank_g >= 1 && (a.dg || a.lo_g);
}
