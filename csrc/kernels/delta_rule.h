// Delta-rule token mixers: per head a state S [dk][dv] of a sequence follows
//   S_t = diag(w_t) S_(t-1) + p_t (z_t^T S_(t-1)) + k_t v_t^T,     o_t = S_t^T q_t
// KIND 0 (general): w = exp(-e^(-1/2) sigmoid(lw + w0)), u = k / sqrt(|k|^2 + 1e-6), z = u, p = -(a u),
//   a = sigmoid(.. + ab); q, k, v are projections; lw a two-step projection with a tanh between.
// KIND 1 (channel): q, k, v pass a short causal convolution and silu; q (times qscale) and k become unit
//   vectors, shared by the H / G heads of a group; w = exp(-exp(A) softplus(lw + dt)), z = w k,
//   p = -beta k, k <- beta k.
// KIND 2 (head): as 1, with one decay per head, exp(-exp(A) softplus(lw + dt)), lw a projection itself.
// KIND 3 (state space): q, k, v are C, B, x after the convolution (with a bias) and silu; with dt = softplus(lw + bias)
//   w = exp(-exp(A) dt), k <- dt k, p = z = 0, and the read-out adds D v.
// KIND 0 - 2: the read-out is RMS-normed per head, times a gain, times sigmoid(gate) (2: silu). KIND 3: times
// silu(gate), then RMS-normed in equal parts of all heads, times a gain.
// Everything after the projections is fp32. `prep_head` derives one head's vectors of one token in LDS.
// KIND 2 and 3 portions read convolution results that a kernel of their own made (`cx`).
#pragma once
#include "common.h"
#include "lanes.h"

struct DeltaArgs {
  const void* x;            // projection rows, row stride ld; column offsets below
  long long ld;
  int o_q, o_k, o_v, o_a, o_g, o_w;  // a: removal logits | beta logits; g: gate logits | its inner; w: decay inner | logits
  int H, G, dk, dv, taps, rank_w, rank_g;
  const void* lo_w;         // [H dk][rank_w] second step of the decay projection
  const void* lo_g;         // [H dv][rank_g] ... of the gate (KIND 1)
  const void* dw;           // its result rows [T][H dk] where a GEMM made them (row stride ldw)
  long long ldw;
  const void* dg;           // [T][H dv]
  long long ldg;
  const void* w0;           // [H dk]: w0 | dt bias (KIND 2, 3: [H])
  const void* ab;           // a's bias [H dk] | A [H]
  const void* conv;         // [2 G dk + H dv][taps], last column the current token's
  const void* gain;         // [H dv] (KIND 0, 3) | [dv]
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
  void* o;                  // read-outs [T][H dv] in the compute type
  const int* ent;           // scan kernel: [n][5]: first row, rows, position of the first row, slot, first prepared row
  const void* cx;           // KIND 2, 3: rows [T][2 G dk + H dv] after convolution and silu (nullable: convolve here)
  const void* convb;        // [2 G dk + H dv] its bias (nullable)
  const void* skip;         // [H] D (nullable)
  int norm_groups;          // KIND 3: equal parts of the closing norm
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
__device__ __forceinline__ float silu(float v) { return v / (1.f + expf(-v)); }
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
  const int pos = a.pos[t], C = 2 * a.G * a.dk + a.H * a.dv;
  const E* x = reinterpret_cast<const E*>(a.x) + (long long)t * a.ld + col;
  const E* w = reinterpret_cast<const E*>(a.conv) + (long long)ch * a.taps + a.taps - 1;
  const float* r = a.ring + (long long)a.slot[t] * a.taps * C + ch;
  float y = ld<E>(w) * ld<E>(x);
  if (a.convb) y += ld<E>(reinterpret_cast<const E*>(a.convb) + ch);
  if (!a.e0 && a.taps <= 4) {  // one token an entry: the loads of all taps fly together
    float v[3], c[3];
#pragma unroll
    for (int i = 1; i < 4; ++i) {
      const bool ok = i < a.taps && i <= pos;
      v[i - 1] = r[(ok ? (pos - i) % a.taps : 0) * C];
      c[i - 1] = ld<E>(w - (i < a.taps ? i : 0));
      if (!ok) c[i - 1] = 0.f, v[i - 1] = 0.f;
    }
#pragma unroll
    for (int i = 0; i < 3; ++i) y = fmaf(c[i], v[i], y);
  } else {
    const int back = a.e0 ? t - a.e0[t] : 0;
    for (int i = 1; i < a.taps && i <= pos; ++i)
      y = fmaf(ld<E>(w - i), i <= back ? ld<E>(x - i * a.ld) : r[((pos - i) % a.taps) * C], y);
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
__host__ __device__ __forceinline__ int prep_floats(int dk, int dv, int rw, int rg) { return 5 * dk + 2 * dv + rw + rg + 64; }

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

// sums of two values over the workgroup; `red` holds 2 floats a wave
__device__ __forceinline__ void block_sum2(float& x, float& y, float* red) {
  x = wave_sum(x);
  y = wave_sum(y);
  if ((threadIdx.x & 63) == 0) red[2 * (threadIdx.x >> 6)] = x, red[2 * (threadIdx.x >> 6) + 1] = y;
  __syncthreads();
  x = y = 0.f;
  for (int i = 0; i < (int)(blockDim.x >> 6); ++i) x += red[2 * i], y += red[2 * i + 1];
}

// vectors of (token row t, head h) in LDS, by a workgroup of at least max(256, dk) threads
template <typename E, int KIND>
__device__ __forceinline__ void prep_head(const DeltaArgs& a, int t, int h, Head& s) {
  const int tid = threadIdx.x, NT = blockDim.x, dk = a.dk, dv = a.dv, sub = tid & 3;
  const E* x = reinterpret_cast<const E*>(a.x) + (long long)t * a.ld;
  const int g = h / (a.H / a.G), nqk = a.G * dk;
  // loads whose results are needed late
  const int cs = tid < dk ? tid : 0;
  const float w0 = ld<E>(reinterpret_cast<const E*>(a.w0) + (KIND >= 2 ? h : h * dk + cs));
  float al = 0.f, ab = 0.f, lh = 0.f;
  if constexpr (KIND == 0) {
    al = ld<E>(x + a.o_a + h * dk + cs);
    ab = ld<E>(reinterpret_cast<const E*>(a.ab) + h * dk + cs);
  } else {
    if constexpr (KIND < 3) al = ld<E>(x + a.o_a + h);
    if constexpr (KIND >= 2) lh = ld<E>(x + a.o_w + h);
    ab = ld<E>(reinterpret_cast<const E*>(a.ab) + h);
  }
  const bool low = KIND < 2 && !a.dw;  // second steps of the projections here
  const int ndot = low ? dk : 0, ng = (KIND == 1 && !a.dg) ? dv : 0, rw = a.rank_w, rg = a.rank_g;
  // a convolution channel: its column of x, its place among the channels
  auto conv = [&](int col, int ch) {
    if (KIND >= 2 && a.cx) return ld<E>(reinterpret_cast<const E*>(a.cx) + (long long)t * (2 * nqk + a.H * dv) + ch);
    return conv_silu<E>(a, t, col, ch);
  };
  auto dot_row = [&](int i) {
    return i < ndot ? reinterpret_cast<const E*>(a.lo_w) + (long long)(h * dk + i) * rw
                    : reinterpret_cast<const E*>(a.lo_g) + (long long)(h * dv + i - ndot) * rg;
  };
  // the first turn's low-rank rows
  U16x8 pre[4];
  const int i0 = tid / 4, n0 = i0 < ndot ? rw : rg;
  const bool fast = sizeof(E) == 2 && i0 < ndot + ng && n0 % 8 == 0 && n0 <= 128 &&
                    ((uintptr_t)a.lo_w & 15) == 0 && ((uintptr_t)a.lo_g & 15) == 0;
  if (fast) {
    const E* row = dot_row(i0);
#pragma unroll
    for (int j = 0; j < 4; ++j) pre[j] = *reinterpret_cast<const U16x8*>(row + (8 * sub + 32 * j < n0 ? 8 * sub + 32 * j : 0));
  }
  float sk = 0.f, sq = 0.f;
  const int items = 2 * dk + dv + (low ? rw : 0) + (KIND == 1 && !a.dg ? rg : 0);
  for (int i = tid; i < items; i += NT) {
    if (i < 2 * dk) {
      const bool key = i >= dk;
      const int c = key ? i - dk : i;
      float v;
      if constexpr (KIND == 0) v = ld<E>(x + (key ? a.o_k : a.o_q) + h * dk + c);
      else v = conv((key ? a.o_k : a.o_q) + g * dk + c, (key ? nqk : 0) + g * dk + c);
      (key ? s.k : s.q)[c] = v;
      if (key) sk = fmaf(v, v, sk);
      else sq = fmaf(v, v, sq);
    } else if (i < 2 * dk + dv) {
      const int c = i - 2 * dk;
      if constexpr (KIND == 0) {
        s.v[c] = ld<E>(x + a.o_v + h * dv + c);
        s.gate[c] = sigmoid(ld<E>(x + a.o_g + h * dv + c));
      } else {
        s.v[c] = conv(a.o_v + h * dv + c, 2 * nqk + h * dv + c);
        if constexpr (KIND == 2) s.gate[c] = silu(ld<E>(x + a.o_g + h * dv + c));
        if (KIND == 1 && a.dg) s.gate[c] = sigmoid(ld<E>(reinterpret_cast<const E*>(a.dg) + (long long)t * a.ldg + h * dv + c));
      }
    } else {
      const int c = i - 2 * dk - dv;
      if (low && c < rw) {
        const float v = ld<E>(x + a.o_w + c);
        s.tw[c] = KIND == 0 ? tanh_t<E>(v) : v;
      } else {
        s.tg[c - (low ? rw : 0)] = ld<E>(x + a.o_g + c - (low ? rw : 0));
      }
    }
  }
  block_sum2(sk, sq, s.red);  // (its barrier also publishes the vectors so far)
  const float ik = KIND == 3 ? 1.f : 1.f / sqrtf(sk + 1e-6f);
  const float iq = KIND == 1 || KIND == 2 ? a.qscale / sqrtf(sq + 1e-6f) : 1.f;
  // decays (and, channel, gates): four lanes a dot
  for (int i = i0; i < ndot + ng; i += NT / 4) {
    const bool dec = i < ndot;
    const int n = dec ? rw : rg;
    const float* v = dec ? s.tw : s.tg;
    float d = 0.f;
    if (fast && i == i0) {
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int o = 8 * sub + 32 * j;
        if (o < n)
#pragma unroll
          for (int e = 0; e < 8; ++e) d = fmaf(bf2f(pre[j].v[e]), v[o + e], d);
      }
      d = lanes_reduce<4>(d, [](float p, float q) { return p + q; });
    } else {
      d = dot4<E>(dot_row(i), v, n, sub);
    }
    if (sub == 0) {
      if (dec) s.w[i] = d;
      else s.gate[i - ndot] = sigmoid(d);
    }
  }
  __syncthreads();
  float qp = 0.f, qk = 0.f;
  if (tid < dk) {
    const int c = tid;
    const float lw = KIND >= 2 ? lh : a.dw ? ld<E>(reinterpret_cast<const E*>(a.dw) + (long long)t * a.ldw + h * dk + c) : s.w[c];
    const float w = expf(log_decay<KIND>(lw, w0, ab));
    const float k = s.k[c], u = k * ik, q = s.q[c] * iq;
    float p, kw = k;
    if constexpr (KIND == 0) {
      p = -u * sigmoid(al + ab);
      s.z[c] = u;
    } else if constexpr (KIND == 3) {
      kw = k * softplus(lw + w0);
      p = s.z[c] = 0.f;
    } else {
      kw = sigmoid(al) * u;
      p = -kw;
      s.z[c] = w * u;
    }
    s.w[c] = w;
    s.p[c] = p;
    s.k[c] = kw;
    s.q[c] = q;
    qp = q * p;
    qk = q * kw;
  }
  block_sum2(qp, qk, s.red + 32);  // (and the vectors are visible to the workgroup)
  s.qp = qp;
  s.qk = qk;
}

}  // namespace delta

static inline bool delta_args_ok(const DeltaArgs& a, int kind) {
  if (kind < 0 || kind > 3 || a.H < 1 || a.G < 1 || a.H % a.G || a.dk < 1 || a.dv < 1 || a.dk > 256 || a.dv > 1024) return false;
  if (!a.x || !a.w0 || !a.ab || !a.gain || !a.state || !a.pos || !a.slot || !a.out) return false;
  if (kind >= 2)
    return a.conv && a.ring && a.taps >= 1 && a.rank_w == 0 && a.rank_g == 0 &&
           (kind == 2 || (a.skip && a.norm_groups >= 1 && (a.H * a.dv) % a.norm_groups == 0));
  if (a.rank_w < 1 || (!a.dw && !a.lo_w)) return false;
  if (kind == 0) return a.G == a.H && a.dk == a.dv;
  return a.conv && a.ring && a.taps >= 1 && a.rank_g >= 1 && (a.dg || a.lo_g);
}
