// Matrix memory with exponential gates (matrix_memory.hip): arguments, and one token of one head.
#pragma once
#include "delta_rule.h"
#include "state_cols.h"

namespace {
using delta::sigmoid;
using delta::softplus;

struct MemArgs {
  const void* x;            // projection rows, row stride ld; column offsets below
  long long ld;
  int o_q, o_k, o_v, o_g, o_i, o_f;
  int H, dk, dv;
  const void* ib;           // [H] biases of the input and forget gates
  const void* fb;
  const void* gain;         // [H dv]
  float cap, qscale, eps, mul;
  float* state;             // [slots][H][dk][dv]
  float* norm;              // [slots][H][dk]
  float* top;               // [slots][H]
  float* norm1;             // what scan and run leave
  float* top1;
  const int* pos;           // [T]
  const int* slot;          // [T]
  const int* e1;            // [T] one past the last row of the token's entry
  void* out;                // rows [H dv], row stride ldo
  long long ldo;
  void* o;                  // read-outs [T][H dv] in the compute type
  const int* ent;           // scan: [n][5] first row, rows, position, slot, -
  const int* ck;            // map: [nchunk][4] first row, rows, -, -
  const int* en;            // run: [n][6] first row, rows, position, slot, first chunk, chunks
  // operands as the run kernel's lanes read them; eight token slots e of lane group g hold the tokens 32 k + 4 g + e
  // (e < 4) and 32 k + 16 + 4 g + e - 4
  bf16_t* am;               // [nchunk][H][4][2][64 lanes][8]: A, t = 16 I + (lane & 15), tokens j of step k
  bf16_t* kt;               // [nchunk][H][DK / 16][2][64 lanes][8]: K'_j[c = 16 m + (lane & 15)]
  float* gd;                // [nchunk][H][3 * 64 + DK]: c, F, row sums of A; sum of K'
};

struct Gates { float i, f; };
template <typename E>
__device__ __forceinline__ Gates gates(const MemArgs& a, const E* x, int h) {
  const float zi = delta::ld<E>(x + a.o_i + h) + delta::ld<E>(reinterpret_cast<const E*>(a.ib) + h);
  const float zf = delta::ld<E>(x + a.o_f + h) + delta::ld<E>(reinterpret_cast<const E*>(a.fb) + h);
  return {a.cap * tanhf(zi / a.cap), -softplus(-a.cap * tanhf(zf / a.cap))};
}

// rows rg + 16 i of a projected vector (zero past dk)
template <typename E, int R>
__device__ __forceinline__ void rows_x(const E* src, int dk, int rg, float mul, float (&x)[R]) {
#pragma unroll
  for (int i = 0; i < R; ++i) x[i] = rg + 16 * i < dk ? delta::ld<E>(src + rg + 16 * i) * mul : 0.f;
}

// One token of the scalars and the normaliser: -> decay of the state, e^(i - m) (k is scaled in place), divisor
template <int R>
__device__ __forceinline__ float advance(Gates g, float& m, float (&n)[R], float (&k)[R], const float (&q)[R], float& w, float& qk) {
  const float top = fmaxf(g.f + m, g.i), put = expf(g.i - top);
  w = expf(g.f + m - top);
  m = top;
  float nq = 0.f;
  qk = 0.f;
#pragma unroll
  for (int i = 0; i < R; ++i) {
    k[i] *= put;
    n[i] = fmaf(w, n[i], k[i]);
    nq = fmaf(n[i], q[i], nq);
    qk = fmaf(k[i], q[i], qk);
  }
  auto add = [](float x, float y) { return x + y; };
  nq = lanes_reduce<16>(nq, add);
  qk = lanes_reduce<16>(qk, add);
  return 1.f / (fmaxf(fabsf(nq), expf(-m)) + 1e-6f);
}

// One token of row b, head h. vals: [dv] read-outs, red: a float a wave (LDS)
template <typename E, int R, int CW>
__device__ __forceinline__ void step_body(const MemArgs& a, int b, int h, float* vals, float* red) {
  const int tid = threadIdx.x, wv = tid >> 6, lane = tid & 63, nw = blockDim.x >> 6;
  const int dk = a.dk, dv = a.dv, rg = lane & 15, cg = lane >> 4, nblk = (dv + 4 * CW - 1) / (4 * CW);
  const long long sh = (long long)a.slot[b] * a.H + h;
  float* S = a.state + sh * dk * dv;
  const bool live = a.pos[b] > 0;
  Cols<R, CW> st;
  st.load(S, dk, dv, rg, wv * 4 * CW + cg * CW, live);
  const E* x = reinterpret_cast<const E*>(a.x) + (long long)b * a.ld;
  float n[R], k[R], q[R], w, qk, m = live ? a.top[sh] : 0.f;
#pragma unroll
  for (int i = 0; i < R; ++i) n[i] = live && rg + 16 * i < dk ? a.norm[sh * dk + rg + 16 * i] : 0.f;
  rows_x<E, R>(x + a.o_k + h * dk, dk, rg, 1.f, k);
  rows_x<E, R>(x + a.o_q + h * dk, dk, rg, a.qscale, q);
  const float inv = advance<R>(gates<E>(a, x, h), m, n, k, q, w, qk);
  float ss = 0.f;
  for (int cb = wv; cb < nblk; cb += nw) {
    const int col = cb * 4 * CW + cg * CW;
    if (cb != wv) st.load(S, dk, dv, rg, col, live);
    float v[CW], o[CW];
#pragma unroll
    for (int e = 0; e < CW; ++e) v[e] = col + e < dv ? delta::ld<E>(x + a.o_v + h * dv + col + e) : 0.f;
    st.decayed(w, k, q, v, qk, o);
    st.store(S, dk, dv, rg, col);
    if (rg == 0)
#pragma unroll
      for (int e = 0; e < CW; ++e)
        if (col + e < dv) {
          const float y = o[e] * inv;
          vals[col + e] = y;
          ss = fmaf(y, y, ss);
        }
  }
  ss = wave_sum(ss);
  if (lane == 0) red[wv] = ss;
  __syncthreads();  // (and every wave has read n and m)
  if (wv == 0 && cg == 0) {
#pragma unroll
    for (int i = 0; i < R; ++i)
      if (rg + 16 * i < dk) a.norm[sh * dk + rg + 16 * i] = n[i];
    if (rg == 0) a.top[sh] = m;
  }
  ss = 0.f;
  for (int i = 0; i < nw; ++i) ss += red[i];
  const float r = a.mul / sqrtf(ss / (float)dv + a.eps);
  E* out = reinterpret_cast<E*>(a.out) + (long long)b * a.ldo + h * dv;
  const E *gain = reinterpret_cast<const E*>(a.gain) + h * dv, *g = x + a.o_g + h * dv;
  for (int c = tid; c < dv; c += blockDim.x) delta::st<E>(out + c, vals[c] * r * delta::ld<E>(gain + c) * sigmoid(delta::ld<E>(g + c)));
}

static bool wide(const MemArgs& a) { return a.dv % 4 == 0 && (uintptr_t)a.state % 16 == 0; }

static bool mem_ok(const MemArgs& a) {
  const long long ends[6] = {a.o_q + (long long)a.H * a.dk, a.o_k + (long long)a.H * a.dk, a.o_v + (long long)a.H * a.dv,
                             a.o_g + (long long)a.H * a.dv, a.o_i + (long long)a.H, a.o_f + (long long)a.H};
  for (long long e : ends)
    if (e > a.ld) return false;
  return a.H >= 1 && a.H <= 65535 && a.dk >= 1 && a.dv >= 1 && a.dk <= 256 && a.dv <= 1024 && a.cap > 0.f && a.x && a.ib && a.fb && a.gain &&
         a.state && a.norm && a.top && a.pos && a.slot && a.o_q >= 0 && a.o_k >= 0 && a.o_v >= 0 && a.o_g >= 0 && a.o_i >= 0 && a.o_f >= 0;
}

}  // namespace
