// Delta-rule mixers (delta_rule.h) token by token: the decode step, and the scan of prompt portions in any
// size or type (bf16 portions of usual head sizes run in chunks on the matrix cores: delta_chunk.hip).
//
//   step kernel   one token per row: projections -> vectors -> state update -> normed, gated output, one launch
//                 (KIND 3: read-outs; the parts kernel norms them)
//   conv kernel   KIND 2, 3: convolution and silu of every row of a batch of portions
//   prep kernel   vectors of every (token, head) of a batch of portions
//   scan kernel   an entry's tokens in order, state in registers; a wave owns 16 value columns of a head
//   gate kernel   head norm, gain and gate of every (token, head); convolution inputs into the slots' rings
//   parts kernel  KIND 3: gate and norm over equal parts of all heads; convolution inputs likewise
//
// The carried state of a sequence lives in its slot and counts as zero at position 0.
#include "delta_rule.h"
#include "state_cols.h"

namespace {
using namespace delta;

template <typename E, int KIND, int R, int CW>
__global__ void __launch_bounds__(R > 8 ? 512 : 1024) delta_step_kernel(DeltaArgs a) {
  extern __shared__ float smem[];
  const int b = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, wv = tid >> 6, lane = tid & 63, nw = blockDim.x >> 6;
  const int dk = a.dk, dv = a.dv, rg = lane & 15, cg = lane >> 4;
  const int nblk = (dv + 4 * CW - 1) / (4 * CW);
  float* S = a.state + ((long long)a.slot[b] * a.H + h) * dk * dv;
  const bool live = a.pos[b] > 0;
  Cols<R, CW> st;
  st.load(S, dk, dv, rg, wv * 4 * CW + cg * CW, live);  // in flight while the vectors are made
  Head hd(smem, dk, dv, a.rank_w, a.rank_g);
  prep_head<E, KIND>(a, b, h, hd);
  if constexpr (KIND >= 1) ring_store<E>(a, b, h, tid, blockDim.x);
  const float skip = KIND == 3 ? delta::ld<E>(reinterpret_cast<const E*>(a.skip) + h) : 0.f;
  float w[R], z[R], p[R], k[R], q[R];
  rows_of<R>(hd.w, dk, rg, w);
  rows_of<R>(hd.z, dk, rg, z);
  rows_of<R>(hd.p, dk, rg, p);
  rows_of<R>(hd.k, dk, rg, k);
  rows_of<R>(hd.q, dk, rg, q);
  float ss = 0.f;
  for (int cb = wv; cb < nblk; cb += nw) {
    const int col = cb * 4 * CW + cg * CW;
    if (cb != wv) st.load(S, dk, dv, rg, col, live);
    float v[CW], o[CW];
#pragma unroll
    for (int e = 0; e < CW; ++e) v[e] = col + e < dv ? hd.v[col + e] : 0.f;
    st.template token<KIND != 3>(w, z, p, k, q, v, hd.qp, hd.qk, o);
    st.store(S, dk, dv, rg, col);
    if (KIND == 3 && rg == 0) {
      E* out = reinterpret_cast<E*>(a.o) + ((long long)b * a.H + h) * dv + col;
#pragma unroll
      for (int e = 0; e < CW; ++e)
        if (col + e < dv) delta::st<E>(out + e, fmaf(skip, v[e], o[e]));
    }
    if (KIND != 3 && rg == 0)
#pragma unroll
      for (int e = 0; e < CW; ++e)
        if (col + e < dv) {  // (this wave alone reads and writes these columns of v)
          hd.v[col + e] = o[e];
          ss = fmaf(o[e], o[e], ss);
        }
  }
  if constexpr (KIND == 3) return;
  float none = 0.f;
  block_sum2(ss, none, hd.red);
  const float n = 1.f / sqrtf(ss / (float)dv + a.eps);
  E* out = reinterpret_cast<E*>(a.out) + (long long)b * a.ldo + h * dv;
  const E* gain = reinterpret_cast<const E*>(a.gain) + (KIND == 0 ? h * dv : 0);
  for (int c = tid; c < dv; c += blockDim.x) delta::st<E>(out + c, hd.v[c] * n * delta::ld<E>(gain + c) * hd.gate[c]);
}

template <typename E, int KIND>
__global__ void __launch_bounds__(256) delta_prep_kernel(DeltaArgs a) {
  extern __shared__ float smem[];
  const int t = a.rows ? a.rows[blockIdx.x] : (int)blockIdx.x, h = blockIdx.y, tid = threadIdx.x, dk = a.dk, dv = a.dv;
  Head hd(smem, dk, dv, a.rank_w, a.rank_g);
  prep_head<E, KIND>(a, t, h, hd);
  float* pk = a.pk + ((long long)blockIdx.x * a.H + h) * pk_stride(dk, dv);
  for (int c = tid; c < 5 * dk + dv; c += 256) pk[c] = smem[c];  // w z p k q v lie in this order
  if (tid == 0) {
    pk[5 * dk + dv] = hd.qp;
    pk[5 * dk + dv + 1] = hd.qk;
  }
}

template <typename E, int R, int CW>
__global__ void __launch_bounds__(256) delta_scan_kernel(DeltaArgs a) {
  const int* en = a.ent + blockIdx.x * 5;
  const int row0 = en[0], n = en[1], pos0 = en[2], slot = en[3], pk0 = en[4], h = blockIdx.y;
  const int wv = threadIdx.x >> 6, lane = threadIdx.x & 63, rg = lane & 15, cg = lane >> 4;
  const int dk = a.dk, dv = a.dv, col = (blockIdx.z * 4 + wv) * 4 * CW + cg * CW;
  if ((int)(blockIdx.z * 4 + wv) * 4 * CW >= dv) return;
  float* S = a.state + ((long long)slot * a.H + h) * dk * dv;
  const int ps = pk_stride(dk, dv);
  const long long step = (long long)a.H * ps;
  const float* pk = a.pk + ((long long)pk0 * a.H + h) * ps;
  E* o = reinterpret_cast<E*>(a.o) + (long long)row0 * a.H * dv + h * dv + col;
  const float skip = a.skip ? delta::ld<E>(reinterpret_cast<const E*>(a.skip) + h) : 0.f;
  Cols<R, CW> st;
  st.load(S, dk, dv, rg, col, pos0 > 0);
  float w[R], z[R], p[R], k[R], q[R], v[CW], qp, qk;
  auto fetch = [&](const float* s) {
    rows_of<R>(s, dk, rg, w);
    rows_of<R>(s + dk, dk, rg, z);
    rows_of<R>(s + 2 * dk, dk, rg, p);
    rows_of<R>(s + 3 * dk, dk, rg, k);
    rows_of<R>(s + 4 * dk, dk, rg, q);
#pragma unroll
    for (int e = 0; e < CW; ++e) v[e] = col + e < dv ? s[5 * dk + col + e] : 0.f;
    qp = s[5 * dk + dv];
    qk = s[5 * dk + dv + 1];
  };
  fetch(pk);
  for (int t = 0; t < n; ++t) {
    float wn[R], zn[R], pn[R], kn[R], qn[R], vn[CW];
    const float qpn = qp, qkn = qk;
#pragma unroll
    for (int i = 0; i < R; ++i) wn[i] = w[i], zn[i] = z[i], pn[i] = p[i], kn[i] = k[i], qn[i] = q[i];
#pragma unroll
    for (int e = 0; e < CW; ++e) vn[e] = v[e];
    pk += step;
    if (t + 1 < n) fetch(pk);  // the next token's loads fly under this one's products
    float y[CW];
    st.token(wn, zn, pn, kn, qn, vn, qpn, qkn, y);
    if (rg == 0)
#pragma unroll
      for (int e = 0; e < CW; ++e)
        if (col + e < dv) delta::st<E>(o + e, fmaf(skip, vn[e], y[e]));
    o += (long long)a.H * dv;
  }
  st.store(S, dk, dv, rg, col);
}

// NL lanes per (token, head), V channels each and turn (V = 4: rows aligned to 4 elements)
template <typename E, int KIND, int NL, int V>
__global__ void __launch_bounds__(256) delta_gate_kernel(DeltaArgs a, int T) {
  struct alignas(sizeof(E) * V) PackE { E v[V]; };
  const long long i = ((long long)blockIdx.x * 256 + threadIdx.x) / NL;
  if (i >= (long long)T * a.H) return;
  const int t = (int)(i / a.H), h = (int)(i - (long long)t * a.H), lane = threadIdx.x % NL, dv = a.dv;
  const E* o = reinterpret_cast<const E*>(a.o) + ((long long)t * a.H + h) * dv;
  const E* gain = reinterpret_cast<const E*>(a.gain) + (KIND == 0 ? h * dv : 0);
  const E* gt = KIND != 1 ? reinterpret_cast<const E*>(a.x) + (long long)t * a.ld + a.o_g + h * dv
                          : reinterpret_cast<const E*>(a.dg) + (long long)t * a.ldg + h * dv;
  E* out = reinterpret_cast<E*>(a.out) + (long long)t * a.ldo + h * dv;
  const int c0 = lane * V;
  PackE y, g, gn;  // the first turn's operands (the only one for usual head sizes)
#pragma unroll
  for (int e = 0; e < V; ++e) delta::st<E>(y.v + e, 0.f);
  if (c0 < dv) {
    y = *reinterpret_cast<const PackE*>(o + c0);
    g = *reinterpret_cast<const PackE*>(gt + c0);
    gn = *reinterpret_cast<const PackE*>(gain + c0);
  }
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < V; ++e) ss = fmaf(delta::ld<E>(y.v + e), delta::ld<E>(y.v + e), ss);
  for (int c = c0 + NL * V; c < dv; c += NL * V) {
    const PackE x = *reinterpret_cast<const PackE*>(o + c);
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(delta::ld<E>(x.v + e), delta::ld<E>(x.v + e), ss);
  }
  ss = lanes_reduce<NL>(ss, [](float p, float q) { return p + q; });
  const float n = 1.f / sqrtf(ss / (float)dv + a.eps);
  for (int c = c0; c < dv; c += NL * V) {
    if (c != c0) {
      y = *reinterpret_cast<const PackE*>(o + c);
      g = *reinterpret_cast<const PackE*>(gt + c);
      gn = *reinterpret_cast<const PackE*>(gain + c);
    }
    PackE r;
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const float z = delta::ld<E>(g.v + e);
      const float sg = (sizeof(E) == 4 ? sigmoid(z) : __builtin_amdgcn_rcpf(1.f + __expf(-z))) * (KIND == 2 ? z : 1.f);
      delta::st<E>(r.v + e, delta::ld<E>(y.v + e) * n * delta::ld<E>(gn.v + e) * sg);
    }
    *reinterpret_cast<PackE*>(out + c) = r;
  }
  if constexpr (KIND >= 1)
    if (a.e1[t] - t <= a.taps) ring_store<E>(a, t, h, lane, NL);
}

// Rows of short convolutions: V channels and ROWS consecutive rows a thread. A row's earlier inputs are the rows
// before it, back to its entry's first, then the slot's ring.
constexpr int CONV_ROWS = 8;
template <typename E, int V>
__global__ void __launch_bounds__(256) delta_conv_kernel(DeltaArgs a, E* out, int T) {
  struct alignas(sizeof(E) * V) PackE { E v[V]; };
  const int nqk = a.G * a.dk, C = 2 * nqk + a.H * a.dv, per = C / V;
  const long long i = (long long)blockIdx.x * 256 + threadIdx.x;
  const int t0 = (int)(i / per) * CONV_ROWS, ch = (int)(i % per) * V;
  if (t0 >= T) return;
  const int col = ch < nqk ? a.o_q + ch : ch < 2 * nqk ? a.o_k + ch - nqk : a.o_v + ch - 2 * nqk;
  const E* x = reinterpret_cast<const E*>(a.x) + col;
  const E* w = reinterpret_cast<const E*>(a.conv) + (long long)ch * a.taps;
  const int t1 = min(t0 + CONV_ROWS, T), first = a.e0[t0];
  auto conv = [&](const PackE& u, float (&v)[V]) {
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] = delta::ld<E>(u.v + e);
  };
  auto load = [&](int t) { return *reinterpret_cast<const PackE*>(x + (long long)t * a.ld); };
  auto before = [&](int t, int n, float (&v)[V]) {  // the input n tokens before row t
    if (t - n >= a.e0[t]) return conv(load(t - n), v);
    const int ps = a.pos[t] - n;
    const float* r = a.ring + ((long long)a.slot[t] * a.taps + (ps >= 0 ? ps % a.taps : 0)) * C + ch;
#pragma unroll
    for (int e = 0; e < V; ++e) v[e] = ps >= 0 ? r[e] : 0.f;
  };
  auto put = [&](int t, const float (&y)[V]) {
    PackE u;
#pragma unroll
    for (int e = 0; e < V; ++e) {
      if constexpr (sizeof(E) == 4) delta::st<E>(u.v + e, silu(y[e]));
      else delta::st<E>(u.v + e, y[e] * __builtin_amdgcn_rcpf(1.f + __expf(-y[e])));
    }
    *reinterpret_cast<PackE*>(out + (long long)t * C + ch) = u;
  };
  float bias[V];
#pragma unroll
  for (int e = 0; e < V; ++e) bias[e] = a.convb ? delta::ld<E>(reinterpret_cast<const E*>(a.convb) + ch + e) : 0.f;
  if (a.taps > 4) {
    for (int t = t0; t < t1; ++t) {
      float y[V], v[V];
#pragma unroll
      for (int e = 0; e < V; ++e) y[e] = bias[e];
      for (int n = 0; n < a.taps; ++n) {
        before(t, n, v);
#pragma unroll
        for (int e = 0; e < V; ++e) y[e] = fmaf(delta::ld<E>(w + (long long)e * a.taps + a.taps - 1 - n), v[e], y[e]);
      }
      put(t, y);
    }
    return;
  }
  float tap[4][V], h[4][V];  // h[n]: the input n tokens back
  auto taps = [&]() {
    if (V > 1 && a.taps == 4 && (uintptr_t)a.conv % (sizeof(E) * V) == 0) {  // channel by channel, V values a load
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const PackE u = *reinterpret_cast<const PackE*>(w + j * V);
#pragma unroll
        for (int e = 0; e < V; ++e) tap[3 - (j * V + e) % 4][(j * V + e) / 4] = delta::ld<E>(u.v + e);
      }
      return;
    }
#pragma unroll
    for (int n = 0; n < 4; ++n)
#pragma unroll
      for (int e = 0; e < V; ++e) tap[n][e] = n < a.taps ? delta::ld<E>(w + (long long)e * a.taps + a.taps - 1 - n) : 0.f;
  };
  auto row = [&](int t) {
    float y[V];
#pragma unroll
    for (int e = 0; e < V; ++e)
      y[e] = fmaf(tap[0][e], h[0][e], fmaf(tap[1][e], h[1][e], fmaf(tap[2][e], h[2][e], fmaf(tap[3][e], h[3][e], bias[e]))));
    put(t, y);
#pragma unroll
    for (int n = 3; n > 0; --n)
#pragma unroll
      for (int e = 0; e < V; ++e) h[n][e] = h[n - 1][e];
  };
  if (t0 - 3 >= first && t0 + CONV_ROWS <= T && a.e0[t1 - 1] == first) {  // all inputs are rows of the entry
    PackE u[CONV_ROWS + 3];
#pragma unroll
    for (int n = 0; n < CONV_ROWS + 3; ++n) u[n] = load(t0 - 3 + n);
    taps();
#pragma unroll
    for (int n = 1; n < 4; ++n) conv(u[3 - n], h[n]);
#pragma unroll
    for (int n = 0; n < CONV_ROWS; ++n) {
      conv(u[n + 3], h[0]);
      row(t0 + n);
    }
    return;
  }
  taps();
#pragma unroll
  for (int n = 0; n < 4; ++n)
#pragma unroll
    for (int e = 0; e < V; ++e) h[n][e] = 0.f;
  for (int t = t0; t < t1; ++t) {
    if (t == t0 || a.e0[t] == t) {
#pragma unroll
      for (int n = 1; n < 4; ++n)
        if (n < a.taps) before(t, n, h[n]);
    }
    conv(load(t), h[0]);
    row(t);
  }
}

// KIND 3: out = N(o * silu(z)) * gain of a row, N over norm_groups equal parts. A part belongs to the workgroup (ALL)
// or to a wave, NCH packs of V channels a thread (0: any size, the gated row read twice).
template <typename E, int V, int NW, bool ALL, int NCH>
__global__ void __launch_bounds__(64 * NW) delta_parts_kernel(DeltaArgs a) {
  struct alignas(sizeof(E) * V) PackE { E v[V]; };
  __shared__ float red[NW];
  const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, n = a.H * a.dv, per = n / a.norm_groups;
  const E* o = reinterpret_cast<const E*>(a.o) + (long long)t * n;
  const E* z = reinterpret_cast<const E*>(a.x) + (long long)t * a.ld + a.o_g;
  const E* gain = reinterpret_cast<const E*>(a.gain);
  E* out = reinterpret_cast<E*>(a.out) + (long long)t * a.ldo;
  const int step = (ALL ? 64 * NW : 64) * V, c0 = (ALL ? tid : lane) * V;
  const int g = ALL ? blockIdx.y : blockIdx.y * NW + wv;
  if (g < a.norm_groups) {  // (whole waves; ALL: always)
    o += g * per;
    z += g * per;
    gain += g * per;
    out += g * per;
    auto gated = [&](const PackE& y, const PackE& q, float (&v)[V]) {
#pragma unroll
      for (int e = 0; e < V; ++e) {
        const float x = delta::ld<E>(q.v + e);
        v[e] = delta::ld<E>(y.v + e) * (sizeof(E) == 4 ? silu(x) : x * __builtin_amdgcn_rcpf(1.f + __expf(-x)));
      }
    };
    auto pack = [&](const E* p, int c) { return *reinterpret_cast<const PackE*>(p + c); };
    constexpr int M = NCH ? NCH : 1;
    PackE y[M], q[M], w[M];
    float ss = 0.f, v[V], u[M][V];
    if constexpr (NCH > 0) {
#pragma unroll
      for (int j = 0; j < NCH; ++j) {
        const int c = min(c0 + j * step, per - V);
        y[j] = pack(o, c);
        q[j] = pack(z, c);
        w[j] = pack(gain, c);
      }
#pragma unroll
      for (int j = 0; j < NCH; ++j) {
        gated(y[j], q[j], u[j]);
        if (c0 + j * step < per)
#pragma unroll
          for (int e = 0; e < V; ++e) ss = fmaf(u[j][e], u[j][e], ss);
      }
    } else {
      for (int c = c0; c < per; c += step) {
        gated(pack(o, c), pack(z, c), v);
#pragma unroll
        for (int e = 0; e < V; ++e) ss = fmaf(v[e], v[e], ss);
      }
    }
    ss = wave_sum(ss);
    if constexpr (ALL) {
      if (lane == 0) red[wv] = ss;
      __syncthreads();
      ss = 0.f;
#pragma unroll
      for (int i = 0; i < NW; ++i) ss += red[i];
    }
    const float r = 1.f / sqrtf(ss / (float)per + a.eps);
    auto put = [&](int c, const float (&x)[V], const PackE& gn) {
      PackE s;
#pragma unroll
      for (int e = 0; e < V; ++e) delta::st<E>(s.v + e, x[e] * r * delta::ld<E>(gn.v + e));
      *reinterpret_cast<PackE*>(out + c) = s;
    };
    if constexpr (NCH > 0) {
#pragma unroll
      for (int j = 0; j < NCH; ++j)
        if (c0 + j * step < per) put(c0 + j * step, u[j], w[j]);
    } else {
      for (int c = c0; c < per; c += step) {
        gated(pack(o, c), pack(z, c), v);
        put(c, v, pack(gain, c));
      }
    }
  }
  if (a.e1 && a.e1[t] - t <= a.taps) {  // all channels of an entry's last inputs, several loads in flight
    const int nqk = a.G * a.dk, C = 2 * nqk + n, NT = 64 * NW * gridDim.y;
    float* r = a.ring + ((long long)a.slot[t] * a.taps + a.pos[t] % a.taps) * C;
    const E* x = reinterpret_cast<const E*>(a.x) + (long long)t * a.ld;
    for (int c0 = blockIdx.y * 64 * NW + tid; c0 < C; c0 += 8 * NT) {
      float v[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const int c = min(c0 + i * NT, C - 1);
        v[i] = delta::ld<E>(x + (c < nqk ? a.o_q + c : c < 2 * nqk ? a.o_k + c - nqk : a.o_v + c - 2 * nqk));
      }
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (c0 + i * NT < C) r[c0 + i * NT] = v[i];
    }
  }
}

bool wide(const DeltaArgs& a) { return a.dv % 4 == 0 && (uintptr_t)a.state % 16 == 0; }

template <typename E, int KIND, int R, int CW>
int step_go(const DeltaArgs& a, int B, hipStream_t s) {
  int nw = (a.dv + 4 * CW - 1) / (4 * CW);
  const int most = R > 8 ? 8 : 16;  // (the kernel's launch bound)
  nw = nw < 4 ? 4 : nw > most ? most : nw;
  const size_t lds = (size_t)prep_floats(a.dk, a.dv, a.rank_w, a.rank_g) * 4;
  if (lds > 64 * 1024) return 10;
  hipLaunchKernelGGL((delta_step_kernel<E, KIND, R, CW>), dim3(B, a.H), dim3(64 * nw), lds, s, a);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
template <typename E, int KIND>
int step_r(const DeltaArgs& a, int B, hipStream_t s) {
#define F(R) (wide(a) ? step_go<E, KIND, R, 4>(a, B, s) : step_go<E, KIND, R, 1>(a, B, s))
  KCA_STATE_ROWS(a.dk, F)
#undef F
}

template <typename E, int R, int CW>
int scan_go(const DeltaArgs& a, int nent, hipStream_t s) {
  const int nblk = (a.dv + 4 * CW - 1) / (4 * CW);
  hipLaunchKernelGGL((delta_scan_kernel<E, R, CW>), dim3(nent, a.H, (nblk + 3) / 4), dim3(256), 0, s, a);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
template <typename E>
int scan_r(const DeltaArgs& a, int nent, hipStream_t s) {
#define F(R) (wide(a) ? scan_go<E, R, 4>(a, nent, s) : scan_go<E, R, 1>(a, nent, s))
  KCA_STATE_ROWS(a.dk, F)
#undef F
}

template <typename E, int KIND>
int prep_go(const DeltaArgs& a, int T, hipStream_t s) {
  const size_t lds = (size_t)prep_floats(a.dk, a.dv, a.rank_w, a.rank_g) * 4;
  if (lds > 64 * 1024) return 10;
  hipLaunchKernelGGL((delta_prep_kernel<E, KIND>), dim3(T, a.H), dim3(256), lds, s, a);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
template <typename E, int KIND>
int gate_go(const DeltaArgs& a, int T, hipStream_t s) {
  const int al = sizeof(E) * 4;
  const bool v4 = a.dv % 4 == 0 && a.ldo % 4 == 0 && (KIND != 1 ? a.ld % 4 == 0 && a.o_g % 4 == 0 : a.ldg % 4 == 0) &&
                  (uintptr_t)a.out % al == 0 && (uintptr_t)(KIND != 1 ? a.x : a.dg) % al == 0 && (uintptr_t)a.gain % al == 0 &&
                  (uintptr_t)a.o % 16 == 0;
  const long long n = (long long)T * a.H;
#define GO(NL, V) hipLaunchKernelGGL((delta_gate_kernel<E, KIND, NL, V>), dim3((unsigned)((n * NL + 255) / 256)), dim3(256), 0, s, a, T)
  if (!v4) GO(64, 1);
  else if (a.dv <= 64) GO(16, 4);
  else if (a.dv <= 128) GO(32, 4);
  else GO(64, 4);
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

template <typename E>
int conv_go(const DeltaArgs& a, void* out, int T, hipStream_t s) {
  constexpr int W = sizeof(E) == 2 ? 8 : 4;
  const int nqk = a.G * a.dk, C = 2 * nqk + a.H * a.dv;
  const bool vec = nqk % W == 0 && C % W == 0 && a.ld % W == 0 && a.o_q % W == 0 && a.o_k % W == 0 && a.o_v % W == 0 &&
                   (uintptr_t)a.x % 16 == 0 && (uintptr_t)out % 16 == 0;
  const long long n = (long long)((T + CONV_ROWS - 1) / CONV_ROWS) * (C / (vec ? W : 1));
  const dim3 g((unsigned)((n + 255) / 256));
  if (vec) hipLaunchKernelGGL((delta_conv_kernel<E, W>), g, dim3(256), 0, s, a, (E*)out, T);
  else hipLaunchKernelGGL((delta_conv_kernel<E, 1>), g, dim3(256), 0, s, a, (E*)out, T);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

template <typename E, int V>
int parts_v(const DeltaArgs& a, int T, hipStream_t s) {
  const int n = a.H * a.dv, per = n / a.norm_groups;
  const int packs = (per + V - 1) / V;
#define GO(NW, ALL, NCH)                                                                                              \
  hipLaunchKernelGGL((delta_parts_kernel<E, V, NW, ALL, NCH>), dim3(T, ALL ? a.norm_groups : (a.norm_groups + NW - 1) / NW), \
                     dim3(64 * NW), 0, s, a)
  if (a.norm_groups >= 4) {
    if (packs <= 64) GO(4, false, 1);
    else if (packs <= 128) GO(4, false, 2);
    else if (packs <= 256) GO(4, false, 4);
    else GO(4, false, 0);
  } else {
    if (packs <= 256) GO(4, true, 1);
    else if (T <= 64 && packs <= 1024) GO(16, true, 1);
    else if (packs <= 512) GO(4, true, 2);
    else if (packs <= 1024) GO(4, true, 4);
    else GO(4, true, 0);
  }
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
template <typename E>
int parts_go(const DeltaArgs& a, int T, hipStream_t s) {
  constexpr int W = sizeof(E) == 2 ? 8 : 4;
  const bool vec = (a.H * a.dv / a.norm_groups) % W == 0 && a.ld % W == 0 && a.ldo % W == 0 && a.o_g % W == 0 &&
                   (uintptr_t)a.x % 16 == 0 && (uintptr_t)a.o % 16 == 0 && (uintptr_t)a.out % 16 == 0 && (uintptr_t)a.gain % 16 == 0;
  return vec ? parts_v<E, W>(a, T, s) : parts_v<E, 1>(a, T, s);
}

}  // namespace

// Mirrored by ops/delta_rule.py
KCA_API int kca_delta_abi() { return (int)sizeof(DeltaArgs); }

#define DELTA_KINDS(FN, N, E)                              \
  switch (kind) {                                          \
    case 0: return FN<E, 0>(a, N, s);                      \
    case 1: return FN<E, 1>(a, N, s);                      \
    case 2: return FN<E, 2>(a, N, s);                      \
    default: return FN<E, 3>(a, N, s);                     \
  }
#define DELTA_DISPATCH(FN, N)                              \
  if (dtype == 0) DELTA_KINDS(FN, N, float)                \
  if (dtype == 1) DELTA_KINDS(FN, N, bf16_t)               \
  return 3;

// one token per row
KCA_API int kca_delta_step(const DeltaArgs* in, int dtype, int kind, int B, hipStream_t s) {
  const DeltaArgs& a = *in;
  if (!delta_args_ok(a, kind) || B < 1 || a.H > 65535 || a.e0 || a.cx || (kind == 3 && !a.o)) return 1;
  DELTA_DISPATCH(step_r, B)
}

// a.pk of T token rows (a.rows)
KCA_API int kca_delta_prep(const DeltaArgs* in, int dtype, int kind, int T, hipStream_t s) {
  const DeltaArgs& a = *in;
  if (!delta_args_ok(a, kind) || T < 1 || a.H > 65535 || !a.pk || !a.e0 || !a.e1) return 1;
  DELTA_DISPATCH(prep_go, T)
}

// a.o of nent entries from a.pk; the slots' states advance
KCA_API int kca_delta_scan(const DeltaArgs* in, int dtype, int nent, hipStream_t s) {
  const DeltaArgs& a = *in;
  if (nent < 1 || !a.pk || !a.o || !a.ent || !a.state || a.H < 1 || a.H > 65535 || a.dk < 1 || a.dk > 256 || a.dv < 1) return 1;
  if (dtype == 0) return scan_r<float>(a, nent, s);
  if (dtype == 1) return scan_r<bf16_t>(a, nent, s);
  return 3;
}

// a.out of every (token, head) from a.o
KCA_API int kca_delta_gate(const DeltaArgs* in, int dtype, int kind, int T, hipStream_t s) {
  const DeltaArgs& a = *in;
  if (!delta_args_ok(a, kind) || T < 1 || !a.o || !a.e0 || !a.e1 || kind > 2 || (kind == 1 && !a.dg)) return 1;
  if (dtype == 0) return kind == 0 ? gate_go<float, 0>(a, T, s) : kind == 1 ? gate_go<float, 1>(a, T, s) : gate_go<float, 2>(a, T, s);
  if (dtype == 1) return kind == 0 ? gate_go<bf16_t, 0>(a, T, s) : kind == 1 ? gate_go<bf16_t, 1>(a, T, s) : gate_go<bf16_t, 2>(a, T, s);
  return 3;
}

// kind 2, 3: convolution and silu of every row -> out [T][2 G dk + H dv]
KCA_API int kca_delta_conv(const DeltaArgs* in, int dtype, int kind, int T, void* out, hipStream_t s) {
  const DeltaArgs& a = *in;
  if (!delta_args_ok(a, kind) || kind < 2 || T < 1 || !a.e0 || !out) return 1;
  if (dtype == 0) return conv_go<float>(a, out, T, s);
  if (dtype == 1) return conv_go<bf16_t>(a, out, T, s);
  return 3;
}

// kind 3: a.out of every token from a.o; a.e1 set: the entries' last inputs go into the rings
KCA_API int kca_delta_parts(const DeltaArgs* in, int dtype, int T, hipStream_t s) {
  const DeltaArgs& a = *in;
  if (!delta_args_ok(a, 3) || T < 1 || !a.o) return 1;
  if (dtype == 0) return parts_go<float>(a, T, s);
  if (dtype == 1) return parts_go<bf16_t>(a, T, s);
  return 3;
}
