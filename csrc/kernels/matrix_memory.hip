// Matrix memory with exponential gates (mLSTM). Per head, from projections q (times qscale), k, v and log gates
//   i = cap tanh((x_i + b_i) / cap),   f = log sigmoid(cap tanh((x_f + b_f) / cap))
// a state S [dk][dv], a normaliser n [dk] and a running maximum m (0 before the first token) follow
//   m_t = max(f + m_(t-1), i),  w = e^(f + m_(t-1) - m_t),  p = e^(i - m_t)
//   S_t = w S_(t-1) + p k v^T,  n_t = w n_(t-1) + p k,      o_t = S_t^T q / (max(|n_t . q|, e^(-m_t)) + 1e-6)
// and the read-out is RMS-normed per head, times a gain, times sigmoid(gate), times mul. Gates, state and norms are fp32.
//
//   step kernel   one token per row, projections -> gated output in one launch
//   scan kernel   an entry's tokens in order, state in registers; a wave owns a few value columns of a head (any size
//                 and type)
//   map kernel    bf16, chunks of 64 tokens at once: with F the running sum of f, b_j = i_j - F_j and c_t the running
//                 maximum of b, all inside the chunk,
//                   A_tj = (q_t . k_j) e^(b_j - c_t) (j <= t), its row sums, K'_j = e^(b_j - c_end) k_j and its sum
//   run kernel    chunks of an entry in order, 16 NC value columns of a head per workgroup: with m_0 the first maximum and
//                 M_t = max(m_0, c_t), m_t = F_t + M_t,
//                   o_t   ~ e^(m_0 - M_t) S_0^T q_t + e^(c_t - M_t) sum_j A_tj v_j       (n . q alike, from the row sums)
//                   S_end = e^(m_0 - M_end) S_0 + e^(c_end - M_end) sum_j K'_j v_j^T
//   gate kernel   head norm, gain and gate of every (token, head)
// Every exponent is at most 0 (but -m_t, a floor of the divisor). A carried sequence's state lives in its slot and counts
// as zero at position 0. The workgroups of a head all read n and m, so scan and run leave the new ones beside the slots'
// (norm1, top1) and the gate kernel moves them.
#include "chunk_ops.h"
#include "matrix_memory.h"

namespace {

template <typename E, int R, int CW>
__global__ void __launch_bounds__(R > 8 ? 512 : 1024) memory_step_kernel(MemArgs a) {
  extern __shared__ float vals[];
  __shared__ float red[16];
  step_body<E, R, CW>(a, blockIdx.x, blockIdx.y, vals, red);
}

template <typename E, int R, int CW>
__global__ void __launch_bounds__(256) memory_scan_kernel(MemArgs a) {
  const int* en = a.ent + blockIdx.x * 5;
  const int row0 = en[0], cnt = en[1], pos0 = en[2], slot = en[3], h = blockIdx.y;
  const int wv = threadIdx.x >> 6, lane = threadIdx.x & 63, rg = lane & 15, cg = lane >> 4;
  const int dk = a.dk, dv = a.dv, blk = blockIdx.z * 4 + wv, col = blk * 4 * CW + cg * CW;
  if (blk * 4 * CW >= dv) return;
  const long long sh = (long long)slot * a.H + h;
  float* S = a.state + sh * dk * dv;
  const bool live = pos0 > 0;
  Cols<R, CW> st;
  st.load(S, dk, dv, rg, col, live);
  float n[R], m = live ? a.top[sh] : 0.f;
#pragma unroll
  for (int i = 0; i < R; ++i) n[i] = live && rg + 16 * i < dk ? a.norm[sh * dk + rg + 16 * i] : 0.f;
  const E* x = reinterpret_cast<const E*>(a.x) + (long long)row0 * a.ld;
  E* out = reinterpret_cast<E*>(a.o) + ((long long)row0 * a.H + h) * dv + col;
  float k[R], q[R], v[CW];
  Gates g;
  auto fetch = [&](const E* r) {
    rows_x<E, R>(r + a.o_k + h * dk, dk, rg, 1.f, k);
    rows_x<E, R>(r + a.o_q + h * dk, dk, rg, a.qscale, q);
#pragma unroll
    for (int e = 0; e < CW; ++e) v[e] = col + e < dv ? delta::ld<E>(r + a.o_v + h * dv + col + e) : 0.f;
    g = gates<E>(a, r, h);
  };
  fetch(x);
  for (int t = 0; t < cnt; ++t) {
    float kn[R], qn[R], vn[CW], o[CW], w, qk;
    const Gates gn = g;
#pragma unroll
    for (int i = 0; i < R; ++i) kn[i] = k[i], qn[i] = q[i];
#pragma unroll
    for (int e = 0; e < CW; ++e) vn[e] = v[e];
    x += a.ld;
    if (t + 1 < cnt) fetch(x);  // the next token's loads fly under this one's products
    const float inv = advance<R>(gn, m, n, kn, qn, w, qk);
    st.decayed(w, kn, qn, vn, qk, o);
    if (rg == 0)
#pragma unroll
      for (int e = 0; e < CW; ++e)
        if (col + e < dv) delta::st<E>(out + e, o[e] * inv);
    out += (long long)a.H * dv;
  }
  st.store(S, dk, dv, rg, col);
  if (blk == 0 && cg == 0) {
#pragma unroll
    for (int i = 0; i < R; ++i)
      if (rg + 16 * i < dk) a.norm1[sh * dk + rg + 16 * i] = n[i];
    if (rg == 0) a.top1[sh] = m;
  }
}

template <int DK>
__global__ void __launch_bounds__(512) memory_map_kernel(MemArgs a) {
  constexpr int LK = DK + 8, KS = DK / 32, NK = DK / 64;
  __shared__ __attribute__((aligned(16))) bf16_t iq[CT * LK], ik[CT * LK];
  __shared__ __attribute__((aligned(16))) float bs[CT], cs[CT], es[CT], rs[4][CT], ns[2][DK];
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l15 = lane & 15, g4 = lane >> 4, tok = tid >> 3, sub = tid & 7;
  const int ci = blockIdx.x, h = blockIdx.y;
  const long long row0 = a.ck[ci * 4];
  const int n = a.ck[ci * 4 + 1];
  const bf16_t* xb = reinterpret_cast<const bf16_t*>(a.x);
  const bf16_t* x = xb + (row0 + min(tok, n - 1)) * a.ld + h * a.dk;
#pragma unroll
  for (int i = 0; i < NK; ++i) {
    const int c = sub * 8 + 64 * i;
    u32x4 q = {0u, 0u, 0u, 0u}, k = {0u, 0u, 0u, 0u};
    if (tok < n && c < a.dk) {
      q = *reinterpret_cast<const u32x4*>(x + a.o_q + c);
      k = *reinterpret_cast<const u32x4*>(x + a.o_k + c);
    }
    *reinterpret_cast<u32x4*>(iq + tok * LK + c) = q;
    *reinterpret_cast<u32x4*>(ik + tok * LK + c) = k;
  }
  float* gd = a.gd + ((long long)ci * a.H + h) * (3 * CT + DK);
  if (w == 0) {  // a lane a token: gates, their running sums and maxima
    const Gates g = gates<bf16_t>(a, xb + (row0 + min(lane, n - 1)) * a.ld, h);
    float F = lane < n ? g.f : 0.f;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float u = __shfl_up(F, o, 64);
      if (lane >= o) F += u;
    }
    const float b = lane < n ? g.i - F : -INFINITY;
    float c = b;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float u = __shfl_up(c, o, 64);
      if (lane >= o) c = fmaxf(c, u);
    }
    bs[lane] = b;
    cs[lane] = c;
    es[lane] = __expf(b - __shfl(c, 63, 64));
    gd[lane] = c;
    gd[CT + lane] = F;
  }
  if (tid < 4 * CT) rs[tid / CT][tid % CT] = 0.f;
  __syncthreads();
  const long long cg = (long long)ci * a.H + h;
  // blocks (I, J <= I | 1) of K Q^T: a lane's four rows are four tokens j at its column t
  for (int i = w; i < 12; i += 8) {
    const int I = i < 2 ? 0 : i < 4 ? 1 : i < 8 ? 2 : 3, J = i < 4 ? i & 1 : i & 3;
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int o = l15 * LK + 32 * k + 8 * g4;
      s = mm32(*reinterpret_cast<const bf16x8*>(ik + 16 * J * LK + o), *reinterpret_cast<const bf16x8*>(iq + 16 * I * LK + o), s);
    }
    const int t = 16 * I + l15, j = 16 * J + 4 * g4;
    const float ct = cs[t];
    const float4 b = *reinterpret_cast<const float4*>(bs + j);
    s[0] = j <= t ? s[0] * __expf(b.x - ct) : 0.f;
    s[1] = j + 1 <= t ? s[1] * __expf(b.y - ct) : 0.f;
    s[2] = j + 2 <= t ? s[2] * __expf(b.z - ct) : 0.f;
    s[3] = j + 3 <= t ? s[3] * __expf(b.w - ct) : 0.f;
    float sum = s[0] + s[1] + s[2] + s[3];
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    if (g4 == 0) rs[J][t] = sum;
    *reinterpret_cast<s16x4*>(a.am + ((cg * 4 + I) * 2 + (J >> 1)) * 512 + lane * 8 + 4 * (J & 1)) = pk4(s);
  }
  for (int i = w; i < DK / 8; i += 8) {
    const int m = i >> 1, k = i & 1, j = 32 * k + 4 * g4;
    const float4 e0 = *reinterpret_cast<const float4*>(es + j), e1 = *reinterpret_cast<const float4*>(es + j + 16);
    const f32x4 u = up4(tok4<LK>(ik, 32 * k, 16 * m)) * f32x4{e0.x, e0.y, e0.z, e0.w};
    const f32x4 v = up4(tok4<LK>(ik, 32 * k + 16, 16 * m)) * f32x4{e1.x, e1.y, e1.z, e1.w};
    float sum = u[0] + u[1] + u[2] + u[3] + (v[0] + v[1] + v[2] + v[3]);
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    if (g4 == 0) ns[k][16 * m + l15] = sum;
    *reinterpret_cast<bf16x8*>(a.kt + ((cg * (DK / 16) + m) * 2 + k) * 512 + lane * 8) = two(pk4(u), pk4(v));
  }
  __syncthreads();
  if (tid < CT) gd[2 * CT + tid] = rs[0][tid] + rs[1][tid] + rs[2][tid] + rs[3][tid];
  else if (tid < CT + DK) gd[2 * CT + tid] = ns[0][tid - CT] + ns[1][tid - CT];
}

// A wave holds DK / 4 state rows (columns lane & 15 of each tile, rows 4 (lane >> 4) + r) and reads out 16 tokens;
// thread c < DK holds n[c].
template <int DK, int NC>
__global__ void __launch_bounds__(256) memory_run_kernel(MemArgs a) {
  constexpr int LS = DK + 8, LX = 16 * NC + 8, KS = DK / 32, MT = DK / 64, GD = 3 * CT + DK;
  __shared__ __attribute__((aligned(16))) bf16_t img[2][NC * 16 * LS], xs[2][CT * LX], nimg[2][DK];
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), l15 = lane & 15, g4 = lane >> 4;
  const int h = blockIdx.x % a.H, v0 = blockIdx.x / a.H * 16 * NC;
  const int* en = a.en + blockIdx.y * 6;
  const int row0 = en[0], cnt = en[1], pos0 = en[2], slot = en[3], ch0 = en[4], nc = en[5];
  const int r0 = w * (DK / 4) + 4 * g4, tok = tid >> 2, c4 = (tid & 3) * 4;
  const bf16_t* xb = reinterpret_cast<const bf16_t*>(a.x);
  const long long sh = (long long)slot * a.H + h;
  float* S = a.state + sh * a.dk * a.dv;
  f32x4 st[NC][MT];
#pragma unroll
  for (int q = 0; q < NC; ++q)
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = r0 + 16 * m + r, v = v0 + 16 * q + l15;
        st[q][m][r] = pos0 > 0 && c < a.dk && v < a.dv ? S[(long long)c * a.dv + v] : 0.f;
      }
  float n = pos0 > 0 && tid < a.dk ? a.norm[sh * a.dk + tid] : 0.f;
  float m0 = pos0 > 0 ? a.top[sh] : 0.f;
  struct Frag {
    bf16x8 q[KS], k[MT][2], a[2];
    uint2 x[NC];
    float4 c, F, rs;      // of the wave's tokens 4 g4 + r
    float ce, Fe, np;
  };
  auto load = [&](int i, Frag& f) {
    const long long cg = (long long)(ch0 + i) * a.H + h;
    const int left = cnt - i * CT;
    const bf16_t* qr = xb + (long long)(row0 + i * CT + min(16 * w + l15, left - 1)) * a.ld + a.o_q + h * a.dk;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      u32x4 u = {0u, 0u, 0u, 0u};
      if (32 * k + 8 * g4 < a.dk) u = *reinterpret_cast<const u32x4*>(qr + 32 * k + 8 * g4);
      f.q[k] = __builtin_bit_cast(bf16x8, u);
    }
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int k = 0; k < 2; ++k)
        f.k[m][k] = *reinterpret_cast<const bf16x8*>(a.kt + ((cg * (DK / 16) + w * MT + m) * 2 + k) * 512 + lane * 8);
#pragma unroll
    for (int k = 0; k < 2; ++k)  // (k = 1 of the first two row blocks: not read below)
      f.a[k] = *reinterpret_cast<const bf16x8*>(a.am + ((cg * 4 + w) * 2 + (w >= 2 ? k : 0)) * 512 + lane * 8);
    const bf16_t* xr = xb + (long long)(row0 + i * CT + min(tok, left - 1)) * a.ld + a.o_v + h * a.dv;
#pragma unroll
    for (int q = 0; q < NC; ++q) {
      const int v = v0 + 16 * q + c4;
      f.x[q] = make_uint2(0u, 0u);
      if (tok < left && v < a.dv) f.x[q] = *reinterpret_cast<const uint2*>(xr + v);
    }
    const float* gd = a.gd + cg * GD;
    const int t = 16 * w + 4 * g4;
    f.c = *reinterpret_cast<const float4*>(gd + t);
    f.F = *reinterpret_cast<const float4*>(gd + CT + t);
    f.rs = *reinterpret_cast<const float4*>(gd + 2 * CT + t);
    f.ce = gd[CT - 1];
    f.Fe = gd[2 * CT - 1];
    f.np = gd[3 * CT + min(tid, DK - 1)];
  };
  auto chunk = [&](int i, const Frag& f) {
    const int bf = i & 1;
    bf16_t* im = img[bf];
#pragma unroll
    for (int q = 0; q < NC; ++q)
#pragma unroll
      for (int m = 0; m < MT; ++m) *reinterpret_cast<s16x4*>(im + (16 * q + l15) * LS + r0 + 16 * m) = pk4(st[q][m]);
#pragma unroll
    for (int q = 0; q < NC; ++q) *reinterpret_cast<uint2*>(xs[bf] + tok * LX + 16 * q + c4) = f.x[q];
    if (tid < DK) nimg[bf][tid] = f2bf(n);
    __syncthreads();
    const float Me = fmaxf(m0, f.ce), all = __expf(m0 - Me), late = __expf(f.ce - Me);
    f32x4 nq = {0.f, 0.f, 0.f, 0.f}, o[NC], in[NC], add[NC][MT];
#pragma unroll
    for (int k = 0; k < KS; ++k) nq = mm32(f.q[k], *reinterpret_cast<const bf16x8*>(nimg[bf] + 32 * k + 8 * g4), nq);
#pragma unroll
    for (int q = 0; q < NC; ++q) {
      o[q] = in[q] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KS; ++k)
        o[q] = mm32(f.q[k], *reinterpret_cast<const bf16x8*>(im + (16 * q + l15) * LS + 32 * k + 8 * g4), o[q]);
#pragma unroll
      for (int m = 0; m < MT; ++m) add[q][m] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      bf16x8 xv[NC];
#pragma unroll
      for (int q = 0; q < NC; ++q) xv[q] = two(tok4<LX>(xs[bf], 32 * k, 16 * q), tok4<LX>(xs[bf], 32 * k + 16, 16 * q));
      if (k == 0 || w >= 2)
#pragma unroll
        for (int q = 0; q < NC; ++q) in[q] = mm32(f.a[k], xv[q], in[q]);
#pragma unroll
      for (int q = 0; q < NC; ++q)
#pragma unroll
        for (int m = 0; m < MT; ++m) add[q][m] = mm32(f.k[m][k], xv[q], add[q][m]);
    }
    const float c[4] = {f.c.x, f.c.y, f.c.z, f.c.w}, F[4] = {f.F.x, f.F.y, f.F.z, f.F.w}, rs[4] = {f.rs.x, f.rs.y, f.rs.z, f.rs.w};
    bf16_t* op = reinterpret_cast<bf16_t*>(a.o) + ((long long)(row0 + i * CT + 16 * w + 4 * g4) * a.H + h) * a.dv;
    const long long os = (long long)a.H * a.dv;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float M = fmaxf(m0, c[r]), old = __expf(m0 - M) * a.qscale, own = __expf(c[r] - M) * a.qscale;
      const float y = 1.f / (fmaxf(fabsf(old * nq[r] + own * rs[r]), __expf(-(F[r] + M))) + 1e-6f);
      if (i * CT + 16 * w + 4 * g4 + r < cnt)
#pragma unroll
        for (int q = 0; q < NC; ++q) {
          const int v = v0 + 16 * q + l15;
          if (v < a.dv) op[r * os + v] = f2bf((old * o[q][r] + own * in[q][r]) * y);
        }
    }
#pragma unroll
    for (int q = 0; q < NC; ++q)
#pragma unroll
      for (int m = 0; m < MT; ++m) st[q][m] = st[q][m] * all + add[q][m] * late;
    n = fmaf(n, all, f.np * late);
    m0 = f.Fe + Me;
  };
  // two chunks ahead of the products, unconditionally (past the end: the last chunk again)
  Frag f0, f1, f2;
  load(0, f0);
  load(min(1, nc - 1), f1);
  int i = 0;
  for (; i + 3 <= nc; i += 3) {
    load(min(i + 2, nc - 1), f2);
    chunk(i, f0);
    load(min(i + 3, nc - 1), f0);
    chunk(i + 1, f1);
    load(min(i + 4, nc - 1), f1);
    chunk(i + 2, f2);
  }
  if (i < nc) chunk(i, f0);
  if (i + 1 < nc) chunk(i + 1, f1);
#pragma unroll
  for (int q = 0; q < NC; ++q)
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = r0 + 16 * m + r, v = v0 + 16 * q + l15;
        if (c < a.dk && v < a.dv) S[(long long)c * a.dv + v] = st[q][m][r];
      }
  if (v0 == 0) {
    if (tid < a.dk) a.norm1[sh * a.dk + tid] = n;
    if (tid == 0) a.top1[sh] = m0;
  }
}

// NL lanes per (token, head), V channels each and turn (V = 4: rows aligned to 4 elements)
template <typename E, int NL, int V>
__global__ void __launch_bounds__(256) memory_gate_kernel(MemArgs a, int T) {
  struct alignas(sizeof(E) * V) Pack { E v[V]; };
  const long long i = ((long long)blockIdx.x * 256 + threadIdx.x) / NL;
  if (i >= (long long)T * a.H) return;
  const int t = (int)(i / a.H), h = (int)(i - (long long)t * a.H), lane = threadIdx.x % NL, dv = a.dv;
  const E* o = reinterpret_cast<const E*>(a.o) + ((long long)t * a.H + h) * dv;
  const E* gain = reinterpret_cast<const E*>(a.gain) + h * dv;
  const E* gt = reinterpret_cast<const E*>(a.x) + (long long)t * a.ld + a.o_g + h * dv;
  E* out = reinterpret_cast<E*>(a.out) + (long long)t * a.ldo + h * dv;
  auto at = [](const E* p, int c) { return *reinterpret_cast<const Pack*>(p + c); };
  const int c0 = lane * V;
  Pack y, g, gn;  // the first turn's operands (the only one for usual head sizes)
#pragma unroll
  for (int e = 0; e < V; ++e) delta::st<E>(y.v + e, 0.f);
  if (c0 < dv) {
    y = at(o, c0);
    g = at(gt, c0);
    gn = at(gain, c0);
  }
  float ss = 0.f;
#pragma unroll
  for (int e = 0; e < V; ++e) ss = fmaf(delta::ld<E>(y.v + e), delta::ld<E>(y.v + e), ss);
  for (int c = c0 + NL * V; c < dv; c += NL * V) {
    const Pack x = at(o, c);
#pragma unroll
    for (int e = 0; e < V; ++e) ss = fmaf(delta::ld<E>(x.v + e), delta::ld<E>(x.v + e), ss);
  }
  ss = lanes_reduce<NL>(ss, [](float p, float q) { return p + q; });
  const float n = a.mul / sqrtf(ss / (float)dv + a.eps);
  for (int c = c0; c < dv; c += NL * V) {
    if (c != c0) {
      y = at(o, c);
      g = at(gt, c);
      gn = at(gain, c);
    }
    Pack r;
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const float z = delta::ld<E>(g.v + e);
      const float sg = sizeof(E) == 4 ? sigmoid(z) : __builtin_amdgcn_rcpf(1.f + __expf(-z));
      delta::st<E>(r.v + e, delta::ld<E>(y.v + e) * n * delta::ld<E>(gn.v + e) * sg);
    }
    *reinterpret_cast<Pack*>(out + c) = r;
  }
  if (a.e1[t] == t + 1) {  // the entry's last token: its normaliser and maximum reach the slot
    const long long sh = (long long)a.slot[t] * a.H + h;
    for (int c = lane; c < a.dk; c += NL) a.norm[sh * a.dk + c] = a.norm1[sh * a.dk + c];
    if (lane == 0) a.top[sh] = a.top1[sh];
  }
}

template <typename E, int R, int CW>
int step_go(const MemArgs& a, int B, hipStream_t s) {
  int nw = (a.dv + 4 * CW - 1) / (4 * CW);
  const int most = R > 8 ? 8 : 16;  // (the kernel's launch bound)
  nw = nw < 4 ? 4 : nw > most ? most : nw;
  hipLaunchKernelGGL((memory_step_kernel<E, R, CW>), dim3(B, a.H), dim3(64 * nw), a.dv * 4, s, a);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
template <typename E>
int step_r(const MemArgs& a, int B, hipStream_t s) {
#define F(R) (wide(a) ? step_go<E, R, 4>(a, B, s) : step_go<E, R, 1>(a, B, s))
  KCA_STATE_ROWS(a.dk, F)
#undef F
}

template <typename E, int R, int CW>
int scan_go(const MemArgs& a, int nent, hipStream_t s) {
  const int nblk = (a.dv + 4 * CW - 1) / (4 * CW);
  hipLaunchKernelGGL((memory_scan_kernel<E, R, CW>), dim3(nent, a.H, (nblk + 3) / 4), dim3(256), 0, s, a);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
template <typename E>
int scan_r(const MemArgs& a, int nent, hipStream_t s) {
#define F(R) (wide(a) ? scan_go<E, R, 4>(a, nent, s) : scan_go<E, R, 1>(a, nent, s))
  KCA_STATE_ROWS(a.dk, F)
#undef F
}

template <int DK>
int run_go(const MemArgs& a, int nent, hipStream_t s) {
  const int tiles = (a.dv + 15) / 16, wg = a.H * nent;
  // more columns a workgroup re-read the shared operands less; fewer leave more workgroups
#define GO(NC) hipLaunchKernelGGL((memory_run_kernel<DK, NC>), dim3(a.H * ((tiles + NC - 1) / NC), nent), dim3(256), 0, s, a)
  if (tiles >= 4 && wg * (tiles / 4) >= 384) GO(4);
  else if (tiles >= 2 && wg * (tiles / 2) >= 256) GO(2);
  else GO(1);
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

template <typename E>
int gate_go(const MemArgs& a, int T, hipStream_t s) {
  const int al = sizeof(E) * 4;
  const bool v4 = a.dv % 4 == 0 && a.ldo % 4 == 0 && a.ld % 4 == 0 && a.o_g % 4 == 0 && (uintptr_t)a.out % al == 0 &&
                  (uintptr_t)a.x % al == 0 && (uintptr_t)a.gain % al == 0 && (uintptr_t)a.o % 16 == 0;
  const long long n = (long long)T * a.H;
#define GO(NL, V) hipLaunchKernelGGL((memory_gate_kernel<E, NL, V>), dim3((unsigned)((n * NL + 255) / 256)), dim3(256), 0, s, a, T)
  if (!v4) GO(64, 1);
  else if (a.dv <= 64) GO(16, 4);
  else if (a.dv <= 128) GO(32, 4);
  else GO(64, 4);
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

}  // namespace

// Mirrored by ops/matrix_memory.py
KCA_API int kca_memory_abi() { return (int)sizeof(MemArgs); }

// one token per row
KCA_API int kca_memory_step(const MemArgs* in, int dtype, int B, hipStream_t s) {
  const MemArgs& a = *in;
  if (!mem_ok(a) || B < 1 || !a.out) return 1;
  if (dtype == 0) return step_r<float>(a, B, s);
  if (dtype == 1) return step_r<bf16_t>(a, B, s);
  return 3;
}

// a.o of nent entries, token by token; their states advance (a.norm1, a.top1 beside the slots')
KCA_API int kca_memory_scan(const MemArgs* in, int dtype, int nent, hipStream_t s) {
  const MemArgs& a = *in;
  if (!mem_ok(a) || nent < 1 || !a.ent || !a.o || !a.norm1 || !a.top1) return 1;
  if (dtype == 0) return scan_r<float>(a, nent, s);
  if (dtype == 1) return scan_r<bf16_t>(a, nent, s);
  return 3;
}

// the same in chunks, bf16: a.am, a.kt, a.gd of nchunk chunks, then a.o of nent entries. 10: sizes for the scan
KCA_API int kca_memory_chunks(const MemArgs* in, int nchunk, int nent, hipStream_t s) {
  const MemArgs& a = *in;
  if (!mem_ok(a) || nchunk < 1 || nent < 1 || nent > 65535 || !a.ck || !a.en || !a.am || !a.kt || !a.gd || !a.o || !a.norm1 || !a.top1) return 1;
  if (a.dk % 8 || a.dv % 8 || a.dk > 128 || a.ld % 8 || a.o_q % 8 || a.o_k % 8 || a.o_v % 4 || (uintptr_t)a.x % 16) return 10;
  if (a.dk <= 64) hipLaunchKernelGGL(memory_map_kernel<64>, dim3(nchunk, a.H), dim3(512), 0, s, a);
  else hipLaunchKernelGGL(memory_map_kernel<128>, dim3(nchunk, a.H), dim3(512), 0, s, a);
  if (hipGetLastError() != hipSuccess) return 4;
  return a.dk <= 64 ? run_go<64>(a, nent, s) : run_go<128>(a, nent, s);
}

// a.out of every (token, head) from a.o; the entries' normalisers and maxima reach their slots
KCA_API int kca_memory_gate(const MemArgs* in, int dtype, int T, hipStream_t s) {
  const MemArgs& a = *in;
  if (!mem_ok(a) || T < 1 || !a.o || !a.out || !a.e1 || !a.norm1 || !a.top1) return 1;
  if (dtype == 0) return gate_go<float>(a, T, s);
  if (dtype == 1) return gate_go<bf16_t>(a, T, s);
  return 3;
}
