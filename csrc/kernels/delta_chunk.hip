// Delta-rule mixers (delta_rule.h) over bf16 prompt portions, in chunks of 64 tokens on the matrix cores.
//
// With G_t the running log decays of a chunk and S_0 its first state, the recurrence
//   S_t = diag(w_t) S_(t-1) + p_t s_t + k_t v_t^T,  s_t = z_t^T S_(t-1)
// unrolls to a unit lower triangular system in s,
//   (I - N) s = Z S_0 + A_zk V,   N[t][j] = z_t p_j e^(G_(t-1) - G_j), A_zk likewise with k (j < t),
// so that W = (I - N)^-1 Z and U = (I - N)^-1 A_zk V give everything a chunk does as maps of S_0:
//   S_end = E S_0 + M S_0 + B,    M = P^T W,          B = P^T U + K^T V      (P, K decayed to the chunk's end)
//   o     = Q' S_0 + O',          Q' = Q + A_qp W,    O' = A_qp U + A_qk V   (j <= t)
//
//   map kernel   all chunks and heads at once: vectors, decays, triangular solve, M, B, Q', O'
//   run kernel   chunks of an entry in order, 16 value columns of a head per workgroup: the fp32 state stays in
//                registers, its bf16 image is the operand of both products
// Decayed products go through blocks of 16 tokens: rows relative to their block's start, columns to their
// block's end, both at most 1; within a block both relative to its middle. There a log decay below -10 counts
// as -10 (what it passes on, 5e-5 of the state, is far under the operands' rounding), which bounds the exponents.
// KIND 1 has p = -k: N = -A_zk, A_qp = -A_qk, so half of the products fall together.
#include "attn_tile.h"
#include "delta_rule.h"

namespace {
using namespace delta;

constexpr int CT = 64;   // tokens of a chunk
constexpr float kFloor = -10.f;

struct ChunkArgs {
  DeltaArgs d;
  const int* ck;         // [nchunk][4]: first row, rows, first row of the entry, position of the chunk's first row
  const int* en;         // [nent][6]: first row, rows, position, slot, first chunk, chunks
  bf16_t* m;             // [nchunk][H][DK][DK]: M[c][c']
  bf16_t* b;             // [nchunk][H][DV][DK]: B^T
  bf16_t* q;             // [nchunk][H][64][DK]: Q'
  bf16_t* oo;            // [nchunk][H][DV][64]: O'^T
  float* e;              // [nchunk][H][DK]: decay of the whole chunk
};

__device__ __forceinline__ f32x4 mm16(s16x4 a, s16x4 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(a, b, c, 0, 0, 0); }
__device__ __forceinline__ f32x4 mm32(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
// 16 x 16 x 16 in fp32: a = four consecutive elements of row lane & 15 from column 4 (lane >> 4), b in the
// accumulators' layout (rows 4 (lane >> 4) + r of column lane & 15)
__device__ __forceinline__ f32x4 mm16f(float4 a, f32x4 b, f32x4 c) {
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b[0], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b[1], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b[2], c, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b[3], c, 0, 0, 0);
}
__device__ __forceinline__ s16x4 pk4(f32x4 v) {
  const uint2 u = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
  return __builtin_bit_cast(s16x4, u);
}
__device__ __forceinline__ s16x4 neg4(s16x4 v) {
  uint2 u = __builtin_bit_cast(uint2, v);
  u.x ^= 0x80008000u;
  u.y ^= 0x80008000u;
  return __builtin_bit_cast(s16x4, u);
}
// operand of four tokens (rows 4 (lane >> 4) of the block) at column lane & 15 of a row-major LDS image
template <int LD>
__device__ __forceinline__ s16x4 tok4(const bf16_t* img, int row, int col) {
  const int lane = threadIdx.x & 63, gi = lane & 15;
  const bf16_t* p = img + (row + 4 * (lane >> 4) + (gi >> 2)) * LD + col + 4 * (gi & 3);
  return __builtin_bit_cast(s16x4, lds_tr4(reinterpret_cast<const char*>(p), 0));
}
__device__ __forceinline__ s16x4 row4(const bf16_t* p) { return *reinterpret_cast<const s16x4*>(p); }
__device__ __forceinline__ f32x4 up4(s16x4 v) {
  const uint2 u = __builtin_bit_cast(uint2, v);
  return f32x4{__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
               __uint_as_float(u.y & 0xffff0000u)};
}

template <int CPL>
__device__ __forceinline__ void ldc(const bf16_t* p, bool ok, float (&v)[CPL]) {
  if constexpr (CPL == 2) {
    const uint32_t u = ok ? *reinterpret_cast<const uint32_t*>(p) : 0u;
    v[0] = __uint_as_float(u << 16);
    v[1] = __uint_as_float(u & 0xffff0000u);
  } else {
    v[0] = ok ? bf2f(*p) : 0.f;
  }
}
template <int CPL>
__device__ __forceinline__ void stc(bf16_t* p, const float (&v)[CPL]) {
  if constexpr (CPL == 2) *reinterpret_cast<uint32_t*>(p) = pack_bf16x2(v[0], v[1]);
  else *p = f2bf(v[0]);
}

template <int KIND, int DK, int DV>
struct Lds {
  static constexpr int LK = DK + 8, LV = DV + 8, LA = CT + 8, LN = CT + 4;
  bf16_t lq[CT * LK], lz[CT * LK], rk[CT * LK], rp[KIND == 0 ? CT * LK : 8];  // first the diagonal blocks' operands
  bf16_t v[CT * LV];
  bf16_t azk[CT * LA], aqk[CT * LA], aqp[KIND == 0 ? CT * LA : 8];
  float n[CT * LN];
  float ti[4][16][20];
  float tot[8][DK];    // log decay of every 8 tokens
  float et[4][DK];     // decay of every block of 16
  float pre[4][DK];    // decay from the chunk's start to the block's
};

template <int KIND, int DK, int DV>
__global__ void __launch_bounds__(512) delta_map_kernel(ChunkArgs p) {
  using L = Lds<KIND, DK, DV>;
  constexpr int CPL = DK / 64, CPV = DV / 64, KS = DK / 32;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  L& s = *reinterpret_cast<L*>(smem);
  const DeltaArgs& a = p.d;
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int lid = blockIdx.x, ci = lid / a.H, h = lid - ci * a.H;
  const int* ck = p.ck + ci * 4;
  const int row0 = ck[0], n = ck[1], first = ck[2], pos0 = ck[3];
  const int l15 = lane & 15, g4 = lane >> 4, blk = w >> 1, half = w & 1;

  // ------------------------------------------------------- vectors of 8 tokens, CPL channels a lane
  const int c0 = lane * CPL;
  const bool inc = c0 < a.dk;
  float q[8][CPL], u[8][CPL], pv[8][CPL], G[8][CPL], kn[8];
  {
    const bf16_t* x = reinterpret_cast<const bf16_t*>(a.x);
    const bf16_t* dw = reinterpret_cast<const bf16_t*>(a.dw);
    float w0[CPL], ab[CPL];
    ldc<CPL>(reinterpret_cast<const bf16_t*>(a.w0) + h * a.dk + c0, inc, w0);
    float A = 0.f;
    const int gq = h / (a.H / a.G), nqk = a.G * a.dk;
    if constexpr (KIND == 0) ldc<CPL>(reinterpret_cast<const bf16_t*>(a.ab) + h * a.dk + c0, inc, ab);
    else A = expf(bf2f(reinterpret_cast<const bf16_t*>(a.ab)[h]));
    const int t0 = 8 * w, slot = a.slot[row0], C = 2 * nqk + a.H * a.dv;
    // rows t0 - 3 .. t0 + 7 of a projection column block through the convolution and silu
    auto conv = [&](int col, int ch, bool ok, auto cpl, auto&& put) {
      constexpr int N = decltype(cpl)::value;
      float in[11][N], tp[4][N];
#pragma unroll
      for (int i = 0; i < 11; ++i) {
        const int t = t0 + i - 3, r = row0 + t;
        if (r >= first) {
          ldc<N>(x + (long long)r * a.ld + col, ok && t < n, in[i]);
        } else {  // before this batch's part of the sequence: what its slot keeps
          const int ps = pos0 + t;
#pragma unroll
          for (int e = 0; e < N; ++e)
            in[i][e] = ok && ps >= 0 && 3 - i < a.taps ? a.ring[((long long)slot * a.taps + ps % a.taps) * C + ch + e] : 0.f;
        }
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)  // tap i: the row i tokens back
#pragma unroll
        for (int e = 0; e < N; ++e)
          tp[i][e] = ok && i < a.taps ? bf2f(reinterpret_cast<const bf16_t*>(a.conv)[(long long)(ch + e) * a.taps + a.taps - 1 - i]) : 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        float y[N];
#pragma unroll
        for (int e = 0; e < N; ++e) {
          float v = tp[0][e] * in[i + 3][e];
#pragma unroll
          for (int j = 1; j < 4; ++j) v = fmaf(tp[j][e], in[i + 3 - j][e], v);
          y[e] = t0 + i < n ? v * __builtin_amdgcn_rcpf(1.f + __expf(-v)) : 0.f;
        }
        put(i, y);
      }
    };
    if constexpr (KIND == 1) {
      conv(a.o_q + gq * a.dk + c0, gq * a.dk + c0, inc, std::integral_constant<int, CPL>{},
           [&](int i, const float (&y)[CPL]) {
#pragma unroll
             for (int e = 0; e < CPL; ++e) q[i][e] = y[e];
           });
      conv(a.o_k + gq * a.dk + c0, nqk + gq * a.dk + c0, inc, std::integral_constant<int, CPL>{},
           [&](int i, const float (&y)[CPL]) {
#pragma unroll
             for (int e = 0; e < CPL; ++e) u[i][e] = y[e];
           });
      const int cv = lane * CPV;
      conv(a.o_v + h * a.dv + cv, 2 * nqk + h * a.dv + cv, cv < a.dv, std::integral_constant<int, CPV>{},
           [&](int i, const float (&y)[CPV]) { stc<CPV>(s.v + (t0 + i) * L::LV + cv, y); });
    } else {
      const int cv = lane * CPV;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const bool ok = t0 + i < n;
        const bf16_t* xr = x + (long long)(row0 + t0 + i) * a.ld;
        ldc<CPL>(xr + a.o_q + h * a.dk + c0, ok && inc, q[i]);
        ldc<CPL>(xr + a.o_k + h * a.dk + c0, ok && inc, u[i]);
        ldc<CPL>(xr + a.o_a + h * a.dk + c0, ok && inc, pv[i]);
        float v[CPV];
        ldc<CPV>(xr + a.o_v + h * a.dv + cv, ok && cv < a.dv, v);
        stc<CPV>(s.v + (t0 + i) * L::LV + cv, v);
      }
    }
    auto add = [](float x, float y) { return x + y; };
    float run[CPL];
#pragma unroll
    for (int e = 0; e < CPL; ++e) run[e] = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int t = t0 + i;
      const bool ok = t < n;
      float lw[CPL], sk = 0.f, sq = 0.f;
      ldc<CPL>(dw + (long long)(row0 + t) * a.ldw + h * a.dk + c0, ok && inc, lw);
#pragma unroll
      for (int e = 0; e < CPL; ++e) {
        sk = fmaf(u[i][e], u[i][e], sk);
        sq = fmaf(q[i][e], q[i][e], sq);
      }
      sk = lanes_reduce<64>(sk, add) + 1e-6f;
      const float ik = rsqrtf(sk);
      float iq = 1.f, beta = 0.f;
      if constexpr (KIND == 1) {
        iq = a.qscale * rsqrtf(lanes_reduce<64>(sq, add) + 1e-6f);
        beta = ok ? sigmoid(bf2f(x[(long long)(row0 + t) * a.ld + a.o_a + h])) : 0.f;
      }
      kn[i] = KIND == 0 ? sk * ik : beta;  // k = u * kn
#pragma unroll
      for (int e = 0; e < CPL; ++e) {
        float l = 0.f;
        if (ok && inc) {
          if constexpr (KIND == 0) l = -0.60653065971263342f * __builtin_amdgcn_rcpf(1.f + __expf(-(lw[e] + w0[e])));
          else l = fmaxf(-A * (fmaxf(lw[e] + w0[e], 0.f) + log1pf(__expf(-fabsf(lw[e] + w0[e])))), kFloor);
        }
        run[e] += l;
        G[i][e] = run[e];
        u[i][e] *= ik;
        q[i][e] *= iq;
        if constexpr (KIND == 0) pv[i][e] = -u[i][e] * __builtin_amdgcn_rcpf(1.f + __expf(-(pv[i][e] + ab[e])));
      }
    }
#pragma unroll
    for (int e = 0; e < CPL; ++e) s.tot[w][c0 + e] = run[e];
  }
  __syncthreads();
  // decays of the blocks, and of what lies before them
  if (tid < DK) {
    float acc = 0.f;
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const float t = s.tot[2 * b][tid] + s.tot[2 * b + 1][tid];
      s.et[b][tid] = __expf(t);
      s.pre[b][tid] = __expf(acc);
      acc += t;
    }
    p.e[((long long)ci * a.H + h) * DK + tid] = __expf(acc);
  }
  float mid[CPL], tot[CPL];
#pragma unroll
  for (int e = 0; e < CPL; ++e) {
    mid[e] = s.tot[w & ~1][c0 + e];
    tot[e] = mid[e] + s.tot[w | 1][c0 + e];
    if (half)
#pragma unroll
      for (int i = 0; i < 8; ++i) G[i][e] += mid[e];
  }
  // the four operand images relative to `ref` on both sides (diagonal blocks) or to the block's start and end
  auto image = [&](bool diag) {
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int o = (8 * w + i) * L::LK + c0;
      float yq[CPL], yz[CPL], yk[CPL], yp[CPL];
#pragma unroll
      for (int e = 0; e < CPL; ++e) {
        const float before = i ? G[i ? i - 1 : 0][e] : (half ? mid[e] : 0.f);
        const float lref = diag ? mid[e] : 0.f, rref = diag ? mid[e] : tot[e];
        const float fl = __expf(G[i][e] - lref), fr = __expf(rref - G[i][e]);
        yq[e] = q[i][e] * fl;
        yz[e] = u[i][e] * (KIND == 0 ? __expf(before - lref) : fl);
        yk[e] = u[i][e] * kn[i] * fr;
        if constexpr (KIND == 0) yp[e] = pv[i][e] * fr;
      }
      stc<CPL>(s.lq + o, yq);
      stc<CPL>(s.lz + o, yz);
      stc<CPL>(s.rk + o, yk);
      if constexpr (KIND == 0) stc<CPL>(s.rp + o, yp);
    }
  };
  image(true);
  __syncthreads();
  // ---------------------------------------------- decayed products: rows of block `blk`, z (half 0) or q (half 1)
  const bf16_t* left = half ? s.lq : s.lz;
  f32x4 ak[4], ap[4];
  auto block = [&](int J, bool scaled, int s0, int s1) {
    f32x4 x = {0.f, 0.f, 0.f, 0.f}, y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int o = k * 32 + 8 * g4;
      bf16x8 fa = *reinterpret_cast<const bf16x8*>(left + (16 * blk + l15) * L::LK + o);
      if (scaled) {
        const U16x8 r = __builtin_bit_cast(U16x8, fa);
        float v[8], f[8], f2[8];
        load8f(&s.et[s0][o], f);
        load8f(&s.et[s1][o], f2);
        U16x8 z;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          v[e] = bf2f(r.v[e]) * f[e] * (s1 != s0 ? f2[e] : 1.f);
          z.v[e] = f2bf(v[e]);
        }
        fa = __builtin_bit_cast(bf16x8, z);
      }
      x = mm32(fa, *reinterpret_cast<const bf16x8*>(s.rk + (16 * J + l15) * L::LK + o), x);
      if constexpr (KIND == 0) y = mm32(fa, *reinterpret_cast<const bf16x8*>(s.rp + (16 * J + l15) * L::LK + o), y);
    }
    ak[J] = x;
    ap[J] = y;
  };
#pragma unroll
  for (int J = 0; J < 4; ++J)
    if (J == blk) {
      block(J, false, 0, 0);
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (half ? l15 > 4 * g4 + r : l15 >= 4 * g4 + r) ak[J][r] = ap[J][r] = 0.f;
    }
  __syncthreads();
  image(false);
  __syncthreads();
#pragma unroll
  for (int J = 0; J < 3; ++J)
    if (J < blk) {
      if (J == blk - 1) block(J, false, 0, 0);
      else if (J == blk - 2) block(J, true, blk - 1, blk - 1);
      else block(J, true, 1, 2);
    }
#pragma unroll
  for (int J = 0; J < 4; ++J)
    if (J <= blk)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * blk + 4 * g4 + r, j = 16 * J + l15;
        (half ? s.aqk : s.azk)[t * L::LA + j] = f2bf(ak[J][r]);
        if (!half) s.n[t * L::LN + j] = KIND == 0 ? ap[J][r] : -ak[J][r];
        else if constexpr (KIND == 0) s.aqp[t * L::LA + j] = f2bf(ap[J][r]);
      }
  __syncthreads();
  // ------------------------------------------------- inverses of the diagonal blocks: a lane per column
  if (!half && lane < 16) {
    float x[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      float v = r == lane ? 1.f : 0.f;
#pragma unroll
      for (int k = 0; k < r; ++k) v = fmaf(s.n[(16 * blk + r) * L::LN + 16 * blk + k], x[k], v);
      x[r] = v;
      s.ti[blk][r][lane] = v;
    }
  }
  __syncthreads();
  // ----------------------------------------------- solve and maps, 16 columns of [W | U] a wave and turn
  const long long cb = (long long)ci * a.H + h;
  bf16_t* gm = p.m + cb * DK * DK;
  bf16_t* gb = p.b + cb * DV * DK;
  bf16_t* gq = p.q + cb * CT * DK;
  bf16_t* go = p.oo + cb * DV * CT;
#pragma unroll 1
  for (int ct = w; ct < (DK + DV) / 16; ct += 8) {
    const bool isw = ct < DK / 16;
    const int col = isw ? ct * 16 : ct * 16 - DK;
    f32x4 X[4];
    s16x4 vb[4];
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      f32x4 y = {0.f, 0.f, 0.f, 0.f};
      if (isw) {
        const float f = s.pre[I][col + l15];
#pragma unroll
        for (int r = 0; r < 4; ++r) y[r] = bf2f(s.lz[(16 * I + 4 * g4 + r) * L::LK + col + l15]) * f;
      } else {
        vb[I] = tok4<L::LV>(s.v, 16 * I, col);
#pragma unroll
        for (int J = 0; J <= I; ++J) y = mm16(row4(s.azk + (16 * I + l15) * L::LA + 16 * J + 4 * g4), vb[J], y);
      }
#pragma unroll
      for (int J = 0; J < I; ++J)
        y = mm16f(*reinterpret_cast<const float4*>(s.n + (16 * I + l15) * L::LN + 16 * J + 4 * g4), X[J], y);
      X[I] = mm16f(*reinterpret_cast<const float4*>(&s.ti[I][l15][4 * g4]), y, f32x4{0.f, 0.f, 0.f, 0.f});
    }
    s16x4 xb[4];
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      if (KIND == 1 && !isw) X[I] = up4(vb[I]) - X[I];  // V - U
      xb[I] = pk4(X[I]);
    }
    if (isw) {
      const int cw = col + 4 * g4;  // this lane's four columns c'
#pragma unroll
      for (int I = 0; I < 4; ++I) {
        const int t = 16 * I + l15;
        f32x4 y = up4(row4(s.lq + t * L::LK + cw));
        const float4 f = *reinterpret_cast<const float4*>(&s.pre[I][cw]);
        y[0] *= f.x; y[1] *= f.y; y[2] *= f.z; y[3] *= f.w;
#pragma unroll
        for (int J = 0; J <= I; ++J)
          y = mm16(KIND == 0 ? xb[J] : neg4(xb[J]), row4((KIND == 0 ? s.aqp : s.aqk) + t * L::LA + 16 * J + 4 * g4), y);
        *reinterpret_cast<s16x4*>(gq + t * DK + cw) = pk4(y);
      }
#pragma unroll 2
      for (int c = 0; c < DK; c += 16) {
        f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int J = 0; J < 4; ++J) {
          const float f = s.et[J][c + l15];
          if (J) y *= f;
          y = mm16(KIND == 0 ? xb[J] : neg4(xb[J]), tok4<L::LK>(KIND == 0 ? s.rp : s.rk, 16 * J, c), y);
        }
        *reinterpret_cast<s16x4*>(gm + (c + l15) * DK + cw) = pk4(y);
      }
    } else {
      const int v = col + l15;
#pragma unroll
      for (int I = 0; I < 4; ++I) {
        f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int J = 0; J <= I; ++J) {
          const int o = (16 * I + l15) * L::LA + 16 * J + 4 * g4;
          if constexpr (KIND == 0) {
            y = mm16(row4(s.aqp + o), xb[J], y);
            y = mm16(row4(s.aqk + o), vb[J], y);
          } else {
            y = mm16(row4(s.aqk + o), xb[J], y);
          }
        }
        *reinterpret_cast<s16x4*>(go + v * CT + 16 * I + 4 * g4) = pk4(y);
      }
#pragma unroll 2
      for (int c = 0; c < DK; c += 16) {
        f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int J = 0; J < 4; ++J) {
          const float4 f = *reinterpret_cast<const float4*>(&s.et[J][c + 4 * g4]);
          if (J) y[0] *= f.x, y[1] *= f.y, y[2] *= f.z, y[3] *= f.w;
          if constexpr (KIND == 0) y = mm16(tok4<L::LK>(s.rp, 16 * J, c), xb[J], y);
          y = mm16(tok4<L::LK>(s.rk, 16 * J, c), KIND == 0 ? vb[J] : xb[J], y);
        }
        *reinterpret_cast<s16x4*>(gb + v * DK + c + 4 * g4) = pk4(y);
      }
    }
  }
}

// A workgroup: 16 value columns of one (entry, head). A wave holds DK / 4 state rows (columns lane & 15, rows
// 4 (lane >> 4) + r of its tiles) and reads out 16 of a chunk's tokens.
template <int DK, int DV>
__global__ void __launch_bounds__(256) delta_run_kernel(ChunkArgs p) {
  constexpr int LS = DK + 8, KS = DK / 32, MT = DK / 64;
  __shared__ __attribute__((aligned(16))) bf16_t img[2][16 * LS];
  const DeltaArgs& a = p.d;
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, l15 = lane & 15, g4 = lane >> 4;
  const int h = blockIdx.x % a.H, vt = blockIdx.x / a.H;
  const int* en = p.en + blockIdx.y * 6;
  const int row0 = en[0], n = en[1], pos0 = en[2], slot = en[3], ch0 = en[4], nc = en[5];
  const int v = vt * 16 + l15, r0 = w * (DK / 4) + 4 * g4;
  float* S = a.state + ((long long)slot * a.H + h) * a.dk * a.dv;
  f32x4 st[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int c = r0 + 16 * m + r;
      st[m][r] = pos0 > 0 && c < a.dk && v < a.dv ? S[(long long)c * a.dv + v] : 0.f;
    }
  struct Frag {
    bf16x8 m[MT][KS], q[KS];
    s16x4 b[MT], o;
    float4 e[MT];
  };
  auto load = [&](int i, Frag& f) {
    const long long cb = (long long)(ch0 + i) * a.H + h;
    const bf16_t* gm = p.m + cb * DK * DK + (w * (DK / 4) + l15) * DK + 8 * g4;
    const bf16_t* gq = p.q + cb * CT * DK + (16 * w + l15) * DK + 8 * g4;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
#pragma unroll
      for (int m = 0; m < MT; ++m) f.m[m][k] = *reinterpret_cast<const bf16x8*>(gm + m * 16 * DK + 32 * k);
      f.q[k] = *reinterpret_cast<const bf16x8*>(gq + 32 * k);
    }
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      f.b[m] = row4(p.b + cb * DV * DK + v * DK + r0 + 16 * m);
      f.e[m] = *reinterpret_cast<const float4*>(p.e + cb * DK + r0 + 16 * m);
    }
    f.o = row4(p.oo + cb * DV * CT + v * CT + 16 * w + 4 * g4);
  };
  auto chunk = [&](int i, const Frag& f) {
    bf16_t* im = img[i & 1];
#pragma unroll
    for (int m = 0; m < MT; ++m) *reinterpret_cast<s16x4*>(im + l15 * LS + r0 + 16 * m) = pk4(st[m]);
    __syncthreads();
    f32x4 o = up4(f.o);
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      const f32x4 b = up4(f.b[m]);
      st[m][0] = fmaf(st[m][0], f.e[m].x, b[0]);
      st[m][1] = fmaf(st[m][1], f.e[m].y, b[1]);
      st[m][2] = fmaf(st[m][2], f.e[m].z, b[2]);
      st[m][3] = fmaf(st[m][3], f.e[m].w, b[3]);
    }
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const bf16x8 x = *reinterpret_cast<const bf16x8*>(im + l15 * LS + 32 * k + 8 * g4);
#pragma unroll
      for (int m = 0; m < MT; ++m) st[m] = mm32(f.m[m][k], x, st[m]);
      o = mm32(f.q[k], x, o);
    }
    if (v < a.dv)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = i * CT + 16 * w + 4 * g4 + r;
        if (t < n) a.o[((long long)(row0 + t) * a.H + h) * a.dv + v] = o[r];
      }
  };
  Frag f0, f1;
  load(0, f0);
  for (int i = 0; i < nc; i += 2) {  // the next chunk's maps are in flight under this one's products
    if (i + 1 < nc) load(i + 1, f1);
    chunk(i, f0);
    if (i + 1 < nc) {
      if (i + 2 < nc) load(i + 2, f0);
      chunk(i + 1, f1);
    }
  }
#pragma unroll
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int c = r0 + 16 * m + r;
      if (c < a.dk && v < a.dv) S[(long long)c * a.dv + v] = st[m][r];
    }
}

template <int KIND, int DK, int DV>
int map_go(const ChunkArgs& p, int nchunk, hipStream_t s) {
  auto kern = delta_map_kernel<KIND, DK, DV>;
  constexpr int lds = sizeof(Lds<KIND, DK, DV>);
  static_assert(lds <= 160 * 1024, "LDS");
  if (hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess) return 5;
  hipLaunchKernelGGL(kern, dim3(nchunk * p.d.H), dim3(512), lds, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
template <int DK, int DV>
int run_go(const ChunkArgs& p, int nent, hipStream_t s) {
  hipLaunchKernelGGL((delta_run_kernel<DK, DV>), dim3(p.d.H * ((p.d.dv + 15) / 16), nent), dim3(256), 0, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

bool chunk_ok(const ChunkArgs& p, int kind) {
  const DeltaArgs& a = p.d;
  return delta_args_ok(a, kind) && a.dk % 8 == 0 && a.dv % 8 == 0 && a.dk <= 128 && a.dv <= 128 && a.taps <= 4 && a.ld % 2 == 0 &&
         a.ldw % 2 == 0 && a.o_q % 2 == 0 && a.o_k % 2 == 0 && a.o_v % 2 == 0 && a.o_a % 2 == 0 && (uintptr_t)a.x % 4 == 0 &&
         (uintptr_t)a.dw % 4 == 0 && (uintptr_t)a.w0 % 4 == 0 && (uintptr_t)a.ab % 4 == 0 && a.dw && a.o && p.ck && p.en &&
         p.m && p.b && p.q && p.oo && p.e;
}

}  // namespace

KCA_API int kca_delta_chunk_abi() { return (int)sizeof(ChunkArgs); }

// bf16. Maps of nchunk chunks; 10: sizes for the token-by-token kernels
KCA_API int kca_delta_map(const ChunkArgs* in, int kind, int nchunk, hipStream_t s) {
  const ChunkArgs& p = *in;
  if (nchunk < 1 || (long long)nchunk * p.d.H > 0x7fffffff) return 1;
  if (!chunk_ok(p, kind)) return 10;
  const bool k1 = p.d.dk > 64, v1 = p.d.dv > 64;
  if (kind == 0) return k1 ? map_go<0, 128, 128>(p, nchunk, s) : map_go<0, 64, 64>(p, nchunk, s);
  if (k1) return v1 ? map_go<1, 128, 128>(p, nchunk, s) : map_go<1, 128, 64>(p, nchunk, s);
  return v1 ? map_go<1, 64, 128>(p, nchunk, s) : map_go<1, 64, 64>(p, nchunk, s);
}

// a.o of nent entries from the maps; the slots' states advance
KCA_API int kca_delta_run(const ChunkArgs* in, int kind, int nent, hipStream_t s) {
  const ChunkArgs& p = *in;
  if (nent < 1 || nent > 65535) return 1;
  if (!chunk_ok(p, kind)) return 10;
  const bool k1 = p.d.dk > 64, v1 = p.d.dv > 64;
  if (k1) return v1 ? run_go<128, 128>(p, nent, s) : run_go<128, 64>(p, nent, s);
  return v1 ? run_go<64, 128>(p, nent, s) : run_go<64, 64>(p, nent, s);
}
