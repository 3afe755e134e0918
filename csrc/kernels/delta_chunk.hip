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
// KIND 1 and 2 have p = -k: N = -A_zk, A_qp = -A_qk, so half of the products fall together.
// KIND 2 has one decay per head: its products need no decayed images, the decays multiply the fp32 sums exactly
// (head_map_kernel).
#include "attn_tile.h"
#include "chunk_ops.h"
#include "delta_rule.h"

namespace {
using namespace delta;

constexpr float kFloor = -10.f;

struct ChunkArgs {
  DeltaArgs d;
  const int* ck;         // [nchunk][4]: first row, rows, first row of the entry, position of the chunk's first row
  const int* en;         // [nent][6]: first row, rows, position, slot, first chunk, chunks
  // the maps lie as the run kernel's lanes read them, every fragment of a wave contiguous:
  bf16_t* m;             // [nchunk][H][DK / 16][DK / 32][64 lanes][8]: M[c = lane & 15][c' = 8 (lane >> 4) ..]
  bf16_t* b;             // [nchunk][H][DV / 16][DK / 16][64 lanes][4]: B[c = 4 (lane >> 4) ..][v = lane & 15]
  bf16_t* q;             // [nchunk][H][4][DK / 32][64 lanes][8]: Q'[t = lane & 15][c' = 8 (lane >> 4) ..]
  bf16_t* oo;            // [nchunk][H][DV / 16][4][64 lanes][4]: O'[t = 4 (lane >> 4) ..][v = lane & 15]
  float* e;              // [nchunk][H][DK]: decay of the whole chunk
};

// CPL neighbouring channels as loaded
template <int CPL>
__device__ __forceinline__ uint32_t ldr(const bf16_t* p) {
  if constexpr (CPL == 2) return *reinterpret_cast<const uint32_t*>(p);
  else return *p;
}
template <int CPL>
__device__ __forceinline__ void unr(uint32_t u, bool ok, float (&v)[CPL]) {
  v[0] = ok ? __uint_as_float(u << 16) : 0.f;
  if constexpr (CPL == 2) v[1] = ok ? __uint_as_float(u & 0xffff0000u) : 0.f;
}
// sum over the wave, the same scalar for every lane
__device__ __forceinline__ float wave_total(float x) {
  x = lanes_reduce<16>(x, [](float a, float b) { return a + b; });
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x142, 0xa, 0xf, true));  // rows 1, 3 += rows 0, 2
  x += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x143, 0xc, 0xf, true));  // rows 2, 3 += row 1
  return __int_as_float(__builtin_amdgcn_readlane(__float_as_int(x), 63));
}
template <int CPL>
__device__ __forceinline__ void stc(bf16_t* p, const float (&v)[CPL]) {
  if constexpr (CPL == 2) *reinterpret_cast<uint32_t*>(p) = pk2(v[0], v[1]);
  else *p = f2bf(v[0]);
}

template <int KIND, int DK, int DV>
struct Lds {
  static constexpr int LK = DK + 8, LV = DV + 8, LA = CT + 8;
  static constexpr int L3 = KIND == 2 ? 8 : 16 * LK;
  bf16_t lq[CT * LK], lz[CT * LK], rk[KIND == 2 ? 8 : CT * LK], rp[KIND == 0 ? CT * LK : 8];  // first the diagonal blocks' operands
  bf16_t lq3[L3], lz3[L3];                                  // block 3's rows relative to block 2's start
  bf16_t rk0[L3], rp0[KIND == 0 ? 16 * LK : 8];             // block 0's columns relative to block 1's end
  bf16_t v[CT * LV];
  bf16_t azk[CT * LA], aqk[CT * LA], aqp[KIND == 0 ? CT * LA : 8];
  bf16_t nb[KIND == 0 ? CT * LA : 8];  // N (KIND 1, 2: -azk)
  // its diagonal blocks, the inverses of I - those (KIND 2: in their place)
  float nd[4][16][20], ti_[KIND == 2 ? 1 : 4][16][20];
  __device__ __forceinline__ float (&ti())[4][16][20] {
    if constexpr (KIND == 2) return nd;
    else return ti_;
  }
  float tot[KIND == 2 ? 1 : 8][DK];  // log decay of every 8 tokens
  float pre[KIND == 2 ? 1 : 4][DK];  // decay from the chunk's start to the block's
  // KIND 2: decay from the chunk's start to the token, its log; write strengths, also decayed to the chunk's end
  float fr[CT], lg[CT], beta[CT], late[CT];
};

// Solve and maps of one (chunk, head) from its LDS images, 16 columns of [W | U] a wave and turn
template <int KIND, int DK, int DV, int NW = 8>
__device__ __forceinline__ void chunk_maps(Lds<KIND, DK, DV>& s, const ChunkArgs& p, long long cb, int w) {
  using L = Lds<KIND, DK, DV>;
  constexpr int KS = DK / 32;
  const int lane = threadIdx.x & 63, l15 = lane & 15, g4 = lane >> 4;
  bf16_t* gm = p.m + cb * DK * DK;
  bf16_t* gb = p.b + cb * DV * DK;
  bf16_t* gq = p.q + cb * CT * DK;
  bf16_t* go = p.oo + cb * DV * CT;
  auto solve = [&](int I, f32x4 y, const f32x4* X, const s16x4* sb) {  // (I - N) X = Y, one block row
    if (I == 1) y = mm16(row4((KIND == 0 ? s.nb : s.azk) + (16 + l15) * L::LA + 4 * g4), sb[0], y);
    if (I >= 2) {
      const bf16_t* nr = (KIND == 0 ? s.nb : s.azk) + (16 * I + l15) * L::LA + 4 * g4;
      y = mm32(two(row4(nr), row4(nr + 16)), two(sb[0], sb[1]), y);
      if (I == 3) y = mm16(row4(nr + 32), sb[2], y);
    }
    return mm16f(*reinterpret_cast<const float4*>(&s.ti()[I][l15][4 * g4]), y, f32x4{0.f, 0.f, 0.f, 0.f});
  };
  // sum over the token blocks 0 .. I of rows (of A at `rows`) times operands x
  auto low = [&](const bf16_t* rows, int I, const s16x4* x, f32x4 y, bool rows_first) {
    const bf16_t* r = rows + (16 * I + l15) * L::LA + 4 * g4;
    if (I == 0) return rows_first ? mm16(row4(r), x[0], y) : mm16(x[0], row4(r), y);
    const bf16x8 ra = two(row4(r), row4(r + 16)), xa = two(x[0], x[1]);
    y = rows_first ? mm32(ra, xa, y) : mm32(xa, ra, y);
    if (I == 2) y = rows_first ? mm16(row4(r + 32), x[2], y) : mm16(x[2], row4(r + 32), y);
    if (I == 3) {
      const bf16x8 rb = two(row4(r + 32), row4(r + 48)), xc = two(x[2], x[3]);
      y = rows_first ? mm32(rb, xc, y) : mm32(xc, rb, y);
    }
    return y;
  };
  // KIND 2: rows of X decayed to the chunk's end, for the plain key image
  auto to_end = [&](const f32x4 (&X)[4], s16x4 (&xb)[4], float sign) {
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      const float4 l = *reinterpret_cast<const float4*>(&s.late[16 * I + 4 * g4]);
      xb[I] = pk4(f32x4{X[I][0] * l.x, X[I][1] * l.y, X[I][2] * l.z, X[I][3] * l.w} * sign);
    }
  };
  auto wtile = [&](int col) {  // 16 columns of W -> M, Q'
    f32x4 X[4];
    s16x4 xb[4], sb[4];
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      f32x4 y;
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * I + 4 * g4 + r;
        y[r] = bf2f(s.lz[t * L::LK + col + l15]) * (KIND == 2 ? s.fr[t] : s.pre[I][col + l15]);
      }
      X[I] = solve(I, y, X, sb);
      xb[I] = pk4(X[I]);
      if (KIND >= 1) xb[I] = neg4(xb[I]);  // N, P and A_qp carry a minus sign
      sb[I] = xb[I];
    }
    const int cw = col + 4 * g4;  // this lane's four columns c'
    const int fo = ((col >> 5) * 64 + ((col >> 3 & 2) + (g4 >> 1)) * 16 + l15) * 8 + (g4 & 1) * 4;
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      f32x4 y = up4(row4(s.lq + (16 * I + l15) * L::LK + cw));
      if constexpr (KIND == 2) {
        y *= s.fr[16 * I + l15];
      } else {
        const float4 fp = *reinterpret_cast<const float4*>(&s.pre[I][cw]);
        y[0] *= fp.x; y[1] *= fp.y; y[2] *= fp.z; y[3] *= fp.w;
      }
      *reinterpret_cast<s16x4*>(gq + I * KS * 512 + fo) = pk4(low(KIND == 0 ? s.aqp : s.aqk, I, xb, y, false));
    }
    if constexpr (KIND == 2) to_end(X, xb, -1.f);
    const bf16x8 x01 = two(xb[0], xb[1]), x23 = two(xb[2], xb[3]);
    const bf16_t* img = KIND == 0 ? s.rp : KIND == 1 ? s.rk : s.lz;
#pragma unroll 4
    for (int c = 0; c < DK; c += 16) {
      f32x4 y = mm32(x01, two(tok4<L::LK>(img, 0, c), tok4<L::LK>(img, 16, c)), f32x4{0.f, 0.f, 0.f, 0.f});
      y = mm32(x23, two(tok4<L::LK>(img, 32, c), tok4<L::LK>(img, 48, c)), y);
      *reinterpret_cast<s16x4*>(gm + (c >> 4) * KS * 512 + fo) = pk4(y);
    }
  };
  auto utile = [&](int col) {  // 16 columns of U -> B, O'
    f32x4 X[4];
    s16x4 vb[4], xb[4], sb[4];
#pragma unroll
    for (int I = 0; I < 4; ++I) vb[I] = tok4<L::LV>(s.v, 16 * I, col);
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      X[I] = solve(I, low(s.azk, I, vb, f32x4{0.f, 0.f, 0.f, 0.f}, true), X, sb);
      sb[I] = xb[I] = pk4(X[I]);
      if (KIND >= 1) {
        sb[I] = neg4(sb[I]);
        const f32x4 d = up4(vb[I]) - X[I];  // V - U
        xb[I] = pk4(d);
        if (KIND == 2) X[I] = d;
      }
    }
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      f32x4 y = low(KIND == 0 ? s.aqp : s.aqk, I, xb, f32x4{0.f, 0.f, 0.f, 0.f}, true);
      if constexpr (KIND == 0) y = low(s.aqk, I, vb, y, true);
      *reinterpret_cast<s16x4*>(go + ((col >> 4) * 4 + I) * 256 + lane * 4) = pk4(y);
    }
    if constexpr (KIND == 2) to_end(X, xb, 1.f);  // (X: V - U by now)
    const bf16x8 x01 = two(xb[0], xb[1]), x23 = two(xb[2], xb[3]), v01 = two(vb[0], vb[1]), v23 = two(vb[2], vb[3]);
    const bf16_t* img = KIND == 0 ? s.rp : KIND == 1 ? s.rk : s.lz;
#pragma unroll 4
    for (int c = 0; c < DK; c += 16) {
      f32x4 y = mm32(two(tok4<L::LK>(img, 0, c), tok4<L::LK>(img, 16, c)), x01, f32x4{0.f, 0.f, 0.f, 0.f});
      y = mm32(two(tok4<L::LK>(img, 32, c), tok4<L::LK>(img, 48, c)), x23, y);
      if constexpr (KIND == 0) {
        y = mm32(two(tok4<L::LK>(s.rk, 0, c), tok4<L::LK>(s.rk, 16, c)), v01, y);
        y = mm32(two(tok4<L::LK>(s.rk, 32, c), tok4<L::LK>(s.rk, 48, c)), v23, y);
      }
      *reinterpret_cast<s16x4*>(gb + ((col >> 4) * (DK / 16) + (c >> 4)) * 256 + lane * 4) = pk4(y);
    }
  };
  if constexpr (DK == 128 && DV == 128 && NW == 8) {
    wtile(16 * w);
    utile(16 * w);
  } else {
#pragma unroll 1
    for (int ct = w; ct < (DK + DV) / 16; ct += NW) {
      if (ct < DK / 16) wtile(16 * ct);
      else utile(16 * ct - DK);
    }
  }
}

// One wave's operands of an item as loaded: its 8 tokens (KIND 1: and the 3 rows before) of each column block
template <int KIND>
struct Raw {
  static constexpr int NR = KIND == 0 ? 8 : 11;
  uint32_t q[NR], k[NR], v[NR], a[8], w[8], w0, ab;
  uint32_t tq[KIND ? 4 : 1], tk[KIND ? 4 : 1], tv[KIND ? 4 : 1];  // taps of two channels
};

// A workgroup walks (chunk, head) items; an item's loads are issued while the one before is solved.
template <int KIND, int DK, int DV>
__global__ void __launch_bounds__(512) delta_map_kernel(ChunkArgs p, int items) {
  using L = Lds<KIND, DK, DV>;
  constexpr int CPL = DK / 64, CPV = DV / 64, KS = DK / 32;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  L& s = *reinterpret_cast<L*>(smem);
  const DeltaArgs& a = p.d;
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l15 = lane & 15, g4 = lane >> 4, blk = w >> 1, half = w & 1;
  const int c0 = lane * CPL, cv = lane * CPV, t0 = 8 * w;
  const bool inc = c0 < a.dk, inv = cv < a.dv;
  const int cs = inc ? c0 : 0, vs = inv ? cv : 0;  // channels that exist
  const int nqk = a.G * a.dk, per = a.H / a.G;

  // at addresses that exist: rows past the end repeat others and are blanked at their use
  auto fetch = [&](int item, Raw<KIND>& r) {
    const int ci = item / a.H, h = item - ci * a.H;
    const int* ck = p.ck + ci * 4;
    const int row0 = ck[0], n = ck[1], first = ck[2];
    const bf16_t* x = reinterpret_cast<const bf16_t*>(a.x);
    const bf16_t* dw = reinterpret_cast<const bf16_t*>(a.dw) + h * a.dk + cs;
    r.w0 = ldr<CPL>(reinterpret_cast<const bf16_t*>(a.w0) + h * a.dk + cs);
    if constexpr (KIND == 0) r.ab = ldr<CPL>(reinterpret_cast<const bf16_t*>(a.ab) + h * a.dk + cs);
    else r.ab = reinterpret_cast<const bf16_t*>(a.ab)[h];
    const int gq = KIND == 0 ? h : h / per;
#pragma unroll
    for (int i = 0; i < Raw<KIND>::NR; ++i) {
      const int t = KIND == 0 ? t0 + i : t0 + i - 3;
      const bf16_t* xr = x + (long long)min(KIND == 0 ? row0 + t : max(row0 + t, first), row0 + n - 1) * a.ld;
      r.q[i] = ldr<CPL>(xr + a.o_q + gq * a.dk + cs);
      r.k[i] = ldr<CPL>(xr + a.o_k + gq * a.dk + cs);
      r.v[i] = ldr<CPV>(xr + a.o_v + h * a.dv + vs);
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const long long t = row0 + min(t0 + i, n - 1);
      r.w[i] = ldr<CPL>(dw + t * a.ldw);
      if constexpr (KIND == 0) r.a[i] = ldr<CPL>(x + t * a.ld + a.o_a + h * a.dk + cs);
      else r.a[i] = x[t * a.ld + a.o_a + h];
    }
    if constexpr (KIND == 1) {
      const bf16_t* cw = reinterpret_cast<const bf16_t*>(a.conv);
      const int chq = gq * a.dk + cs, chk = nqk + chq, chv = 2 * nqk + h * a.dv + vs;
#pragma unroll
      for (int i = 0; i < 4; ++i) {  // tap i: the row i tokens back
        const int o = max(a.taps - 1 - i, 0);
        r.tq[i] = cw[chq * a.taps + o] | (uint32_t)cw[(chq + CPL - 1) * a.taps + o] << 16;
        r.tk[i] = cw[chk * a.taps + o] | (uint32_t)cw[(chk + CPL - 1) * a.taps + o] << 16;
        r.tv[i] = cw[chv * a.taps + o] | (uint32_t)cw[(chv + CPV - 1) * a.taps + o] << 16;
      }
    }
  };
  Raw<KIND> raw;
  fetch(blockIdx.x, raw);
#pragma unroll 1
  for (int item = blockIdx.x; item < items; item += gridDim.x) {
  const int ci = item / a.H, h = item - ci * a.H;
  const int* ck = p.ck + ci * 4;
  const int row0 = ck[0], n = ck[1], first = ck[2], pos0 = ck[3];

  // ------------------------------------------------------- vectors of 8 tokens, CPL channels a lane
  float q[8][CPL], u[8][CPL], pv[8][CPL], G[8][CPL], kn[8];
  {
    if constexpr (KIND == 0) {
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const bool ok = t0 + i < n;
        float v[CPV];
        unr<CPL>(raw.q[i], ok && inc, q[i]);
        unr<CPL>(raw.k[i], ok && inc, u[i]);
        unr<CPL>(raw.a[i], ok && inc, pv[i]);
        unr<CPV>(raw.v[i], ok && inv, v);
        stc<CPV>(s.v + (t0 + i) * L::LV + cv, v);
      }
    } else {
      float hq[3][CPL], hk[3][CPL], hv[3][CPV];  // the three rows before
      if (w == 0 && row0 == first) {             // ... which the sequence's slot keeps
        const int slot = a.slot[row0], C = 2 * nqk + a.H * a.dv;
        const int chq = h / per * a.dk + cs, chk = nqk + chq, chv = 2 * nqk + h * a.dv + vs;
#pragma unroll
        for (int i = 0; i < 3; ++i) {
          const int ps = pos0 + i - 3;
          const bool ok = ps >= 0 && 3 - i < a.taps;
          const float* r = a.ring + ((long long)slot * a.taps + (ok ? ps % a.taps : 0)) * C;
#pragma unroll
          for (int e = 0; e < CPL; ++e) {
            const float x0 = r[chq + e], x1 = r[chk + e];
            hq[i][e] = ok ? x0 : 0.f;
            hk[i][e] = ok ? x1 : 0.f;
          }
#pragma unroll
          for (int e = 0; e < CPV; ++e) {
            const float x2 = r[chv + e];
            hv[i][e] = ok ? x2 : 0.f;
          }
        }
      } else {
#pragma unroll
        for (int i = 0; i < 3; ++i) {
          unr<CPL>(raw.q[i], true, hq[i]);
          unr<CPL>(raw.k[i], true, hk[i]);
          unr<CPV>(raw.v[i], true, hv[i]);
        }
      }
      auto conv = [&](auto cpl, const auto& hist, const auto& rw, const auto& tap, bool okc, auto&& put) {
        constexpr int N = decltype(cpl)::value;
        float tp[4][N], p1[N], p2[N], p3[N];
#pragma unroll
        for (int i = 0; i < 4; ++i) unr<N>(tap[i], i < a.taps, tp[i]);
#pragma unroll
        for (int e = 0; e < N; ++e) p3[e] = hist[0][e], p2[e] = hist[1][e], p1[e] = hist[2][e];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          float z[N], y[N];
          unr<N>(rw[i + 3], true, z);
          const bool ok = okc && t0 + i < n;
#pragma unroll
          for (int e = 0; e < N; ++e) {
            const float v = fmaf(tp[3][e], p3[e], fmaf(tp[2][e], p2[e], fmaf(tp[1][e], p1[e], tp[0][e] * z[e])));
            y[e] = ok ? v * __builtin_amdgcn_rcpf(1.f + __expf(-v)) : 0.f;
            p3[e] = p2[e];
            p2[e] = p1[e];
            p1[e] = z[e];
          }
          put(i, y);
        }
      };
      conv(std::integral_constant<int, CPL>{}, hq, raw.q, raw.tq, inc, [&](int i, const float (&y)[CPL]) {
#pragma unroll
        for (int e = 0; e < CPL; ++e) q[i][e] = y[e];
      });
      conv(std::integral_constant<int, CPL>{}, hk, raw.k, raw.tk, inc, [&](int i, const float (&y)[CPL]) {
#pragma unroll
        for (int e = 0; e < CPL; ++e) u[i][e] = y[e];
      });
      conv(std::integral_constant<int, CPV>{}, hv, raw.v, raw.tv, inv,
           [&](int i, const float (&y)[CPV]) { stc<CPV>(s.v + (t0 + i) * L::LV + cv, y); });
    }
    float w0[CPL], ab[CPL], run[CPL];
    unr<CPL>(raw.w0, true, w0);
    if constexpr (KIND == 0) unr<CPL>(raw.ab, true, ab);
    const float A = KIND == 1 ? __expf(__uint_as_float(raw.ab << 16)) : 0.f;
#pragma unroll
    for (int e = 0; e < CPL; ++e) run[e] = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const bool ok = t0 + i < n;
      float lw[CPL], sk = 0.f, sq = 0.f;
      unr<CPL>(raw.w[i], true, lw);
#pragma unroll
      for (int e = 0; e < CPL; ++e) {
        sk = fmaf(u[i][e], u[i][e], sk);
        sq = fmaf(q[i][e], q[i][e], sq);
      }
      sk = wave_total(sk) + 1e-6f;
      const float ik = rsqrtf(sk);
      float iq = 1.f;
      kn[i] = sk * ik;  // k = u * kn
      if constexpr (KIND == 1) {
        iq = a.qscale * rsqrtf(wave_total(sq) + 1e-6f);
        kn[i] = ok ? __builtin_amdgcn_rcpf(1.f + __expf(-__uint_as_float(raw.a[i] << 16))) : 0.f;
      }
#pragma unroll
      for (int e = 0; e < CPL; ++e) {
        const float z = lw[e] + w0[e];
        float l;
        if constexpr (KIND == 0) l = -0.60653065971263342f * __builtin_amdgcn_rcpf(1.f + __expf(-z));
        else l = fmaxf(-A * (fmaxf(z, 0.f) + __logf(1.f + __expf(-fabsf(z)))), kFloor);
        run[e] += ok && inc ? l : 0.f;
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
  // decays of what lies before the blocks
  if (tid < DK) {
    float acc = 0.f;
#pragma unroll
    for (int b = 0; b < 4; ++b) {
      const float t = s.tot[2 * b][tid] + s.tot[2 * b + 1][tid];
      s.pre[b][tid] = __expf(acc);
      acc += t;
    }
    p.e[((long long)ci * a.H + h) * DK + tid] = __expf(acc);
  }
  // decays of the tokens relative to their block's middle: f = e^(G - mid); b0: of the token before the first
  float f[8][CPL], fi[8][CPL], b0[CPL], em[CPL], er[CPL];
#pragma unroll
  for (int e = 0; e < CPL; ++e) {
    const float mid = s.tot[w & ~1][c0 + e], late = s.tot[w | 1][c0 + e];
    em[e] = __expf(mid);   // from the block's start to its middle
    er[e] = __expf(late);  // ... from there to its end
    b0[e] = half ? 1.f : __expf(-mid);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      f[i][e] = __expf(half ? G[i][e] : G[i][e] - mid);
      fi[i][e] = __builtin_amdgcn_rcpf(f[i][e]);
    }
  }
  // The four operand images. PASS 0: relative to the block's middle on both sides (diagonal blocks); 1: to its
  // start and end, with block 3's rows and block 0's columns also a block further; 2: the columns alone, decayed
  // to the chunk's end
  auto image = [&](auto pass) {
    constexpr int PASS = decltype(pass)::value;
    float fx[CPL], fe[CPL];
#pragma unroll
    for (int e = 0; e < CPL; ++e) {
      fx[e] = 1.f;
      fe[e] = PASS ? er[e] : 1.f;
      if (PASS == 1 && (blk == 3 || blk == 0)) {
        const int o = blk == 3 ? 4 : 2;
        fx[e] = __expf(s.tot[o][c0 + e] + s.tot[o + 1][c0 + e]);
      }
      if (PASS == 2) {
        float z = 0.f;
        for (int o = 2 * blk + 2; o < 8; ++o) z += s.tot[o][c0 + e];
        fe[e] *= __expf(z);
      }
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int o = (8 * w + i) * L::LK + c0, o1 = (8 * half + i) * L::LK + c0;
      float yq[CPL], yz[CPL], yk[CPL], yp[CPL];
#pragma unroll
      for (int e = 0; e < CPL; ++e) {
        const float fr = fi[i][e] * fe[e];
        yk[e] = u[i][e] * kn[i] * fr;
        if constexpr (KIND == 0) yp[e] = pv[i][e] * fr;
        if constexpr (PASS < 2) {
          const float before = i ? f[i ? i - 1 : 0][e] : b0[e];
          yq[e] = q[i][e] * f[i][e];
          yz[e] = u[i][e] * (KIND == 0 ? before : f[i][e]);
          if (PASS == 1) yq[e] *= em[e], yz[e] *= em[e];
        }
      }
      stc<CPL>(s.rk + o, yk);
      if constexpr (KIND == 0) stc<CPL>(s.rp + o, yp);
      if constexpr (PASS < 2) {
        stc<CPL>(s.lq + o, yq);
        stc<CPL>(s.lz + o, yz);
      }
      if constexpr (PASS == 1) {
        if (blk == 3) {
#pragma unroll
          for (int e = 0; e < CPL; ++e) yq[e] *= fx[e], yz[e] *= fx[e];
          stc<CPL>(s.lq3 + o1, yq);
          stc<CPL>(s.lz3 + o1, yz);
        } else if (blk == 0) {
#pragma unroll
          for (int e = 0; e < CPL; ++e) {
            yk[e] *= fx[e];
            if constexpr (KIND == 0) yp[e] *= fx[e];
          }
          stc<CPL>(s.rk0 + o1, yk);
          if constexpr (KIND == 0) stc<CPL>(s.rp0 + o1, yp);
        }
      }
    }
  };
  image(std::integral_constant<int, 0>{});
  __syncthreads();
  // ---------------------------------------------- decayed products: rows of block `blk`, z (half 0) or q (half 1)
  f32x4 ak[4], ap[4];
  auto block = [&](int J, const bf16_t* left, const bf16_t* rk, const bf16_t* rp) {
    f32x4 x = {0.f, 0.f, 0.f, 0.f}, y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int o = l15 * L::LK + k * 32 + 8 * g4;
      const bf16x8 fa = *reinterpret_cast<const bf16x8*>(left + o);
      x = mm32(fa, *reinterpret_cast<const bf16x8*>(rk + o), x);
      if constexpr (KIND == 0) y = mm32(fa, *reinterpret_cast<const bf16x8*>(rp + o), y);
    }
    ak[J] = x;
    ap[J] = y;
  };
  constexpr int BR = 16 * L::LK;  // a block's rows
  const bf16_t *left = (half ? s.lq : s.lz) + blk * BR, *left3 = half ? s.lq3 : s.lz3;
#pragma unroll
  for (int J = 0; J < 4; ++J)
    if (J == blk) {
      block(J, left, s.rk + J * BR, s.rp + (KIND == 0 ? J * BR : 0));
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (half ? l15 > 4 * g4 + r : l15 >= 4 * g4 + r) ak[J][r] = ap[J][r] = 0.f;
      if (!half)
#pragma unroll
        for (int r = 0; r < 4; ++r) s.nd[blk][4 * g4 + r][l15] = KIND == 0 ? ap[J][r] : -ak[J][r];
    }
  __syncthreads();
  image(std::integral_constant<int, 1>{});
  __syncthreads();
#pragma unroll
  for (int J = 0; J < 3; ++J)
    if (J < blk) {
      const bool far = blk >= 2 && J < 2;  // rows from block 2's start, columns to block 1's end
      block(J, far && blk == 3 ? left3 : left, far && J == 0 ? s.rk0 : s.rk + J * BR,
            KIND == 1 ? s.rp : far && J == 0 ? s.rp0 : s.rp + J * BR);
    }
#pragma unroll
  for (int J = 0; J < 4; ++J)
    if (J <= blk)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int t = 16 * blk + 4 * g4 + r, j = 16 * J + l15;
        (half ? s.aqk : s.azk)[t * L::LA + j] = f2bf(ak[J][r]);
        if constexpr (KIND == 0) (half ? s.aqp : s.nb)[t * L::LA + j] = f2bf(ap[J][r]);
      }
  // inverses of the four diagonal blocks, a lane per (block, column), by a wave without products of its own here
  if (w == 0) {
    float x[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      float v = r == l15 ? 1.f : 0.f;
#pragma unroll
      for (int k = 0; k < r; ++k) v = fmaf(s.nd[g4][r][k], x[k], v);
      x[r] = v;
      s.ti()[g4][r][l15] = v;
    }
  }
  __syncthreads();
  image(std::integral_constant<int, 2>{});
  fetch(min(item + (int)gridDim.x, items - 1), raw);
  __syncthreads();
  chunk_maps<KIND, DK, DV>(s, p, (long long)ci * a.H + h, w);
  __syncthreads();  // the next item reuses the LDS
  }
}

// KIND 2 from convolution results: four threads a token make the vectors, a lane a token the decays. Two workgroups
// a CU, so that one solves while the other loads and stores.
template <int DK, int DV>
__global__ void __launch_bounds__(256, 2) head_map_kernel(ChunkArgs p, int items) {
  using L = Lds<2, DK, DV>;
  constexpr int NK = DK / 32, NV = DV / 32, KS = DK / 32;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  L& s = *reinterpret_cast<L*>(smem);
  const DeltaArgs& a = p.d;
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l15 = lane & 15, g4 = lane >> 4, tok = tid >> 2, sub = tid & 3;
  const int nqk = a.G * a.dk, C = 2 * nqk + a.H * a.dv, per = a.H / a.G;
  struct Raw {
    U16x8 q[NK], k[NK], v[NV];
    bf16_t a, b, w0, al;
  };
  auto fetch = [&](int item, Raw& r) {  // at addresses that exist
    const int ci = item / a.H, h = item - ci * a.H;
    const int* ck = p.ck + ci * 4;
    const long long row0 = ck[0];
    const int n = ck[1];
    const bf16_t* x = reinterpret_cast<const bf16_t*>(a.cx) + (row0 + min(tok, n - 1)) * C;
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int c = sub * 8 + 32 * i < a.dk ? sub * 8 + 32 * i : 0;
      r.q[i] = *reinterpret_cast<const U16x8*>(x + h / per * a.dk + c);
      r.k[i] = *reinterpret_cast<const U16x8*>(x + nqk + h / per * a.dk + c);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i)
      r.v[i] = *reinterpret_cast<const U16x8*>(x + 2 * nqk + h * a.dv + (sub * 8 + 32 * i < a.dv ? sub * 8 + 32 * i : 0));
    const bf16_t* y = reinterpret_cast<const bf16_t*>(a.x) + (row0 + min(lane, n - 1)) * a.ld;
    r.a = y[a.o_w + h];
    r.b = y[a.o_a + h];
    r.w0 = reinterpret_cast<const bf16_t*>(a.w0)[h];
    r.al = reinterpret_cast<const bf16_t*>(a.ab)[h];
  };
  Raw raw;
  fetch(blockIdx.x, raw);
#pragma unroll 1
  for (int item = blockIdx.x; item < items; item += gridDim.x) {
    const int ci = item / a.H, n = p.ck[ci * 4 + 1];
    // a lane a token: running log decays and write strengths
    float G = lane < n ? -expf(bf2f(raw.al)) * softplus(bf2f(raw.a) + bf2f(raw.w0)) : 0.f;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float u = __shfl_up(G, o, 64);
      if (lane >= o) G += u;
    }
    const float end = __shfl(G, 63, 64), beta = lane < n ? sigmoid(bf2f(raw.b)) : 0.f;
    if (w == 0) {
      s.lg[lane] = G;
      s.fr[lane] = __expf(G);
      s.beta[lane] = beta;
      s.late[lane] = __expf(end - G) * beta;
    }
    if (tid < DK) p.e[(long long)item * DK + tid] = __expf(end);
    // four threads a token: unit vectors
    float q[NK][8], k[NK][8], sq = 0.f, sk = 0.f;
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const bool ok = tok < n && sub * 8 + 32 * i < a.dk;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        q[i][e] = ok ? bf2f(raw.q[i].v[e]) : 0.f;
        k[i][e] = ok ? bf2f(raw.k[i].v[e]) : 0.f;
        sq = fmaf(q[i][e], q[i][e], sq);
        sk = fmaf(k[i][e], k[i][e], sk);
      }
    }
    auto add = [](float x, float y) { return x + y; };
    const float iq = a.qscale / sqrtf(lanes_reduce<4>(sq, add) + 1e-6f), ik = 1.f / sqrtf(lanes_reduce<4>(sk, add) + 1e-6f);
#pragma unroll
    for (int i = 0; i < NK; ++i) {
      const int o = tok * L::LK + sub * 8 + 32 * i;
      uint32_t zq[4], zk[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        zq[e] = pk2(q[i][2 * e] * iq, q[i][2 * e + 1] * iq);
        zk[e] = pk2(k[i][2 * e] * ik, k[i][2 * e + 1] * ik);
      }
      *reinterpret_cast<u32x4*>(s.lq + o) = u32x4{zq[0], zq[1], zq[2], zq[3]};
      *reinterpret_cast<u32x4*>(s.lz + o) = u32x4{zk[0], zk[1], zk[2], zk[3]};
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      const bool ok = tok < n && sub * 8 + 32 * i < a.dv;
      *reinterpret_cast<u32x4*>(s.v + tok * L::LV + sub * 8 + 32 * i) =
          ok ? __builtin_bit_cast(u32x4, raw.v[i]) : u32x4{0u, 0u, 0u, 0u};
    }
    __syncthreads();
    // rows of block w, keys and queries, against the keys of the blocks up to it
#pragma unroll
    for (int J = 0; J < 4; ++J)
      if (J <= w) {
        f32x4 xz = {0.f, 0.f, 0.f, 0.f}, xq = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int c = 0; c < KS; ++c) {
          const int o = l15 * L::LK + c * 32 + 8 * g4;
          const bf16x8 kj = *reinterpret_cast<const bf16x8*>(s.lz + 16 * J * L::LK + o);
          xz = mm32(*reinterpret_cast<const bf16x8*>(s.lz + 16 * w * L::LK + o), kj, xz);
          xq = mm32(*reinterpret_cast<const bf16x8*>(s.lq + 16 * w * L::LK + o), kj, xq);
        }
        const int j = 16 * J + l15;
        const float lj = s.lg[j], bj = s.beta[j];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = 16 * w + 4 * g4 + r;
          const float d = bj * __expf(s.lg[t] - lj), z = j < t ? xz[r] * d : 0.f;
          s.azk[t * L::LA + j] = f2bf(z);
          s.aqk[t * L::LA + j] = f2bf(j <= t ? xq[r] * d : 0.f);
          if (J == w) s.nd[w][4 * g4 + r][l15] = -z;
        }
      }
    __syncthreads();
    fetch(min(item + (int)gridDim.x, items - 1), raw);
    if (w == 0) {  // inverses of the four diagonal blocks, a lane per (block, column)
      float x[16];
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        float v = r == l15 ? 1.f : 0.f;
#pragma unroll
        for (int k = 0; k < r; ++k) v = fmaf(s.nd[g4][r][k], x[k], v);
        x[r] = v;
        s.ti()[g4][r][l15] = v;
      }
    }
    __syncthreads();
    chunk_maps<2, DK, DV, 4>(s, p, item, w);
    __syncthreads();  // the next item reuses the LDS
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
    const bf16_t* gm = p.m + cb * DK * DK + w * MT * KS * 512 + lane * 8;
    const bf16_t* gq = p.q + cb * CT * DK + w * KS * 512 + lane * 8;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
#pragma unroll
      for (int m = 0; m < MT; ++m) f.m[m][k] = *reinterpret_cast<const bf16x8*>(gm + (m * KS + k) * 512);
      f.q[k] = *reinterpret_cast<const bf16x8*>(gq + k * 512);
    }
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      f.b[m] = row4(p.b + cb * DV * DK + (vt * (DK / 16) + w * MT + m) * 256 + lane * 4);
      f.e[m] = *reinterpret_cast<const float4*>(p.e + cb * DK + r0 + 16 * m);
    }
    f.o = row4(p.oo + cb * DV * CT + (vt * 4 + w) * 256 + lane * 4);
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
    bf16_t* op = reinterpret_cast<bf16_t*>(a.o) + ((long long)(row0 + i * CT + 16 * w + 4 * g4) * a.H + h) * a.dv + v;
    const long long os = (long long)a.H * a.dv;
    if (vt * 16 + 16 <= a.dv && i * CT + CT <= n) {
#pragma unroll
      for (int r = 0; r < 4; ++r) op[r * os] = f2bf(o[r]);
    } else if (v < a.dv) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (i * CT + 16 * w + 4 * g4 + r < n) op[r * os] = f2bf(o[r]);
    }
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
  for (int m = 0; m < MT; ++m)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int c = r0 + 16 * m + r;
      if (c < a.dk && v < a.dv) S[(long long)c * a.dv + v] = st[m][r];
    }
}

template <int KIND, int DK, int DV>
int map_go(const ChunkArgs& p, int nchunk, hipStream_t s) {
  void (*kern)(ChunkArgs, int);
  if constexpr (KIND == 2) kern = head_map_kernel<DK, DV>;
  else kern = delta_map_kernel<KIND, DK, DV>;
  constexpr int lds = sizeof(Lds<KIND, DK, DV>);
  static_assert(lds <= 160 * 1024, "LDS");
  if (hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess) return 5;
  const int items = nchunk * p.d.H, per_cu = lds <= 80 * 1024 ? 2 : 1;
  hipLaunchKernelGGL(kern, dim3(items < 256 * per_cu ? items : 256 * per_cu), dim3(KIND == 2 ? 256 : 512), lds, s, p, items);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
template <int DK, int DV>
int run_go(const ChunkArgs& p, int nent, hipStream_t s) {
  hipLaunchKernelGGL((delta_run_kernel<DK, DV>), dim3(p.d.H * ((p.d.dv + 15) / 16), nent), dim3(256), 0, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

bool chunk_ok(const ChunkArgs& p, int kind) {
  const DeltaArgs& a = p.d;
  if (kind == 2)
    return delta_args_ok(a, kind) && a.dk % 8 == 0 && a.dv % 8 == 0 && a.dk <= 128 && a.dv <= 128 && (uintptr_t)a.cx % 16 == 0 &&
           a.cx && a.o && p.ck && p.en && p.m && p.b && p.q && p.oo && p.e;
  return kind < 2 && delta_args_ok(a, kind) && a.dk % 8 == 0 && a.dv % 8 == 0 && a.dk <= 128 && a.dv <= 128 && a.taps <= 4 && a.ld % 2 == 0 &&
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
  if (kind == 2) {
    if (k1) return v1 ? map_go<2, 128, 128>(p, nchunk, s) : map_go<2, 128, 64>(p, nchunk, s);
    return v1 ? map_go<2, 64, 128>(p, nchunk, s) : map_go<2, 64, 64>(p, nchunk, s);
  }
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
