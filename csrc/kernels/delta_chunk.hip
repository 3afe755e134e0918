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
  // the maps lie as the run kernel's lanes read them, every fragment of a wave contiguous:
  bf16_t* m;             // [nchunk][H][DK / 16][DK / 32][64 lanes][8]: M[c = lane & 15][c' = 8 (lane >> 4) ..]
  bf16_t* b;             // [nchunk][H][DV / 16][DK / 16][64 lanes][4]: B[c = 4 (lane >> 4) ..][v = lane & 15]
  bf16_t* q;             // [nchunk][H][4][DK / 32][64 lanes][8]: Q'[t = lane & 15][c' = 8 (lane >> 4) ..]
  bf16_t* oo;            // [nchunk][H][DV / 16][4][64 lanes][4]: O'[t = 4 (lane >> 4) ..][v = lane & 15]
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
  if constexpr (CPL == 2) *reinterpret_cast<uint32_t*>(p) = pack_bf16x2(v[0], v[1]);
  else *p = f2bf(v[0]);
}

template <int KIND, int DK, int DV>
struct Lds {
  static constexpr int LK = DK + 8, LV = DV + 8, LA = CT + 8;
  bf16_t lq[CT * LK], lz[CT * LK], rk[CT * LK], rp[KIND == 0 ? CT * LK : 8];  // first the diagonal blocks' operands
  bf16_t v[CT * LV];
  bf16_t azk[CT * LA], aqk[CT * LA], aqp[KIND == 0 ? CT * LA : 8];
  bf16_t nb[KIND == 0 ? CT * LA : 8];  // N (KIND 1: -azk)
  float nd[4][16][20], ti[4][16][20];  // its diagonal blocks, the inverses of I - those
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
    const int t0 = 8 * w, cv = lane * CPV, cs = inc ? c0 : 0, vs = cv < a.dv ? cv : 0;
    const bool inv = cv < a.dv;
    const int gq = h / (a.H / a.G), nqk = a.G * a.dk;
    // every load is issued before the first use, at addresses that exist: rows and channels past the end repeat
    // others and are blanked afterwards
    uint32_t rw[8], rb[8];
    const bf16_t* dw = reinterpret_cast<const bf16_t*>(a.dw) + h * a.dk + cs;
    const uint32_t rw0 = ldr<CPL>(reinterpret_cast<const bf16_t*>(a.w0) + h * a.dk + cs);
    uint32_t rab = 0;
    if constexpr (KIND == 0) rab = ldr<CPL>(reinterpret_cast<const bf16_t*>(a.ab) + h * a.dk + cs);
    else rab = reinterpret_cast<const bf16_t*>(a.ab)[h];
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const long long r = row0 + min(t0 + i, n - 1);
      rw[i] = ldr<CPL>(dw + r * a.ldw);
      if constexpr (KIND == 1) rb[i] = x[r * a.ld + a.o_a + h];
    }
    if constexpr (KIND == 0) {
      uint32_t rq[8], rk[8], ra[8], rv[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const bf16_t* xr = x + (long long)(row0 + min(t0 + i, n - 1)) * a.ld + h * a.dk + cs;
        rq[i] = ldr<CPL>(xr + a.o_q);
        rk[i] = ldr<CPL>(xr + a.o_k);
        ra[i] = ldr<CPL>(xr + a.o_a);
        rv[i] = ldr<CPV>(xr + a.o_v);  // (dk = dv)
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const bool ok = t0 + i < n;
        float v[CPV];
        unr<CPL>(rq[i], ok && inc, q[i]);
        unr<CPL>(rk[i], ok && inc, u[i]);
        unr<CPL>(ra[i], ok && inc, pv[i]);
        unr<CPV>(rv[i], ok && inv, v);
        stc<CPV>(s.v + (t0 + i) * L::LV + cv, v);
      }
    } else {
      // rows t0 - 3 .. t0 + 7 of the three column blocks, then the convolutions
      uint32_t rq[11], rk[11], rv[11], tq[4], tk[4], tv[4], tq1[4], tk1[4], tv1[4];
#pragma unroll
      for (int i = 0; i < 11; ++i) {
        const bf16_t* xr = x + (long long)min(max(row0 + t0 + i - 3, first), row0 + n - 1) * a.ld;
        rq[i] = ldr<CPL>(xr + a.o_q + gq * a.dk + cs);
        rk[i] = ldr<CPL>(xr + a.o_k + gq * a.dk + cs);
        rv[i] = ldr<CPV>(xr + a.o_v + h * a.dv + vs);
      }
      const int chq = gq * a.dk + cs, chk = nqk + chq, chv = 2 * nqk + h * a.dv + vs;
      const bf16_t* cw = reinterpret_cast<const bf16_t*>(a.conv);
#pragma unroll
      for (int i = 0; i < 4; ++i) {  // tap i: the row i tokens back
        const int o = max(a.taps - 1 - i, 0);
        tq[i] = cw[chq * a.taps + o];
        tk[i] = cw[chk * a.taps + o];
        tv[i] = cw[chv * a.taps + o];
        if (CPL == 2) tq1[i] = cw[(chq + 1) * a.taps + o], tk1[i] = cw[(chk + 1) * a.taps + o];
        if (CPV == 2) tv1[i] = cw[(chv + 1) * a.taps + o];
      }
      float hq[3][CPL], hk[3][CPL], hv[3][CPV];  // the three rows before
      if (w == 0 && row0 == first) {             // ... which the sequence's slot keeps
        const int slot = a.slot[row0], C = 2 * nqk + a.H * a.dv;
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
          unr<CPL>(rq[i], true, hq[i]);
          unr<CPL>(rk[i], true, hk[i]);
          unr<CPV>(rv[i], true, hv[i]);
        }
      }
      auto conv = [&](auto cpl, const auto& hist, const uint32_t(&raw)[11], const uint32_t(&ta)[4], const uint32_t(&tb)[4], bool okc,
                      auto&& put) {
        constexpr int N = decltype(cpl)::value;
        float tp[4][N], p1[N], p2[N], p3[N];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          tp[i][0] = i < a.taps ? __uint_as_float(ta[i] << 16) : 0.f;
          if constexpr (N == 2) tp[i][1] = i < a.taps ? __uint_as_float(tb[i] << 16) : 0.f;
        }
#pragma unroll
        for (int e = 0; e < N; ++e) p3[e] = hist[0][e], p2[e] = hist[1][e], p1[e] = hist[2][e];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          float z[N], y[N];
          unr<N>(raw[i + 3], true, z);
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
      conv(std::integral_constant<int, CPL>{}, hq, rq, tq, tq1, inc, [&](int i, const float (&y)[CPL]) {
#pragma unroll
        for (int e = 0; e < CPL; ++e) q[i][e] = y[e];
      });
      conv(std::integral_constant<int, CPL>{}, hk, rk, tk, tk1, inc, [&](int i, const float (&y)[CPL]) {
#pragma unroll
        for (int e = 0; e < CPL; ++e) u[i][e] = y[e];
      });
      conv(std::integral_constant<int, CPV>{}, hv, rv, tv, tv1, inv,
           [&](int i, const float (&y)[CPV]) { stc<CPV>(s.v + (t0 + i) * L::LV + cv, y); });
    }
    float w0[CPL], ab[CPL], run[CPL];
    unr<CPL>(rw0, true, w0);
    if constexpr (KIND == 0) unr<CPL>(rab, true, ab);
    const float A = KIND == 1 ? __expf(__uint_as_float(rab << 16)) : 0.f;
#pragma unroll
    for (int e = 0; e < CPL; ++e) run[e] = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const bool ok = t0 + i < n;
      float lw[CPL], sk = 0.f, sq = 0.f;
      unr<CPL>(rw[i], true, lw);
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
        kn[i] = ok ? __builtin_amdgcn_rcpf(1.f + __expf(-__uint_as_float(rb[i] << 16))) : 0.f;
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
        if constexpr (KIND == 0) (half ? s.aqp : s.nb)[t * L::LA + j] = f2bf(ap[J][r]);
        if (!half && J == blk) s.nd[blk][4 * g4 + r][l15] = KIND == 0 ? ap[J][r] : -ak[J][r];
      }
  // ------------------------------------------------- inverses of the diagonal blocks: a lane per column
  wave_sync();
  if (!half && lane < 16) {
    float x[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      float v = r == lane ? 1.f : 0.f;
#pragma unroll
      for (int k = 0; k < r; ++k) v = fmaf(s.nd[blk][r][k], x[k], v);
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
    s16x4 vb[4], sb[4];
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
        y = mm16(row4((KIND == 0 ? s.nb : s.azk) + (16 * I + l15) * L::LA + 16 * J + 4 * g4), sb[J], y);
      X[I] = mm16f(*reinterpret_cast<const float4*>(&s.ti[I][l15][4 * g4]), y, f32x4{0.f, 0.f, 0.f, 0.f});
      sb[I] = KIND == 0 ? pk4(X[I]) : neg4(pk4(X[I]));
    }
    s16x4 xb[4];
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      if (KIND == 1 && !isw) X[I] = up4(vb[I]) - X[I];  // V - U
      xb[I] = pk4(X[I]);
    }
    if (isw) {
      const int cw = col + 4 * g4;  // this lane's four columns c'
      const int fo = ((col >> 5) * 64 + ((col >> 3 & 2) + (g4 >> 1)) * 16 + l15) * 8 + (g4 & 1) * 4;
#pragma unroll
      for (int I = 0; I < 4; ++I) {
        const int t = 16 * I + l15;
        f32x4 y = up4(row4(s.lq + t * L::LK + cw));
        const float4 f = *reinterpret_cast<const float4*>(&s.pre[I][cw]);
        y[0] *= f.x; y[1] *= f.y; y[2] *= f.z; y[3] *= f.w;
#pragma unroll
        for (int J = 0; J <= I; ++J)
          y = mm16(KIND == 0 ? xb[J] : neg4(xb[J]), row4((KIND == 0 ? s.aqp : s.aqk) + t * L::LA + 16 * J + 4 * g4), y);
        *reinterpret_cast<s16x4*>(gq + I * KS * 512 + fo) = pk4(y);
      }
#pragma unroll 4
      for (int c = 0; c < DK; c += 16) {
        f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int J = 0; J < 4; ++J) {
          const float f = s.et[J][c + l15];
          if (J) y *= f;
          y = mm16(KIND == 0 ? xb[J] : neg4(xb[J]), tok4<L::LK>(KIND == 0 ? s.rp : s.rk, 16 * J, c), y);
        }
        *reinterpret_cast<s16x4*>(gm + (c >> 4) * KS * 512 + fo) = pk4(y);
      }
    } else {
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
        *reinterpret_cast<s16x4*>(go + ((col >> 4) * 4 + I) * 256 + lane * 4) = pk4(y);
      }
#pragma unroll 4
      for (int c = 0; c < DK; c += 16) {
        f32x4 y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int J = 0; J < 4; ++J) {
          const float4 f = *reinterpret_cast<const float4*>(&s.et[J][c + 4 * g4]);
          if (J) y[0] *= f.x, y[1] *= f.y, y[2] *= f.z, y[3] *= f.w;
          if constexpr (KIND == 0) y = mm16(tok4<L::LK>(s.rp, 16 * J, c), xb[J], y);
          y = mm16(tok4<L::LK>(s.rk, 16 * J, c), KIND == 0 ? vb[J] : xb[J], y);
        }
        *reinterpret_cast<s16x4*>(gb + ((col >> 4) * (DK / 16) + (c >> 4)) * 256 + lane * 4) = pk4(y);
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
    float* op = a.o + ((long long)(row0 + i * CT + 16 * w + 4 * g4) * a.H + h) * a.dv + v;
    const long long os = (long long)a.H * a.dv;
    if (vt * 16 + 16 <= a.dv && i * CT + CT <= n) {
#pragma unroll
      for (int r = 0; r < 4; ++r) op[r * os] = o[r];
    } else if (v < a.dv) {
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (i * CT + 16 * w + 4 * g4 + r < n) op[r * os] = o[r];
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
