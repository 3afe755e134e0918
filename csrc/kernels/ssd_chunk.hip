// State-space mixers (delta_rule.h, KIND 3) over bf16 prompt portions, in chunks of 64 tokens on the matrix cores.
// With G_t the running log decays of a chunk and S_0 its first state,
//   o_t   = e^(G_t) S_0^T C_t + sum_(j <= t) (C_t . B_j) e^(G_t - G_j) dt_j x_j + D x_t
//   S_end = e^(G_end) S_0 + sum_j B_j (e^(G_end - G_j) dt_j x_j)^T
//
//   prep kernel   all chunks at once: C B^T and the transposed B of a group, decays and steps of its heads
//   run kernel    chunks of an entry in order, 16 NC value columns of a head per workgroup: the fp32 state stays in
//                 registers, its bf16 image is the operand of the read-out
// Every exponent is at most 0. What the heads of a group share stays in L2.
#include "chunk_ops.h"
#include "delta_rule.h"

namespace {
using namespace delta;

struct SsdArgs {
  DeltaArgs d;
  const int* ck;   // [nchunk][4]: first row, rows, first row of the entry, position of the chunk's first row
  const int* en;   // [nent][6]: first row, rows, position, slot, first chunk, chunks
  // operands as the run kernel's lanes read them; eight token slots e of lane group g hold the tokens
  // 32 k + 4 g + e (e < 4) and 32 k + 16 + 4 g + e - 4
  bf16_t* cb;      // [nchunk][G][4][2][64 lanes][8]: C_t . B_j, t = 16 I + (lane & 15), tokens j of step k
  bf16_t* bt;      // [nchunk][G][DK / 16][2][64 lanes][8]: B_j[c = 16 m + (lane & 15)]
  float* gd;       // [nchunk][H][2][64]: running log decays, steps
};

template <int DK>
__global__ void __launch_bounds__(512) ssd_prep_kernel(SsdArgs p) {
  constexpr int LK = DK + 8, KS = DK / 32, NK = DK / 64;
  __shared__ __attribute__((aligned(16))) bf16_t ic[CT * LK], ib[CT * LK];
  const DeltaArgs& a = p.d;
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l15 = lane & 15, g4 = lane >> 4, tok = tid >> 3, sub = tid & 7;
  const int ci = blockIdx.x, g = blockIdx.y, per = a.H / a.G, nqk = a.G * a.dk, C = 2 * nqk + a.H * a.dv;
  const long long row0 = p.ck[ci * 4];
  const int n = p.ck[ci * 4 + 1];
  const bf16_t* x = reinterpret_cast<const bf16_t*>(a.cx) + (row0 + min(tok, n - 1)) * C + g * a.dk;
#pragma unroll
  for (int i = 0; i < NK; ++i) {
    const int c = sub * 8 + 64 * i;
    const bool ok = tok < n && c < a.dk;
    u32x4 q = {0u, 0u, 0u, 0u}, k = {0u, 0u, 0u, 0u};
    if (ok) {
      q = *reinterpret_cast<const u32x4*>(x + c);
      k = *reinterpret_cast<const u32x4*>(x + nqk + c);
    }
    *reinterpret_cast<u32x4*>(ic + tok * LK + c) = q;
    *reinterpret_cast<u32x4*>(ib + tok * LK + c) = k;
  }
  // a lane a token: decays and steps of the group's heads
  const bf16_t* y = reinterpret_cast<const bf16_t*>(a.x) + (row0 + min(lane, n - 1)) * a.ld + a.o_w;
  for (int i = w; i < per; i += 8) {
    const int h = g * per + i;
    const float w0 = bf2f(reinterpret_cast<const bf16_t*>(a.w0)[h]), A = expf(bf2f(reinterpret_cast<const bf16_t*>(a.ab)[h]));
    const float dt = lane < n ? softplus(bf2f(y[h]) + w0) : 0.f;
    float G = -A * dt;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float u = __shfl_up(G, o, 64);
      if (lane >= o) G += u;
    }
    float* gd = p.gd + ((long long)ci * a.H + h) * 128;
    gd[lane] = G;
    gd[64 + lane] = dt;
  }
  __syncthreads();
  const long long cg = (long long)ci * a.G + g;
  // blocks (I, J <= I | 1) of B C^T: a lane's four rows are four tokens j at its column t
  for (int i = w; i < 12; i += 8) {
    const int I = i < 2 ? 0 : i < 4 ? 1 : i < 8 ? 2 : 3, J = i < 4 ? i & 1 : i & 3;
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      const int o = l15 * LK + 32 * k + 8 * g4;
      s = mm32(*reinterpret_cast<const bf16x8*>(ib + 16 * J * LK + o), *reinterpret_cast<const bf16x8*>(ic + 16 * I * LK + o), s);
    }
    *reinterpret_cast<s16x4*>(p.cb + ((cg * 4 + I) * 2 + (J >> 1)) * 512 + lane * 8 + 4 * (J & 1)) = pk4(s);
  }
  for (int i = w; i < DK / 8; i += 8) {
    const int m = i >> 1, k = i & 1;
    *reinterpret_cast<bf16x8*>(p.bt + ((cg * (DK / 16) + m) * 2 + k) * 512 + lane * 8) =
        two(tok4<LK>(ib, 32 * k, 16 * m), tok4<LK>(ib, 32 * k + 16, 16 * m));
  }
}

// A wave holds DK / 4 state rows (columns lane & 15 of each tile, rows 4 (lane >> 4) + r) and reads out 16 tokens.
template <int DK, int NC>
__global__ void __launch_bounds__(256) ssd_run_kernel(SsdArgs p) {
  constexpr int LS = DK + 8, LX = 16 * NC + 8, KS = DK / 32, MT = DK / 64;
  __shared__ __attribute__((aligned(16))) bf16_t img[2][NC * 16 * LS], xs[2][CT * LX], xd[2][CT * LX];
  __shared__ __attribute__((aligned(16))) float gs[2][2 * CT];
  const DeltaArgs& a = p.d;
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), l15 = lane & 15, g4 = lane >> 4;
  const int h = blockIdx.x % a.H, v0 = blockIdx.x / a.H * 16 * NC, g = h / (a.H / a.G);
  const int* en = p.en + blockIdx.y * 6;
  const int row0 = en[0], n = en[1], pos0 = en[2], slot = en[3], ch0 = en[4], nc = en[5];
  const int nqk = a.G * a.dk, C = 2 * nqk + a.H * a.dv, r0 = w * (DK / 4) + 4 * g4;
  const int tok = tid >> 2, c4 = (tid & 3) * 4;
  const bf16_t* cx = reinterpret_cast<const bf16_t*>(a.cx);
  const float skip = bf2f(reinterpret_cast<const bf16_t*>(a.skip)[h]);
  float* S = a.state + ((long long)slot * a.H + h) * a.dk * a.dv;
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
  struct Frag {
    bf16x8 c[KS], b[MT][2], cb[2];
    uint2 x[NC];
    float gt, dt, ge;
    float2 gl;  // (log decay, step) of token `lane`
  };
  auto load = [&](int i, Frag& f) {
    const long long cg = (long long)(ch0 + i) * a.G + g;
    const int left = n - i * CT;
    const bf16_t* cr = cx + (long long)(row0 + i * CT + min(16 * w + l15, left - 1)) * C + g * a.dk;
#pragma unroll
    for (int k = 0; k < KS; ++k) {
      u32x4 u = {0u, 0u, 0u, 0u};
      if (32 * k + 8 * g4 < a.dk) u = *reinterpret_cast<const u32x4*>(cr + 32 * k + 8 * g4);
      f.c[k] = __builtin_bit_cast(bf16x8, u);
    }
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int k = 0; k < 2; ++k)
        f.b[m][k] = *reinterpret_cast<const bf16x8*>(p.bt + ((cg * (DK / 16) + w * MT + m) * 2 + k) * 512 + lane * 8);
#pragma unroll
    for (int k = 0; k < 2; ++k)  // (k = 1 of the first two row blocks: not read below)
      f.cb[k] = *reinterpret_cast<const bf16x8*>(p.cb + ((cg * 4 + w) * 2 + (w >= 2 ? k : 0)) * 512 + lane * 8);
    const bf16_t* xr = cx + (long long)(row0 + i * CT + min(tok, left - 1)) * C + 2 * nqk + h * a.dv;
#pragma unroll
    for (int q = 0; q < NC; ++q) {
      const int v = v0 + 16 * q + c4;
      f.x[q] = make_uint2(0u, 0u);
      if (tok < left && v < a.dv) f.x[q] = *reinterpret_cast<const uint2*>(xr + v);
    }
    const float* gd = p.gd + ((long long)(ch0 + i) * a.H + h) * 128;
    f.gt = gd[tok];
    f.dt = gd[64 + tok];
    f.ge = gd[63];
    f.gl = make_float2(gd[lane], gd[64 + lane]);
  };
  auto chunk = [&](int i, const Frag& f) {
    const int bf = i & 1;
    bf16_t* im = img[bf];
#pragma unroll
    for (int q = 0; q < NC; ++q)
#pragma unroll
      for (int m = 0; m < MT; ++m) *reinterpret_cast<s16x4*>(im + (16 * q + l15) * LS + r0 + 16 * m) = pk4(st[q][m]);
    const float late = __expf(f.ge - f.gt) * f.dt, all = __expf(f.ge);
#pragma unroll
    for (int q = 0; q < NC; ++q) {
      const f32x4 v = up4(__builtin_bit_cast(s16x4, f.x[q]));
      *reinterpret_cast<uint2*>(xs[bf] + tok * LX + 16 * q + c4) = f.x[q];
      *reinterpret_cast<s16x4*>(xd[bf] + tok * LX + 16 * q + c4) = pk4(v * late);
    }
    if (w == 0) {
      gs[bf][lane] = f.gl.x;
      gs[bf][CT + lane] = f.gl.y;
    }
    __syncthreads();
    const float gt = gs[bf][16 * w + l15];
    f32x4 o[NC];
    const float4 go = *reinterpret_cast<const float4*>(&gs[bf][16 * w + 4 * g4]);
    const f32x4 eo = {__expf(go.x), __expf(go.y), __expf(go.z), __expf(go.w)};
#pragma unroll
    for (int q = 0; q < NC; ++q) {
      o[q] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < KS; ++k)
        o[q] = mm32(f.c[k], *reinterpret_cast<const bf16x8*>(im + (16 * q + l15) * LS + 32 * k + 8 * g4), o[q]);
      o[q] *= eo;
#pragma unroll
      for (int m = 0; m < MT; ++m) st[q][m] *= all;
    }
#pragma unroll
    for (int k = 0; k < 2; ++k) {
      bf16x8 xv[NC], xw[NC];
#pragma unroll
      for (int q = 0; q < NC; ++q) {
        xv[q] = two(tok4<LX>(xs[bf], 32 * k, 16 * q), tok4<LX>(xs[bf], 32 * k + 16, 16 * q));
        xw[q] = two(tok4<LX>(xd[bf], 32 * k, 16 * q), tok4<LX>(xd[bf], 32 * k + 16, 16 * q));
      }
      if (k == 0 || w >= 2) {
        const U16x8 cb = __builtin_bit_cast(U16x8, f.cb[k]);
        uint32_t u[4];
#pragma unroll
        for (int e = 0; e < 8; e += 4) {
          const int j = 32 * k + 4 * e + 4 * g4;  // (the second four slots: 16 tokens further)
          const float4 gj = *reinterpret_cast<const float4*>(&gs[bf][j]), dj = *reinterpret_cast<const float4*>(&gs[bf][CT + j]);
          const int t = 16 * w + l15;
          const float y0 = j <= t ? bf2f(cb.v[e]) * __expf(gt - gj.x) * dj.x : 0.f;
          const float y1 = j + 1 <= t ? bf2f(cb.v[e + 1]) * __expf(gt - gj.y) * dj.y : 0.f;
          const float y2 = j + 2 <= t ? bf2f(cb.v[e + 2]) * __expf(gt - gj.z) * dj.z : 0.f;
          const float y3 = j + 3 <= t ? bf2f(cb.v[e + 3]) * __expf(gt - gj.w) * dj.w : 0.f;
          u[e / 2] = pk2(y0, y1);
          u[e / 2 + 1] = pk2(y2, y3);
        }
        const bf16x8 am = __builtin_bit_cast(bf16x8, u32x4{u[0], u[1], u[2], u[3]});
#pragma unroll
        for (int q = 0; q < NC; ++q) o[q] = mm32(am, xv[q], o[q]);
      }
#pragma unroll
      for (int q = 0; q < NC; ++q)
#pragma unroll
        for (int m = 0; m < MT; ++m) st[q][m] = mm32(f.b[m][k], xw[q], st[q][m]);
    }
    bf16_t* op = reinterpret_cast<bf16_t*>(a.o) + ((long long)(row0 + i * CT + 16 * w + 4 * g4) * a.H + h) * a.dv;
    const long long os = (long long)a.H * a.dv;
#pragma unroll
    for (int q = 0; q < NC; ++q) {
      const int v = v0 + 16 * q + l15;
      const f32x4 xr = up4(tok4<LX>(xs[bf], 16 * w, 16 * q));  // this lane's tokens at its column
      if (v < a.dv)
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (i * CT + 16 * w + 4 * g4 + r < n) op[r * os + v] = f2bf(fmaf(skip, xr[r], o[q][r]));
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
  for (int q = 0; q < NC; ++q)
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int c = r0 + 16 * m + r, v = v0 + 16 * q + l15;
        if (c < a.dk && v < a.dv) S[(long long)c * a.dv + v] = st[q][m][r];
      }
}

template <int DK>
int run_go(const SsdArgs& p, int nent, hipStream_t s) {
  const int tiles = (p.d.dv + 15) / 16, wg = p.d.H * nent;
  // more columns a workgroup re-read the shared operands less; fewer leave more workgroups
#define GO(NC) hipLaunchKernelGGL((ssd_run_kernel<DK, NC>), dim3(p.d.H * ((tiles + NC - 1) / NC), nent), dim3(256), 0, s, p)
  if (tiles >= 4 && wg * (tiles / 4) >= 384) GO(4);
  else if (tiles >= 2 && wg * (tiles / 2) >= 256) GO(2);
  else GO(1);
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

bool ssd_ok(const SsdArgs& p) {
  const DeltaArgs& a = p.d;
  return delta_args_ok(a, 3) && a.dk % 8 == 0 && a.dv % 8 == 0 && a.dk <= 128 && a.cx && (uintptr_t)a.cx % 16 == 0 && a.o && p.ck &&
         p.en && p.cb && p.bt && p.gd;
}

}  // namespace

KCA_API int kca_ssd_chunk_abi() { return (int)sizeof(SsdArgs); }

// bf16, from convolution results (a.cx): p.cb, p.bt, p.gd of nchunk chunks, then a.o of nent entries; the slots'
// states advance. 10: sizes for the token-by-token kernels
KCA_API int kca_ssd_chunks(const SsdArgs* in, int nchunk, int nent, hipStream_t s) {
  const SsdArgs& p = *in;
  if (nchunk < 1 || nent < 1 || nent > 65535 || p.d.G > 65535) return 1;
  if (!ssd_ok(p)) return 10;
  if (p.d.dk <= 64) hipLaunchKernelGGL(ssd_prep_kernel<64>, dim3(nchunk, p.d.G), dim3(512), 0, s, p);
  else hipLaunchKernelGGL(ssd_prep_kernel<128>, dim3(nchunk, p.d.G), dim3(512), 0, s, p);
  if (hipGetLastError() != hipSuccess) return 4;
  return p.d.dk <= 64 ? run_go<64>(p, nent, s) : run_go<128>(p, nent, s);
}
