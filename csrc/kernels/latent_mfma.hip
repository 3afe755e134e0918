// Latent attention (latent_attn.h) in bf16 on the matrix cores:
//
//   head_mm kernel   y[b][h] = w[h] x[b][h] for few rows b: the absorbed queries W_uk^T q
//   rows kernel      one query token and 16 (32) heads per workgroup: a tile of 64 cached latents in LDS is both
//                    the keys (rows) and the values (columns, transposing reads); key splits -> partial softmaxes
//   merge kernel     merges the splits of 16 tokens of a head and applies W_uv
//   gather kernel    contexts out of their pages, contiguous
//   tile kernel      prompt portions over expanded keys and values: 128 queries of one head per workgroup
#include "attn_tile.h"
#include "lanes.h"
#include "latent_attn.h"

namespace {

__device__ __forceinline__ f32x4 mm32(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

// a wave: 16 outputs n of 16 rows b
__global__ void __launch_bounds__(256) head_mm_mfma_kernel(const bf16_t* x, long long ldx, int hx, const bf16_t* w, bf16_t* y,
                                                           long long ldy, int hy, int B, int N, int K, const int* row_of) {
  const int lane = threadIdx.x & 63, l15 = lane & 15, g4 = lane >> 4, h = blockIdx.y;
  const int b = blockIdx.x * 16 + l15, n0 = (blockIdx.z * 4 + (threadIdx.x >> 6)) * 16;
  if (n0 >= N) return;
  const int bb = min(b, B - 1);
  const bf16_t* xr = x + (row_of ? row_of[bb] : bb) * ldx + (long long)h * hx;
  const bf16_t* wr = w + ((long long)h * N + min(n0 + l15, N - 1)) * K;
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  const bf16x8 zero = {};
  for (int k0 = 0; k0 < K; k0 += 128) {
    bf16x8 fa[4], fb[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int k = k0 + 32 * i + 8 * g4;
      fa[i] = k < K ? *reinterpret_cast<const bf16x8*>(wr + k) : zero;
      fb[i] = k < K ? *reinterpret_cast<const bf16x8*>(xr + k) : zero;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) acc = mm32(fa[i], fb[i], acc);
  }
  if (b >= B) return;
  bf16_t* yr = y + b * ldy + (long long)h * hy + n0 + 4 * g4;
#pragma unroll
  for (int r = 0; r < 4; ++r)
    if (n0 + 4 * g4 + r < N) yr[r] = f2bf(acc[r]);
}

// NHG groups of 16 heads; NB 16-column tiles of the latent per wave; NPF 16-B chunks of a tile per thread.
// 2 NHG waves, a (32-key tile's half, head group) of the scores each; two workgroups share a CU.
template <int NHG, int NB, int NPF>
__global__ void __launch_bounds__(128 * NHG, NHG == 2 ? 2 : 1) latent_rows_mfma_kernel(LatentArgs a) {
  constexpr int HB = 16 * NHG, BK = 32, NW = 2 * NHG, NT = 64 * NW, LP = BK + 8;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int KL = a.C + a.R, KP = (KL + 31) / 32 * 32, LS = KP + 8;
  bf16_t* sq = reinterpret_cast<bf16_t*>(smem);          // [HB][LS]
  bf16_t* sk = sq + HB * LS;                             // [BK][LS]
  bf16_t* sp = sk + BK * LS;                             // [HB][LP] weights
  float* smax = reinterpret_cast<float*>(sp + HB * LP);  // [2][HB]
  float* sl = smax + 2 * HB;                             // [2][HB]
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, l15 = lane & 15, g4 = lane >> 4;
  const int b = blockIdx.x, h0 = blockIdx.y * HB, spl = blockIdx.z;
  const int row = a.row_of ? a.row_of[b] : b, pos = a.pos[row], kv = pos + 1;
  const int lo = spl * a.chunk, hi = min(kv, lo + a.chunk);
  if (lo >= kv) return;
  const int nh = min(HB, a.H - h0);
  const int* tbl = a.table + (long long)a.slot[row] * a.tstride;
  const int pmask = (1 << a.shift) - 1, CH = KL / 8, total = BK * CH;
  const bf16_t* kc = reinterpret_cast<const bf16_t*>(a.kc);

  // this thread's chunks of a tile: row in the tile, place in the row's image
  int tr[NPF], to[NPF];
#pragma unroll
  for (int i = 0; i < NPF; ++i) {
    const int c = min(tid + NT * i, total - 1);
    tr[i] = c / CH;
    to[i] = (c - tr[i] * CH) * 8;
  }
  auto load = [&](int k0, u32x4 (&st)[NPF]) {
#pragma unroll
    for (int i = 0; i < NPF; ++i) {
      const int key = min(k0 + tr[i], hi - 1);  // (past the end: a repeated row, whose weight is zero)
      st[i] = *reinterpret_cast<const u32x4*>(kc + (long long)tbl[key >> a.shift] * a.k_sp + (key & pmask) * KL + to[i]);
    }
  };
  auto store = [&](const u32x4 (&st)[NPF]) {
#pragma unroll
    for (int i = 0; i < NPF; ++i)
      if (tid + NT * i < total) *reinterpret_cast<u32x4*>(sk + tr[i] * LS + to[i]) = st[i];
  };
  u32x4 st[NPF];
  load(lo, st);
  {  // queries: absorbed part, rotated part, zero padding
    const bf16_t* qa = reinterpret_cast<const bf16_t*>(a.qa) + ((long long)b * a.H + h0) * a.C;
    const bf16_t* qr = reinterpret_cast<const bf16_t*>(a.q) + ((long long)row * a.H + h0) * (a.D + a.R) + a.D;
    const int cc = a.C / 8, rest = KP - a.C, pr = rest / 2;
    for (int i = tid; i < HB * cc; i += NT) {
      const int hh = i / cc, c = (i - hh * cc) * 8;
      u32x4 v = {0u, 0u, 0u, 0u};
      if (hh < nh) v = *reinterpret_cast<const u32x4*>(qa + (long long)hh * a.C + c);
      *reinterpret_cast<u32x4*>(sq + hh * LS + c) = v;
    }
    for (int i = tid; i < HB * pr; i += NT) {  // pairs
      const int hh = i / pr, c = (i - hh * pr) * 2;
      float x = 0.f, y = 0.f;
      if (hh < nh && c < a.R) {
        const uint32_t u = *reinterpret_cast<const uint32_t*>(qr + (long long)hh * (a.D + a.R) + c);
        x = __uint_as_float(u << 16);
        y = __uint_as_float(u & 0xffff0000u);
        if (c < a.nr) {
          float sn, cs;
          sincosf((float)pos * a.freq[c >> 1], &sn, &cs);
          const float z = x * cs - y * sn;
          y = y * cs + x * sn;
          x = z;
        }
      }
      *reinterpret_cast<uint32_t*>(sq + hh * LS + a.C + c) = pk_bf16(x, y);
    }
    const int pad = KP - KL;
    for (int i = tid; i < BK * pad; i += NT) sk[(i / pad) * LS + KL + i % pad] = 0;
  }
  const float sl2 = a.scale * kLog2e;
  const int kt = w & 1, hg = w >> 1;
  float m[NHG][4], l[4];
  f32x4 acc[NHG][NB];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    l[r] = 0.f;
#pragma unroll
    for (int g = 0; g < NHG; ++g) m[g][r] = -INFINITY;
  }
#pragma unroll
  for (int g = 0; g < NHG; ++g)
#pragma unroll
    for (int n = 0; n < NB; ++n) acc[g][n] = f32x4{0.f, 0.f, 0.f, 0.f};
  const bf16_t* qp = sq + (16 * hg + l15) * LS + 8 * g4;
  const bf16_t* kp = sk + (16 * kt + l15) * LS + 8 * g4;
  for (int k0 = lo; k0 < hi; k0 += BK) {
    __syncthreads();  // the tile before is read
    store(st);
    __syncthreads();
    load(min(k0 + BK, hi - 1), st);  // (past the end: not used)
    f32x4 s = {0.f, 0.f, 0.f, 0.f}, s2 = s;
    int k = 0;
    for (; k + 128 <= KP; k += 128) {
      bf16x8 fq[4], fk[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        fq[i] = *reinterpret_cast<const bf16x8*>(qp + k + 32 * i);
        fk[i] = *reinterpret_cast<const bf16x8*>(kp + k + 32 * i);
      }
      s = mm32(fq[0], fk[0], s);
      s2 = mm32(fq[1], fk[1], s2);
      s = mm32(fq[2], fk[2], s);
      s2 = mm32(fq[3], fk[3], s2);
    }
    for (; k < KP; k += 32) s = mm32(*reinterpret_cast<const bf16x8*>(qp + k), *reinterpret_cast<const bf16x8*>(kp + k), s);
    const bool in = k0 + 16 * kt + l15 < hi;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      s[r] = in ? (s[r] + s2[r]) * sl2 : -INFINITY;
      const float mx = lanes_reduce<16>(s[r], [](float x, float y) { return fmaxf(x, y); });
      if (l15 == 0) smax[kt * HB + 16 * hg + 4 * g4 + r] = mx;
    }
    __syncthreads();
    float al[NHG][4];
    bool same = true;
#pragma unroll
    for (int g = 0; g < NHG; ++g)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float* q = smax + 16 * g + 4 * g4 + r;
        const float mn = fmaxf(fmaxf(q[0], q[HB]), m[g][r]);
        same = same && mn == m[g][r];
        al[g][r] = __builtin_amdgcn_exp2f(m[g][r] - mn);
        m[g][r] = mn;
      }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float mn = NHG == 1 || hg == 0 ? m[0][r] : m[NHG - 1][r];
      const float am = NHG == 1 || hg == 0 ? al[0][r] : al[NHG - 1][r];
      const float e = __builtin_amdgcn_exp2f(s[r] - mn);
      l[r] = fmaf(l[r], am, e);
      sp[(16 * hg + 4 * g4 + r) * LP + 16 * kt + l15] = f2bf(e);
    }
    if (!__all(same))
#pragma unroll
      for (int g = 0; g < NHG; ++g)
#pragma unroll
        for (int n = 0; n < NB; ++n)
#pragma unroll
          for (int r = 0; r < 4; ++r) acc[g][n][r] *= al[g][r];
    __syncthreads();
    bf16x8 pf[NHG];
#pragma unroll
    for (int g = 0; g < NHG; ++g) pf[g] = *reinterpret_cast<const bf16x8*>(sp + (16 * g + l15) * LP + 8 * g4);
#pragma unroll
    for (int n = 0; n < NB; ++n) {
      const int c = (w + NW * n) * 16;
      if (c >= a.C) continue;
      const bf16_t* p0 = sk + (8 * g4 + (l15 >> 2)) * LS + c + 4 * (l15 & 3);
      const bf16x8 vf = cat8(lds_tr4(reinterpret_cast<const char*>(p0), 0), lds_tr4(reinterpret_cast<const char*>(p0 + 4 * LS), 0));
#pragma unroll
      for (int g = 0; g < NHG; ++g) acc[g][n] = mm32(pf[g], vf, acc[g][n]);
    }
  }
  // sums of the two key halves
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const float t = lanes_reduce<16>(l[r], [](float x, float y) { return x + y; });
    if (l15 == 0) sl[kt * HB + 16 * hg + 4 * g4 + r] = t;
  }
  __syncthreads();
  const int stp = a.C + 4;
#pragma unroll
  for (int g = 0; g < NHG; ++g)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int hh = 16 * g + 4 * g4 + r;
      if (hh >= nh) continue;
      float* part = a.part + (((long long)b * a.H + h0 + hh) * a.nsplit + spl) * stp;
      if (w == 0 && l15 == 0) {
        part[0] = m[g][r] * kLn2;
        part[1] = sl[hh] + sl[HB + hh];
      }
#pragma unroll
      for (int n = 0; n < NB; ++n) {
        const int c = (w + NW * n) * 16 + l15;
        if (c < a.C) part[4 + c] = acc[g][n][r];
      }
    }
}

constexpr int MSPL = 256;  // splits the merge kernel takes

// MR tokens of a head (a row of the products is a token; rows past MR are zero); 8 waves
template <int MR>
__global__ void __launch_bounds__(512) latent_merge_mfma_kernel(LatentArgs a, int rows) {
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int CP = (a.C + 31) / 32 * 32, LS = CP + 8;
  bf16_t* ob = reinterpret_cast<bf16_t*>(smem);            // [16][LS]
  float* wz = reinterpret_cast<float*>(ob + 16 * LS);      // [MR][nsplit]
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, l15 = lane & 15, g4 = lane >> 4;
  const int h = blockIdx.y, b0 = blockIdx.x * MR, nb = min(MR, rows - b0), st = a.C + 4;
  const float sink = bf2f(reinterpret_cast<const bf16_t*>(a.sink)[h]);
  const bf16x8 zero = {};
  // W_uv fragments of this wave's first 16 outputs
  bf16x8 fw[4];
  const bf16_t* wr = reinterpret_cast<const bf16_t*>(a.wuv) + ((long long)h * a.E + min(w * 16 + l15, a.E - 1)) * a.C;
#pragma unroll
  for (int i = 0; i < 4; ++i) fw[i] = 32 * i + 8 * g4 < a.C ? *reinterpret_cast<const bf16x8*>(wr + 32 * i + 8 * g4) : zero;
  for (int i = w; i < nb; i += 8) {
    const int row = a.row_of ? a.row_of[b0 + i] : b0 + i, used = (a.pos[row] + a.chunk) / a.chunk;
    const float* part = a.part + ((long long)(b0 + i) * a.H + h) * a.nsplit * st;
    float M = sink, L = 0.f;
    for (int z = lane; z < used; z += 64) M = fmaxf(M, part[(long long)z * st]);
    M = wave_max(M);
    for (int z = lane; z < used; z += 64) L += part[(long long)z * st + 1] * __expf(part[(long long)z * st] - M);
    L = 1.f / (wave_sum(L) + __expf(sink - M));
    for (int z = lane; z < used; z += 64) wz[i * a.nsplit + z] = __expf(part[(long long)z * st] - M) * L;
  }
  __syncthreads();
  // four columns a thread, eight splits' loads in flight
  const int cq = CP / 4;
  for (int u = tid; u < 16 * cq; u += 512) {
    const int i = u / cq, c = (u - i * cq) * 4;
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if (i < nb && c < a.C) {
      const int row = a.row_of ? a.row_of[b0 + i] : b0 + i, used = (a.pos[row] + a.chunk) / a.chunk;
      const float* part = a.part + ((long long)(b0 + i) * a.H + h) * a.nsplit * st + 4 + c;
      for (int z0 = 0; z0 < used; z0 += 8) {
        float4 x[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) x[j] = *reinterpret_cast<const float4*>(part + (long long)min(z0 + j, used - 1) * st);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
          const float f = z0 + j < used ? wz[i * a.nsplit + z0 + j] : 0.f;
          v.x = fmaf(f, x[j].x, v.x);
          v.y = fmaf(f, x[j].y, v.y);
          v.z = fmaf(f, x[j].z, v.z);
          v.w = fmaf(f, x[j].w, v.w);
        }
      }
    }
    *reinterpret_cast<uint2*>(ob + i * LS + c) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
  }
  __syncthreads();
  const int b = b0 + l15;
  const bool live = l15 < nb;
  const int row = live ? (a.row_of ? a.row_of[b] : b) : 0;
  bf16_t* out = reinterpret_cast<bf16_t*>(a.out) + row * a.ldo + (long long)h * a.E;
  for (int e0 = w * 16; e0 < a.E; e0 += 128) {
    const bf16_t* wp = reinterpret_cast<const bf16_t*>(a.wuv) + ((long long)h * a.E + min(e0 + l15, a.E - 1)) * a.C;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < CP; k0 += 128) {
      bf16x8 fa[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int k = k0 + 32 * i + 8 * g4;
        fa[i] = k0 == 0 && e0 == w * 16 ? fw[i] : k < a.C ? *reinterpret_cast<const bf16x8*>(wp + k) : zero;
      }
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (k0 + 32 * i < CP) acc = mm32(fa[i], *reinterpret_cast<const bf16x8*>(ob + l15 * LS + k0 + 32 * i + 8 * g4), acc);
    }
    if (live)
#pragma unroll
      for (int r = 0; r < 4; ++r)
        if (e0 + 4 * g4 + r < a.E) out[e0 + 4 * g4 + r] = f2bf(acc[r]);
  }
}

// context rows [first row, length, slot] out of their pages
__global__ void __launch_bounds__(256) latent_gather_kernel(const bf16_t* kc, long long k_sp, const int* table, int tstride,
                                                            int shift, int KL, const int* ctx, bf16_t* out) {
  const int r0 = ctx[blockIdx.y * 3], n = ctx[blockIdx.y * 3 + 1], slot = ctx[blockIdx.y * 3 + 2], CH = KL / 8;
  const int* tbl = table + (long long)slot * tstride;
  for (long long i = (long long)blockIdx.x * 256 + threadIdx.x; i < (long long)n * CH; i += (long long)gridDim.x * 256) {
    const int t = (int)(i / CH), c = (int)(i - (long long)t * CH) * 8;
    *reinterpret_cast<u32x4*>(out + (long long)(r0 + t) * KL + c) = *reinterpret_cast<const u32x4*>(
        kc + (long long)tbl[t >> shift] * k_sp + (long long)(t & ((1 << shift) - 1)) * KL + c);
  }
}

// 4 waves of 32 queries; 32-key tiles of K | V double buffered in LDS (the image of attn_tile.h); S^T = K Q^T
// leaves a query per lane, and P^T feeds O^T += V^T P^T from registers.
template <int DK, int DV>
__global__ void __launch_bounds__(256, DV > 128 ? 1 : 2) latent_tile_kernel(LatentArgs p, int ntiles) {
  constexpr int BN = 32, TK = BN * DK * 2, TV = BN * DV * 2, BUF = TK + TV;
  constexpr int KS = DK / 16, NB = DV / 32;
  constexpr int CK = BN * (DK / 8), CV = BN * (DV / 8), NC = CK + CV, CPT = (NC + 255) / 256;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int tid = threadIdx.x, lane = tid & 63, qg = tid >> 6;
  const int l32 = lane & 31, hh = lane >> 5, gi = lane & 15;
  const int lid = xcd_remap(blockIdx.x, gridDim.x);
  const int h = lid / ntiles, ti = lid - h * ntiles;  // a head's tiles share its keys in one L2
  const int* tl = p.tiles + ti * 4;
  const int row0 = tl[0], nrow = tl[1], pos0 = tl[2], ctx0 = tl[3];
  const int qi = qg * 32 + l32;
  const bool live = qi < nrow;
  const int row = row0 + min(qi, nrow - 1), pos = pos0 + min(qi, nrow - 1);
  const int kv_hi = pos0 + nrow, nkt = (kv_hi + BN - 1) / BN;
  const int wave_hi = pos0 + min(qg * 32 + 32, nrow);
  const bool busy = qg * 32 < nrow;
  const int D = p.D, R = p.R, E = p.E, KL = p.C + p.R;
  const bf16_t* kg = reinterpret_cast<const bf16_t*>(p.kv) + ctx0 * p.ldkv + h * D;
  const bf16_t* vg = reinterpret_cast<const bf16_t*>(p.kv) + ctx0 * p.ldkv + p.H * D + h * E;
  const bf16_t* rg = reinterpret_cast<const bf16_t*>(p.kr) + (long long)ctx0 * KL + p.C;

  bf16x8 qf[KS];
  {
    const bf16_t* q = reinterpret_cast<const bf16_t*>(p.q) + ((long long)row * p.H + h) * (D + R);
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int c = 16 * s + 8 * hh;
      u32x4 v = {0u, 0u, 0u, 0u};
      if (c < D + R) v = *reinterpret_cast<const u32x4*>(q + c);
      if (c >= D && c < D + R) {
        const int i0 = c - D;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int i = i0 + 2 * j;
          if (i < p.nr) {
            float sn, cs;
            sincosf((float)pos * p.freq[i >> 1], &sn, &cs);
            const float x = __uint_as_float(v[j] << 16), y = __uint_as_float(v[j] & 0xffff0000u);
            v[j] = pk_bf16(x * cs - y * sn, y * cs + x * sn);
          }
        }
      }
      qf[s] = __builtin_bit_cast(bf16x8, v);
    }
  }
  const float sl2 = p.scale * kLog2e;

  auto load = [&](int k0, u32x4 (&st)[CPT]) {
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int c = tid + 256 * i;
      st[i] = u32x4{0u, 0u, 0u, 0u};
      if (c < CK) {
        const int r = c / (DK / 8), e = (c % (DK / 8)) * 8, key = k0 + r;
        if (key < kv_hi) {
          if (e < D) st[i] = *reinterpret_cast<const u32x4*>(kg + key * p.ldkv + e);
          else if (e < D + R) st[i] = *reinterpret_cast<const u32x4*>(rg + (long long)key * KL + e - D);
        }
      } else if (c < NC) {
        const int cv = c - CK, r = cv / (DV / 8), e = (cv % (DV / 8)) * 8, key = k0 + r;
        if (key < kv_hi && e < E) st[i] = *reinterpret_cast<const u32x4*>(vg + key * p.ldkv + e);
      }
    }
  };
  auto store = [&](const u32x4 (&st)[CPT], char* buf) {
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int c = tid + 256 * i;
      if (c < CK) *reinterpret_cast<u32x4*>(buf + img_off<DK>(c / (DK / 8), c % (DK / 8))) = st[i];
      else if (c < NC) *reinterpret_cast<u32x4*>(buf + TK + img_off<DV>((c - CK) / (DV / 8), (c - CK) % (DV / 8))) = st[i];
    }
  };

  const int xr = (l32 >> 2) & 3;
  const int kb_e = (l32 >> 3) * 16 * DK + 64 * (l32 & 7) + 16 * (hh ^ xr);
  const int kb_o = (l32 >> 3) * 16 * DK + 64 * (l32 & 7) + 16 * ((2 + hh) ^ xr);
  const int c3 = 2 * ((lane >> 4) & 1) + ((gi & 3) >> 1);
  const int vb_1 = TK + 64 * (4 * hh + (gi >> 2)) + 16 * (c3 ^ hh) + 8 * (gi & 1);
  const int vb_2 = TK + 16 * DV + 64 * (4 * hh + (gi >> 2)) + 16 * (c3 ^ hh ^ 2) + 8 * (gi & 1);

  f32x16 o[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[b][r] = 0.f;
  float mref = -INFINITY, ls = 0.f;

  u32x4 st[CPT];
  load(0, st);
  store(st, smem);
  __syncthreads();
  for (int t = 0; t < nkt; ++t) {
    const char* buf = smem + (t & 1) * BUF;
    const int k0 = t * BN;
    const bool more = t + 1 < nkt;
    if (more) load(k0 + BN, st);
    if (busy && k0 < wave_hi) {  // (tiles past the wave's last query: staging only)
      f32x16 s;
#pragma unroll
      for (int r = 0; r < 16; ++r) s[r] = 0.f;
      bf16x8 fk[3];  // K fragments two steps ahead of their products
      fk[0] = lds_b128(buf, kb_e);
      fk[1] = lds_b128(buf, kb_o);
      __builtin_amdgcn_sched_group_barrier(0x100, 2, 0);
#pragma unroll
      for (int k = 0; k < KS; ++k) {
        if (k + 2 < KS) {
          fk[(k + 2) % 3] = lds_b128(buf, ((k & 1) ? kb_o : kb_e) + 512 * ((k + 2) >> 1));
          __builtin_amdgcn_sched_group_barrier(0x100, 1, 0);
        }
        s = __builtin_amdgcn_mfma_f32_32x32x16_bf16(fk[k % 3], qf[k], s, 0, 0, 0);
        __builtin_amdgcn_sched_group_barrier(0x8, 1, 0);
      }
      // s[r]: key k0 + (r & 3) + 8 (r >> 2) + 4 hh of this lane's query
      if (k0 + BN > pos0 + qg * 32) {
        const int lim = pos - k0 - 4 * hh;
#pragma unroll
        for (int r = 0; r < 16; ++r)
          if ((r & 3) + 8 * (r >> 2) > lim) s[r] = -INFINITY;
      }
      float mt = s[0];
#pragma unroll
      for (int r = 1; r < 16; ++r) mt = fmaxf(mt, s[r]);
      mt = fmaxf(mt, __shfl_xor(mt, 32, 64)) * sl2;
      // the reference maximum follows only when a tile exceeds it by more than 2^8
      if (__any(mt > mref + kRescaleThr)) {
        const float mn = fmaxf(mref, mt);
        const float al = mref == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(mref - mn);
        ls *= al;
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
          for (int r = 0; r < 16; ++r) o[b][r] *= al;
        mref = mn;
      }
      float sum = 0.f;
      uint32_t u[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float w0 = __builtin_amdgcn_exp2f(fmaf(s[2 * i], sl2, -mref));
        const float w1 = __builtin_amdgcn_exp2f(fmaf(s[2 * i + 1], sl2, -mref));
        sum += w0 + w1;
        u[i] = pk_bf16(w0, w1);
      }
      ls += sum;
      const bf16x8 p0 = __builtin_bit_cast(bf16x8, u32x4{u[0], u[1], u[2], u[3]});
      const bf16x8 p1 = __builtin_bit_cast(bf16x8, u32x4{u[4], u[5], u[6], u[7]});
      auto vfrag = [&](int b, int h2) {
        return cat8(lds_tr4(buf, vb_1 + 32 * DV * h2 + 512 * b), lds_tr4(buf, vb_2 + 32 * DV * h2 + 512 * b));
      };
      bf16x8 v0[2], v1[2];  // V fragments one block ahead
      v0[0] = vfrag(0, 0);
      v1[0] = vfrag(0, 1);
      __builtin_amdgcn_sched_group_barrier(0x100, 4, 0);
#pragma unroll
      for (int b = 0; b < NB; ++b) {
        if (b + 1 < NB) {
          v0[(b + 1) & 1] = vfrag(b + 1, 0);
          v1[(b + 1) & 1] = vfrag(b + 1, 1);
          __builtin_amdgcn_sched_group_barrier(0x100, 4, 0);
        }
        o[b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v0[b & 1], p0, o[b], 0, 0, 0);
        o[b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(v1[b & 1], p1, o[b], 0, 0, 0);
        __builtin_amdgcn_sched_group_barrier(0x8, 2, 0);
      }
    }
    if (more) store(st, smem + ((t + 1) & 1) * BUF);
    __syncthreads();
  }
  if (!live) return;
  const float sink = bf2f(reinterpret_cast<const bf16_t*>(p.sink)[h]) * kLog2e;
  const float n = 1.f / (ls + __shfl_xor(ls, 32, 64) + __builtin_amdgcn_exp2f(sink - mref));
  bf16_t* orow = reinterpret_cast<bf16_t*>(p.out) + row * p.ldo + (long long)h * E;
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int q4 = 0; q4 < 4; ++q4) {
      const int c = 32 * b + 8 * q4 + 4 * hh;
      if (c < E)
        *reinterpret_cast<uint2*>(orow + c) = make_uint2(pk_bf16(o[b][4 * q4] * n, o[b][4 * q4 + 1] * n),
                                                         pk_bf16(o[b][4 * q4 + 2] * n, o[b][4 * q4 + 3] * n));
    }
}

template <int NHG, int NB, int NPF>
int rows_go(const LatentArgs& a, int rows, hipStream_t s) {
  const int KP = (a.C + a.R + 31) / 32 * 32, HB = 16 * NHG;
  const size_t lds = (size_t)(HB + 32) * (KP + 8) * 2 + (size_t)HB * 40 * 2 + (size_t)4 * HB * 4;
  if (lds > 160 * 1024 || 32 * ((a.C + a.R) / 8) > 128 * NHG * NPF || a.C > 32 * NHG * NB) return 10;
  auto kern = latent_rows_mfma_kernel<NHG, NB, NPF>;
  if (hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return 5;
  hipLaunchKernelGGL(kern, dim3(rows, (a.H + HB - 1) / HB, a.nsplit), dim3(128 * NHG), lds, s, a);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
int rows_heads(const LatentArgs& a, int rows, hipStream_t s) {
  const int KL = a.C + a.R;
  if (a.H > 16) {
    if (a.C <= 128 && KL <= 256) return rows_go<2, 2, 4>(a, rows, s);
    if (a.C <= 256 && KL <= 384) return rows_go<2, 4, 6>(a, rows, s);
    return rows_go<2, 8, 9>(a, rows, s);
  }
  if (a.C <= 128 && KL <= 256) return rows_go<1, 4, 8>(a, rows, s);
  if (a.C <= 256 && KL <= 384) return rows_go<1, 8, 12>(a, rows, s);
  return rows_go<1, 16, 18>(a, rows, s);
}

template <int DK, int DV>
int tile_go(const LatentArgs& p, int ntiles, hipStream_t s) {
  constexpr int lds = 2 * 32 * (DK + DV) * 2;
  auto kern = latent_tile_kernel<DK, DV>;
  if (lds > 48 * 1024)
    if (hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess) return 5;
  hipLaunchKernelGGL(kern, dim3(ntiles * p.H), dim3(256), lds, s, p, ntiles);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
template <int DK>
int tile_dv(const LatentArgs& p, int ntiles, hipStream_t s) {
  if (p.E <= 64) return tile_go<DK, 64>(p, ntiles, s);
  if (p.E <= 128) return tile_go<DK, 128>(p, ntiles, s);
  return tile_go<DK, 256>(p, ntiles, s);
}

bool al16(const void* p) { return (uintptr_t)p % 16 == 0; }

}  // namespace

// bf16 forms of kca_head_mm, kca_latent_rows, kca_latent_merge; 10: sizes for those
KCA_API int kca_head_mm_mfma(const void* x, long long ldx, int hx, const void* w, void* y, long long ldy, int hy, int B, int H,
                             int N, int K, const void* row_of, hipStream_t s) {
  if (!x || !w || !y || B < 1 || H < 1 || H > 65535 || N < 1 || K < 1) return 1;
  if (K % 8 || ldx % 8 || hx % 8 || !al16(x) || !al16(w)) return 10;
  hipLaunchKernelGGL(head_mm_mfma_kernel, dim3((B + 15) / 16, H, (N + 63) / 64), dim3(256), 0, s, (const bf16_t*)x, ldx, hx,
                     (const bf16_t*)w, (bf16_t*)y, ldy, hy, B, N, K, (const int*)row_of);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

KCA_API int kca_latent_rows_mfma(const LatentArgs* in, int rows, int max_kv, hipStream_t s) {
  const LatentArgs& a = *in;
  if (!latent_args_ok(a) || rows < 1 || !a.q || !a.qa || !a.part || a.nsplit < 1 || a.nsplit > 65535 || a.chunk < 1) return 1;
  if ((long long)a.nsplit * a.chunk < max_kv) return 2;
  if (a.C % 8 || a.R % 8 || a.k_sp % 8 || !al16(a.kc) || !al16(a.qa)) return 10;
  return rows_heads(a, rows, s);
}

KCA_API int kca_latent_merge_mfma(const LatentArgs* in, int rows, hipStream_t s) {
  const LatentArgs& a = *in;
  if (!latent_args_ok(a) || rows < 1 || !a.part || !a.out || !a.wuv || !a.sink || a.chunk < 1 || a.H > 65535) return 1;
  if (a.C % 8 || !al16(a.wuv) || a.nsplit > MSPL || a.C > 1024) return 10;
  // few tokens: a workgroup each, so that the partials stream on more of them
  const int mr = rows <= 32 ? 4 : 16;
  const size_t lds = (size_t)16 * ((a.C + 31) / 32 * 32 + 8) * 2 + (size_t)mr * a.nsplit * 4;
  const dim3 g((rows + mr - 1) / mr, a.H);
  if (mr == 4) hipLaunchKernelGGL(latent_merge_mfma_kernel<4>, g, dim3(512), lds, s, a, rows);
  else hipLaunchKernelGGL(latent_merge_mfma_kernel<16>, g, dim3(512), lds, s, a, rows);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

// bf16. Cached rows of nctx contexts (ctx [nctx][3]: first output row, length, slot), max_len rows at most each
KCA_API int kca_latent_gather(const void* kc, long long k_sp, const void* table, int tstride, int shift, int KL,
                              const void* ctx, int nctx, int max_len, void* out, hipStream_t s) {
  if (!kc || !table || !ctx || !out || nctx < 1 || nctx > 65535 || max_len < 1 || KL < 8 || KL % 8 || k_sp % 8 || shift < 4 ||
      !al16(kc) || !al16(out))
    return 1;
  hipLaunchKernelGGL(latent_gather_kernel, dim3(kca_grid((long long)max_len * (KL / 8), 256), nctx), dim3(256), 0, s,
                     (const bf16_t*)kc, k_sp, (const int*)table, tstride, shift, KL, (const int*)ctx, (bf16_t*)out);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

KCA_API int kca_latent_tiles(const LatentArgs* in, int ntiles, hipStream_t s) {
  const LatentArgs& p = *in;
  if (!latent_args_ok(p) || ntiles < 1 || (long long)ntiles * p.H > 0x7fffffff || !p.q || !p.kv || !p.kr || !p.tiles || !p.out ||
      !p.sink)
    return 1;
  if (p.D % 8 || p.R % 8 || p.E % 8 || p.C % 8 || p.D + p.R > 256 || p.E > 256 || p.ldkv % 8 || !al16(p.q) || !al16(p.kv) ||
      !al16(p.kr) || p.ldo % 4 || (uintptr_t)p.out % 8 || !(p.scale > 0.f))
    return 10;
  const int dk = p.D + p.R;
  if (dk <= 64) return tile_dv<64>(p, ntiles, s);
  if (dk <= 128) return tile_dv<128>(p, ntiles, s);
  if (dk <= 192) return tile_dv<192>(p, ntiles, s);
  return tile_dv<256>(p, ntiles, s);
}
