// Differential attention over the paged cache: every head runs two softmax maps over the same values,
// and the difference of the two outputs is normalised per head:
//   a_i = softmax_j(q_i . k_i,j * f) V  (i = 1, 2),  f = scale * (1 + coef ln(floor((pos + 1) / every) + 1))
//   o = a_1 - lambda a_2;  o <- o / sqrt(mean(o^2) + eps) * gain
// K pages are [2G][PS][dim] (key head 2g + i is map i of group g), V pages [G][PS][vdim]; q / k / v rows
// come from one projection buffer [q: H x 2 x dim | k: G x 2 x dim | v: G x vdim]. Scores, weights and
// the normalisation are fp32.
//
//   kv_append_kernel   K / V of new tokens into their pages
//   rows kernel        one query token per row, any dims, fp32 or bf16 (vector units): decode (split over
//                      keys, the last arriving split merges; the new token's K / V is appended here) and
//                      every shape or type the matrix-core kernel does not take
//   tile kernel        bf16 prompt portions on the matrix cores: 128 queries of one (entry, head) per
//                      workgroup, one wave per (32 queries, map)
#include "attn_rows.h"
#include "attn_tile.h"
#include "decode_tail.h"
#include "lanes.h"

namespace {

struct DiffArgs {
  const void* qkv;          // rows of the projection, row stride ld
  long long ld;
  void* kc;                 // [pages][2G][PS][dim]
  void* vc;                 // [pages][G][PS][vdim]
  long long k_sp, v_sp;     // page strides (elements)
  const int* table;         // [slots][tstride] page of each block
  int tstride, shift;
  const int* pos;           // [rows] position of the row's token
  const int* slot;          // [rows]
  void* out;                // [rows][H * vdim], row stride ldo
  long long ldo;
  int H, G, dim, vdim;
  float scale, coef;
  double every;             // <= 0: no temperature
  float lambda, eps, gain;
  int append;               // rows kernel: key `pos` comes from the row's own k / v, which it also stores
  int nsplit, chunk;        // rows kernel: keys per split
  float* ws;                // split partials
  unsigned* cnt;            // [rows * G * subgroups] arrival counters (zero, re-armed)
  const int* tiles;         // tile kernel: [ntiles][4] first row, rows, position of first row, slot
  const int* row_of;        // rows kernel: row index of block b (nullable: b)
};

__device__ __forceinline__ float row_scale(const DiffArgs& p, int pos) {
  if (!(p.every > 0)) return p.scale;
  return p.scale * (1.f + p.coef * logf((float)floor((double)(pos + 1) / p.every) + 1.f));
}

// V elements per access (V > 1: head sizes, rows and pools are multiples of V)
template <typename E, int V>
__global__ void __launch_bounds__(256) kv_append_kernel(DiffArgs p, int T) {
  struct alignas(sizeof(E) * V) Pack { E v[V]; };
  const int nk = 2 * p.G * p.dim, n = nk + p.G * p.vdim, per = n / V;
  for (long long i = (long long)blockIdx.x * 256 + threadIdx.x; i < (long long)T * per; i += (long long)gridDim.x * 256) {
    const int t = (int)(i / per), e = (int)(i - (long long)t * per) * V;
    const int ps = p.pos[t], in_page = ps & ((1 << p.shift) - 1);
    const long long pg = p.table[(long long)p.slot[t] * p.tstride + (ps >> p.shift)];
    const bool key = e < nk;
    const int j = key ? e : e - nk, sz = key ? p.dim : p.vdim, hd = j / sz, c = j - hd * sz;
    E* dst = key ? reinterpret_cast<E*>(p.kc) + pg * p.k_sp : reinterpret_cast<E*>(p.vc) + pg * p.v_sp;
    *reinterpret_cast<Pack*>(dst + (((long long)hd << p.shift) + in_page) * sz + c) =
        *reinterpret_cast<const Pack*>(reinterpret_cast<const E*>(p.qkv) + t * p.ld + 2 * p.H * p.dim + e);
  }
}

// ---------------------------------------------------------------------------------------- rows kernel
// Workgroup: (row, kv group g, RB query heads of the group, key split), 4 waves. Each wave walks its own
// KT-key tiles of the split with its own online softmax: LPK lanes share a key's dot products, LPV lanes
// a value row; a wave-private LDS array carries the 2 x RB x KT weights between the two layouts. The
// waves, then the splits, merge at the end.

constexpr int MAX_SPLITS = 256;

template <typename E, int RB, int LPK, int LPV, bool VEC>
__global__ void __launch_bounds__(256) diff_rows_kernel(DiffArgs p) {
  constexpr int KT = LPV >= 64 ? 4 : (LPV >= 32 ? 8 : 16);            // keys per tile of a wave
  constexpr int KPK = 64 / LPK, NPK = KT / KPK > 0 ? KT / KPK : 1;   // keys per pass, passes (scores)
  constexpr int KPV = 64 / LPV, NPV = KT / KPV > 0 ? KT / KPV : 1;   // (values)
  static_assert(KPK <= KT && KPV <= KT, "a pass covers at most one tile");
  constexpr int NS = 2 * RB;                                         // score rows: [map][head]
  constexpr int NP = NS * KT, PPL = (NP + 63) / 64;                  // (score row, key) pairs, pairs per lane
  __shared__ __attribute__((aligned(16))) float sc[4][KT][NS], als[4][NS];
  __shared__ float wm[4][NS], wl[4][NS];
  __shared__ int s_last;
  extern __shared__ __attribute__((aligned(16))) float merged[];     // [4][NS][vdim] then reused
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int D = p.dim, Vd = p.vdim, Hg = p.H / p.G;
  const int nsub = (Hg + RB - 1) / RB;
  const int row = p.row_of ? p.row_of[blockIdx.x] : (int)blockIdx.x;
  const int g = blockIdx.y / nsub, sub = blockIdx.y % nsub, sp = blockIdx.z;
  const int h0 = g * Hg + sub * RB, nh = min(RB, Hg - sub * RB);
  const int pos = p.pos[row], slot = p.slot[row], kv = pos + 1;
  const int lo = sp * p.chunk, hi = min(kv, lo + p.chunk);
  const int used = (kv + p.chunk - 1) / p.chunk;                     // splits that hold keys
  if (sp >= used) return;
  const int* tbl = p.table + (long long)slot * p.tstride;
  const int pmask = (1 << p.shift) - 1;
  const E* qr = reinterpret_cast<const E*>(p.qkv) + row * p.ld;
  const E* kn = qr + 2 * p.H * D + 2 * g * D;                        // the row's own keys (map 1, map 2)
  const E* vn = qr + 2 * p.H * D + 2 * p.G * D + g * Vd;
  E* kc = reinterpret_cast<E*>(p.kc);
  E* vc = reinterpret_cast<E*>(p.vc);

  const int lk = lane % LPK, jk = lane / LPK, lv = lane % LPV, jv = lane / LPV;
  const float f = row_scale(p, pos);
  float q[2][RB][8];
#pragma unroll
  for (int r = 0; r < RB; ++r)
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      const int h = h0 + min(r, nh - 1);
      Raw8<E> x;
      ld8g<E, VEC>(qr + (2 * h + m) * D + lk * 8, D - lk * 8, x);
#pragma unroll
      for (int i = 0; i < 8; ++i) q[m][r][i] = x.f(i) * f;
    }
  auto add = [](float x, float y) { return x + y; };
  auto mxf = [](float x, float y) { return fmaxf(x, y); };
  float acc[NS][8];
#pragma unroll
  for (int s = 0; s < NS; ++s)
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[s][i] = 0.f;
  float mx[PPL], l[PPL];  // running maximum and sum of the score row this lane's pairs belong to
#pragma unroll
  for (int j = 0; j < PPL; ++j) mx[j] = -INFINITY, l[j] = 0.f;
  for (int k0 = lo + wv * KT; k0 < hi; k0 += 4 * KT) {
    Raw8<E> kx[NPK][2];
#pragma unroll
    for (int n = 0; n < NPK; ++n) {
      const int key = min(k0 + n * KPK + jk, hi - 1);
      const bool own = p.append && key == pos;
      const long long pg = tbl[key >> p.shift];
#pragma unroll
      for (int m = 0; m < 2; ++m) {
        const E* src = own ? kn + m * D
                           : kc + pg * p.k_sp + (((long long)(2 * g + m) << p.shift) + (key & pmask)) * D;
        ld8g<E, VEC>(src + lk * 8, D - lk * 8, kx[n][m]);
      }
    }
    Raw8<E> vx[NPV];
#pragma unroll
    for (int n = 0; n < NPV; ++n) {
      const int key = min(k0 + n * KPV + jv, hi - 1);
      const bool own = p.append && key == pos;
      const long long pg = tbl[key >> p.shift];
      const E* src = own ? vn : vc + pg * p.v_sp + (((long long)g << p.shift) + (key & pmask)) * Vd;
      ld8g<E, VEC>(src + lv * 8, Vd - lv * 8, vx[n]);
    }
#pragma unroll
    for (int n = 0; n < NPK; ++n)
#pragma unroll
      for (int m = 0; m < 2; ++m)
#pragma unroll
        for (int r = 0; r < RB; ++r) {
          float d = 0.f;
#pragma unroll
          for (int i = 0; i < 8; ++i) d = fmaf(q[m][r][i], kx[n][m].f(i), d);
          d = lanes_reduce<LPK>(d, add);
          const int kt = n * KPK + jk;
          if (lk == 0) sc[wv][kt][m * RB + r] = k0 + kt < hi ? d : -INFINITY;
        }
    wave_sync();
    float e[PPL];
#pragma unroll
    for (int j = 0; j < PPL; ++j) {  // pair (score row, key): the KT lanes of a row reduce together
      const int pr = min(lane + 64 * j, NP - KT + lane % KT), s = pr / KT, kt = pr % KT;
      const float x = sc[wv][kt][s];
      const float mn = fmaxf(mx[j], lanes_reduce<KT>(x, mxf));
      const float al = El<E>::ex(mx[j] - mn);
      e[j] = El<E>::ex(x - mn);
      l[j] = l[j] * al + lanes_reduce<KT>(e[j], add);
      mx[j] = mn;
      if (kt == 0) als[wv][s] = al;
    }
    wave_sync();
#pragma unroll
    for (int j = 0; j < PPL; ++j) {
      const int pr = min(lane + 64 * j, NP - KT + lane % KT);
      sc[wv][pr % KT][pr / KT] = e[j];
    }
    wave_sync();
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      const float al = als[wv][s];
#pragma unroll
      for (int i = 0; i < 8; ++i) acc[s][i] *= al;
    }
#pragma unroll
    for (int n = 0; n < NPV; ++n) {
      float w[NS];
#pragma unroll
      for (int s = 0; s < NS; ++s) w[s] = sc[wv][n * KPV + jv][s];
#pragma unroll
      for (int s = 0; s < NS; ++s)
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[s][i] = fmaf(w[s], vx[n].f(i), acc[s][i]);
    }
    wave_sync();
  }
  // the key lanes of a value row, then the four waves
#pragma unroll
  for (int s = 0; s < NS; ++s)
#pragma unroll
    for (int i = 0; i < 8; ++i)
#pragma unroll
      for (int o = LPV; o < 64; o <<= 1) acc[s][i] += __shfl_xor(acc[s][i], o, 64);
  if (jv == 0)
#pragma unroll
    for (int s = 0; s < NS; ++s)
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (lv * 8 + i < Vd) merged[(wv * NS + s) * Vd + lv * 8 + i] = acc[s][i];
#pragma unroll
  for (int j = 0; j < PPL; ++j) {
    const int pr = lane + 64 * j;
    if (pr < NP && pr % KT == 0) {
      wm[wv][pr / KT] = mx[j];
      wl[wv][pr / KT] = l[j];
    }
  }
  __syncthreads();
  if (p.append && hi == kv && sub == 0) {  // the split that holds the new token stores it
    const long long pg = tbl[pos >> p.shift];
    for (int i = tid; i < 2 * D + Vd; i += 256) {
      if (i < 2 * D) {
        const int m = i / D, c = i - m * D;
        kc[pg * p.k_sp + (((long long)(2 * g + m) << p.shift) + (pos & pmask)) * D + c] = kn[i];
      } else {
        const int c = i - 2 * D;
        vc[pg * p.v_sp + (((long long)g << p.shift) + (pos & pmask)) * Vd + c] = vn[c];
      }
    }
  }
  // waves -> this split's (m, l, acc)
  const long long blk = ((long long)blockIdx.x * gridDim.y + blockIdx.y);
  const int stride = NS * (Vd + 2);
  float* part = p.ws + (blk * p.nsplit + sp) * stride;
  for (int s = wv; s < NS; s += 4) {
    float M = fmaxf(fmaxf(wm[0][s], wm[1][s]), fmaxf(wm[2][s], wm[3][s]));
    float c[4], L = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      c[w] = wm[w][s] == -INFINITY ? 0.f : El<E>::ex(wm[w][s] - M);
      L += c[w] * wl[w][s];
    }
    for (int i = lane; i < Vd; i += 64) {
      float o = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) o += c[w] * merged[(w * NS + s) * Vd + i];
      if (used == 1) merged[s * Vd + i] = o / L;  // (wave w's slice s: read by this wave alone)
      else st_pub(part + s * (Vd + 2) + 2 + i, o);
    }
    if (used > 1 && lane == 0) {
      st_pub(part + s * (Vd + 2), M);
      st_pub(part + s * (Vd + 2) + 1, L);
    }
  }
  if (used > 1) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    if (tid == 0) {
      unsigned* ct = p.cnt + blk;
      const int last =
          __hip_atomic_fetch_add(ct, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == (unsigned)used - 1;
      if (last) {
        __hip_atomic_store(ct, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "agent");
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      }
      s_last = last;
    }
    __syncthreads();
    if (!s_last) return;
    // weights of the splits first (a wave per score row), then every thread sums outputs, UZ splits' loads
    // in flight
    const float* base = p.ws + blk * p.nsplit * stride;
    __shared__ float wz[NS][MAX_SPLITS];
    for (int s = wv; s < NS; s += 4) {
      const float* b = base + s * (Vd + 2);
      float M = -INFINITY, L = 0.f;
      for (int z = lane; z < used; z += 64) M = fmaxf(M, b[(long long)z * stride]);
      M = wave_max(M);
      for (int z = lane; z < used; z += 64) {
        const float c = El<E>::ex(b[(long long)z * stride] - M);
        wz[s][z] = c;
        L += c * b[(long long)z * stride + 1];
      }
      L = 1.f / wave_sum(L);
      for (int z = lane; z < used; z += 64) wz[s][z] *= L;
    }
    __syncthreads();
    constexpr int UZ = 16;
    for (int i = tid; i < NS * Vd; i += 256) {
      const int s = i / Vd;
      const float* b = base + i + 2 * s + 2;  // s * (Vd + 2) + 2 + i % Vd
      float o = 0.f;
      for (int z0 = 0; z0 < used; z0 += UZ) {
        float x[UZ];
#pragma unroll
        for (int u = 0; u < UZ; ++u) x[u] = b[(long long)min(z0 + u, used - 1) * stride];
#pragma unroll
        for (int u = 0; u < UZ; ++u)
          if (z0 + u < used) o = fmaf(wz[s][z0 + u], x[u], o);
      }
      merged[i] = o;
    }
  }
  __syncthreads();
  E* orow = reinterpret_cast<E*>(p.out) + row * p.ldo;
  for (int r = wv; r < nh; r += 4) {
    const float *a1 = merged + r * Vd, *a2 = merged + (RB + r) * Vd;
    float ss = 0.f;
    for (int i = lane; i < Vd; i += 64) {
      const float o = a1[i] - p.lambda * a2[i];
      ss = fmaf(o, o, ss);
    }
    const float n = p.gain / sqrtf(wave_sum(ss) / (float)Vd + p.eps);
    for (int i = lane; i < Vd; i += 64) El<E>::st(orow + (h0 + r) * Vd + i, (a1[i] - p.lambda * a2[i]) * n);
  }
}

// ---------------------------------------------------------------------------------------- tile kernel
// 8 waves: four groups of 32 queries of one head, a wave per map (wave w and w + 4 share the queries and
// a SIMD, so one map's softmax runs under the other's matrix products). 32-key tiles of K1 | K2 | V double
// buffered in LDS (the image of attn_tile.h); S^T = K Q^T leaves a query per lane, and P^T feeds
// O^T += V^T P^T from registers. At the end the second map's output crosses over through LDS.
template <int DK, int DV>
__global__ void __launch_bounds__(512, 2) diff_tile_kernel(DiffArgs p) {
  constexpr int BN = 32, TK = BN * DK * 2, TV = BN * DV * 2, BUF = 2 * TK + TV;
  constexpr int KS = DK / 16, NB = DV / 32;
  constexpr int CK = 2 * BN * (DK / 8), CV = BN * (DV / 8), NC = CK + CV;  // 16-B chunks per tile
  constexpr int CPT = (NC + 511) / 512;
  constexpr int NR = 2 * BUF / 16384 < NB ? 2 * BUF / 16384 : NB;          // 32-dim blocks crossing per round
  static_assert(NR >= 1, "cross-over buffer");
  extern __shared__ __attribute__((aligned(16))) char smem[];  // [2][K1 | K2 | V]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, qg = wave & 3;
  const int map = __builtin_amdgcn_readfirstlane(wave >> 2);
  const int l32 = lane & 31, hh = lane >> 5, gi = lane & 15;
  const int lid = xcd_remap(blockIdx.x, gridDim.x);
  const int ti = lid / p.H, h = lid % p.H, g = h / (p.H / p.G);
  const int* tl = p.tiles + ti * 4;
  const int row0 = tl[0], nrow = tl[1], pos0 = tl[2], slot = tl[3];
  const int qi = qg * 32 + l32;
  const bool live = qi < nrow;
  const int row = row0 + min(qi, nrow - 1), pos = pos0 + min(qi, nrow - 1);
  const int kv_hi = pos0 + nrow;                                  // keys any query of the tile sees
  const int ntiles = (kv_hi + BN - 1) / BN;
  const int wave_hi = pos0 + min(qg * 32 + 32, nrow);             // ... any query of this wave
  const bool busy = qg * 32 < nrow;
  const int D = p.dim, Vd = p.vdim;
  const int* tbl = p.table + (long long)slot * p.tstride;
  const bf16_t* kc = reinterpret_cast<const bf16_t*>(p.kc);
  const bf16_t* vc = reinterpret_cast<const bf16_t*>(p.vc);

  bf16x8 qf[KS];
#pragma unroll
  for (int s = 0; s < KS; ++s) {
    const int c = 16 * s + 8 * hh;
    u32x4 v = {0u, 0u, 0u, 0u};
    if (c < D)
      v = *reinterpret_cast<const u32x4*>(reinterpret_cast<const bf16_t*>(p.qkv) + row * p.ld + (2 * h + map) * D + c);
    qf[s] = __builtin_bit_cast(bf16x8, v);
  }
  const float sl2 = row_scale(p, pos) * kLog2e;

  // this thread's chunks: K chunks first (map, row, chunk), then V
  auto load = [&](int k0, u32x4 (&st)[CPT]) {
    const long long pg = tbl[k0 >> p.shift];
    const int o0 = k0 & ((1 << p.shift) - 1);
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int c = tid + 512 * i;
      st[i] = u32x4{0u, 0u, 0u, 0u};
      if (c < CK) {
        const int m = c / (BN * (DK / 8)), r = (c / (DK / 8)) % BN, ch = c % (DK / 8);
        if (ch * 8 < D)
          st[i] = *reinterpret_cast<const u32x4*>(kc + pg * p.k_sp +
                                                  (((long long)(2 * g + m) << p.shift) + o0 + r) * D + ch * 8);
      } else if (c < NC) {
        const int cv = c - CK, r = cv / (DV / 8), ch = cv % (DV / 8);
        if (ch * 8 < Vd && k0 + r < kv_hi)
          st[i] = *reinterpret_cast<const u32x4*>(vc + pg * p.v_sp + (((long long)g << p.shift) + o0 + r) * Vd + ch * 8);
      }
    }
  };
  auto store = [&](const u32x4 (&st)[CPT], char* buf) {
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const int c = tid + 512 * i;
      if (c < CK) {
        const int m = c / (BN * (DK / 8)), r = (c / (DK / 8)) % BN, ch = c % (DK / 8);
        *reinterpret_cast<u32x4*>(buf + m * TK + img_off<DK>(r, ch)) = st[i];
      } else if (c < NC) {
        const int cv = c - CK, r = cv / (DV / 8), ch = cv % (DV / 8);
        *reinterpret_cast<u32x4*>(buf + 2 * TK + img_off<DV>(r, ch)) = st[i];
      }
    }
  };

  const int xr = (l32 >> 2) & 3;
  const int kb_e = map * TK + (l32 >> 3) * 16 * DK + 64 * (l32 & 7) + 16 * (hh ^ xr);
  const int kb_o = map * TK + (l32 >> 3) * 16 * DK + 64 * (l32 & 7) + 16 * ((2 + hh) ^ xr);
  const int c3 = 2 * ((lane >> 4) & 1) + ((gi & 3) >> 1);
  const int vb_1 = 2 * TK + 64 * (4 * hh + (gi >> 2)) + 16 * (c3 ^ hh) + 8 * (gi & 1);
  const int vb_2 = 2 * TK + 16 * DV + 64 * (4 * hh + (gi >> 2)) + 16 * (c3 ^ hh ^ 2) + 8 * (gi & 1);

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
  for (int t = 0; t < ntiles; ++t) {
    const char* buf = smem + (t & 1) * BUF;
    const int k0 = t * BN;
    const bool more = t + 1 < ntiles;
    if (more) load(k0 + BN, st);
    if (busy && k0 < wave_hi) {  // (tiles past the wave's last query: staging only)
      f32x16 s;
#pragma unroll
      for (int r = 0; r < 16; ++r) s[r] = 0.f;
      bf16x8 fk[3];  // K fragments two steps ahead of their products
      fk[0] = lds_b128(buf, kb_e);
      if constexpr (KS > 1) fk[1] = lds_b128(buf, kb_o);
      __builtin_amdgcn_sched_group_barrier(0x100, KS > 1 ? 2 : 1, 0);
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
      mt = fmaxf(mt, __shfl_xor(mt, 32, 64));
      mt = sl2 >= 0.f ? mt * sl2 : mt;  // (see the minimum below)
      if (sl2 < 0.f) {                  // a negative temperature turns the row's maximum into its minimum
        float mi = INFINITY;
#pragma unroll
        for (int r = 0; r < 16; ++r) mi = s[r] == -INFINITY ? mi : fminf(mi, s[r]);
        mt = fminf(mi, __shfl_xor(mi, 32, 64)) * sl2;
#pragma unroll
        for (int r = 0; r < 16; ++r)
          if (s[r] == -INFINITY) s[r] = INFINITY;  // masked keys: weight exp2(-inf)
      }
      // the reference maximum follows only when a tile exceeds it by more than 2^8: weights stay finite
      // and the rescale leaves the common path
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
  // o <- o / l (second map: lambda o / l), the second map's block by block to the first's wave
  const float l = ls + __shfl_xor(ls, 32, 64);
  const float mul = (map ? p.lambda : 1.f) / (l > 0.f ? l : 1.f);
  float* cross = reinterpret_cast<float*>(smem) + qg * (NR * 1024);  // [NR][4][64 lanes][4]
  float ss = 0.f;
#pragma unroll
  for (int b0 = 0; b0 < NB; b0 += NR) {
    if (map) {
#pragma unroll
      for (int b = 0; b < NR; ++b)
        if (b0 + b < NB)
#pragma unroll
          for (int q4 = 0; q4 < 4; ++q4)
            *reinterpret_cast<float4*>(cross + ((b * 4 + q4) * 64 + lane) * 4) =
                make_float4(o[b0 + b][4 * q4] * mul, o[b0 + b][4 * q4 + 1] * mul, o[b0 + b][4 * q4 + 2] * mul,
                            o[b0 + b][4 * q4 + 3] * mul);
    }
    __syncthreads();
    if (!map) {
#pragma unroll
      for (int b = 0; b < NR; ++b)
        if (b0 + b < NB)
#pragma unroll
          for (int q4 = 0; q4 < 4; ++q4) {
            const float4 y = *reinterpret_cast<const float4*>(cross + ((b * 4 + q4) * 64 + lane) * 4);
            const float yy[4] = {y.x, y.y, y.z, y.w};
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              const float x = o[b0 + b][4 * q4 + e] * mul - yy[e];  // (padded dims: zero)
              o[b0 + b][4 * q4 + e] = x;
              ss = fmaf(x, x, ss);
            }
          }
    }
    __syncthreads();
  }
  if (map) return;
  ss += __shfl_xor(ss, 32, 64);
  const float n = p.gain / sqrtf(ss / (float)Vd + p.eps);
  if (!live) return;
  bf16_t* orow = reinterpret_cast<bf16_t*>(p.out) + row * p.ldo + h * Vd;
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int q4 = 0; q4 < 4; ++q4) {
      const int c = 32 * b + 8 * q4 + 4 * hh;
      if (c < Vd)
        *reinterpret_cast<uint2*>(orow + c) = make_uint2(pk_bf16(o[b][4 * q4] * n, o[b][4 * q4 + 1] * n),
                                                         pk_bf16(o[b][4 * q4 + 2] * n, o[b][4 * q4 + 3] * n));
    }
}

template <typename E, int RB, int LPK, int LPV, bool VEC>
int rows_go(const DiffArgs& p, int rows, hipStream_t s) {
  const int Hg = p.H / p.G, nsub = (Hg + RB - 1) / RB;
  const size_t lds = (size_t)4 * 2 * RB * p.vdim * 4;
  auto kern = diff_rows_kernel<E, RB, LPK, LPV, VEC>;
  if (lds > 48 * 1024)
    if (hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) != hipSuccess) return 5;
  hipLaunchKernelGGL(kern, dim3(rows, p.G * nsub, p.nsplit), dim3(256), lds, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

int rb_for(int Hg, bool vec) { return vec && Hg > 1 ? 4 : 1; }

template <typename E>
int rows_dispatch(const DiffArgs& p, int rows, bool vec, hipStream_t s) {
  int lk = lanes_for(p.dim), lv = lanes_for(p.vdim);
  if (lk > 64 || lv > 64) return 10;
  if (!vec) return rows_go<E, 1, 64, 64, false>(p, rows, s);
  const bool half = lk * 2 == lv;
  if (lk != lv && !half) lk = lv = lk > lv ? lk : lv;
  const bool r4 = rb_for(p.H / p.G, vec) == 4;
#define R2(A, B) (r4 ? rows_go<E, 4, A, B, true>(p, rows, s) : rows_go<E, 1, A, B, true>(p, rows, s))
  if (half) {
    if (lv == 16) return R2(8, 16);
    if (lv == 32) return R2(16, 32);
    return R2(32, 64);
  }
  if (lv == 8) return R2(8, 8);
  if (lv == 16) return R2(16, 16);
  if (lv == 32) return R2(32, 32);
  return R2(64, 64);
#undef R2
}

template <int DK, int DV>
int tile_go(const DiffArgs& p, int ntiles, hipStream_t s) {
  constexpr int lds = 2 * (2 * 32 * DK * 2 + 32 * DV * 2);
  auto kern = diff_tile_kernel<DK, DV>;
  if (lds > 48 * 1024)
    if (hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess) return 5;
  hipLaunchKernelGGL(kern, dim3(ntiles * p.H), dim3(512), lds, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

template <int DK>
int tile_dv(const DiffArgs& p, int ntiles, hipStream_t s) {
  if (p.vdim <= 64) return tile_go<DK, 64>(p, ntiles, s);
  if (p.vdim <= 96) return tile_go<DK, 96>(p, ntiles, s);
  if (p.vdim <= 128) return tile_go<DK, 128>(p, ntiles, s);
  if (p.vdim <= 192) return tile_go<DK, 192>(p, ntiles, s);
  return tile_go<DK, 256>(p, ntiles, s);
}

bool args_ok(const DiffArgs& p) {
  return p.H > 0 && p.G > 0 && p.H % p.G == 0 && p.dim > 0 && p.vdim > 0 && p.shift >= 4 && p.qkv && p.kc && p.vc &&
         p.table && p.ld >= 2LL * p.H * p.dim + 2LL * p.G * p.dim + (long long)p.G * p.vdim;
}

bool vec_ok(const DiffArgs& p) {
  return p.dim % 8 == 0 && p.vdim % 8 == 0 && p.ld % 8 == 0 && (uintptr_t)p.qkv % 16 == 0 && (uintptr_t)p.kc % 16 == 0 &&
         (uintptr_t)p.vc % 16 == 0 && p.k_sp % 8 == 0 && p.v_sp % 8 == 0;
}

}  // namespace

// Mirrored by ops/diff_attention.py (checked by kca_diff_attn_abi)
struct KcaDiffAttn {
  DiffArgs a;
};
KCA_API int kca_diff_attn_abi() { return (int)sizeof(KcaDiffAttn); }

// K / V of T tokens (rows of qkv) into their pages
KCA_API int kca_diff_append(const KcaDiffAttn* in, int dtype, int T, hipStream_t s) {
  const DiffArgs& p = in->a;
  if (!args_ok(p) || !p.pos || !p.slot || T < 1) return 1;
  if (dtype != 0 && dtype != 1) return 3;
  const bool vec = vec_ok(p);
  const long long work = (long long)T * (2 * p.G * p.dim + p.G * p.vdim) / (vec ? (dtype ? 8 : 4) : 1);
  const dim3 g(kca_grid(work, 256, 8192));
  if (dtype == 0 && vec) hipLaunchKernelGGL((kv_append_kernel<float, 4>), g, dim3(256), 0, s, p, T);
  else if (dtype == 0) hipLaunchKernelGGL((kv_append_kernel<float, 1>), g, dim3(256), 0, s, p, T);
  else if (vec) hipLaunchKernelGGL((kv_append_kernel<bf16_t, 8>), g, dim3(256), 0, s, p, T);
  else hipLaunchKernelGGL((kv_append_kernel<bf16_t, 1>), g, dim3(256), 0, s, p, T);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

// head sub-groups a group's query heads are cut in, i.e. workspace / counter blocks per (row, group)
KCA_API int kca_diff_rows_plan(const KcaDiffAttn* in, int* sub, int* rb) {
  const DiffArgs& p = in->a;
  if (!args_ok(p)) return 1;
  *rb = rb_for(p.H / p.G, vec_ok(p));
  *sub = (p.H / p.G + *rb - 1) / *rb;
  return 0;
}

// One query token per row. nsplit * chunk must cover every row's pos + 1 keys.
KCA_API int kca_diff_rows(const KcaDiffAttn* in, int dtype, int rows, long long ws_floats, long long n_cnt, int max_kv,
                          hipStream_t s) {
  const DiffArgs& p = in->a;
  if (!args_ok(p) || !p.pos || !p.slot || !p.out || rows < 1 || p.nsplit < 1 || p.chunk < 1 || p.nsplit > MAX_SPLITS)
    return 1;
  if ((long long)p.nsplit * p.chunk < max_kv) return 2;
  const bool vec = vec_ok(p);
  const int rb = rb_for(p.H / p.G, vec), nsub = (p.H / p.G + rb - 1) / rb;
  if (p.nsplit > 1) {
    const long long blk = (long long)rows * p.G * nsub;
    if (!p.ws || !p.cnt || n_cnt < blk || ws_floats < blk * p.nsplit * 2 * rb * (p.vdim + 2)) return 5;
  }
  if (dtype == 0) return rows_dispatch<float>(p, rows, vec, s);
  if (dtype == 1) return rows_dispatch<bf16_t>(p, rows, vec, s);
  return 3;
}

// 10: a shape for the rows kernel
KCA_API int kca_diff_tiles(const KcaDiffAttn* in, int ntiles, hipStream_t s) {
  const DiffArgs& p = in->a;
  if (!args_ok(p) || !p.tiles || !p.out || ntiles < 1) return 1;
  if (!vec_ok(p) || p.dim > 128 || p.vdim > 256 || p.shift < 5 || p.ldo % 4 || (uintptr_t)p.out % 8) return 10;
  if (p.dim <= 32) return tile_dv<32>(p, ntiles, s);
  if (p.dim <= 64) return tile_dv<64>(p, ntiles, s);
  if (p.dim <= 96) return tile_dv<96>(p, ntiles, s);
  return tile_dv<128>(p, ntiles, s);
}
