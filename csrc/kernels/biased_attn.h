// Causal attention over the paged cache, kernels of biased_attn.hip (POOL false) and pooled_attn.hip (POOL true):
//   w_j = exp(q . k_j * scale + bias[h][min(pos - j, nb - 1)])
//   o = sum_j w_j v_j / (exp(sink_h) + sum_j w_j) * sigmoid(g)
// Query heads share key / value heads in groups. K pages [G][PS][dim], V pages [G][PS][vdim]. q / k / v / g are column
// blocks of one projection buffer. Norms, angles, scores, weights and the gate are fp32.
// POOL: a query at pos sees the tokens (pos - window, pos] and, as one key and value each, the means of the whole blocks
// of `pool` tokens that end at or before pos - window; a page holds the means of the blocks that end in it
// ([G][per][dim] / [vdim], block b in row (end % PS) / pool). No bias, no gate; `mul` scales the output.
//
//   rows kernel        one query token per row, any dims, fp32 or bf16 (vector units): decode (split over
//                      keys, the last arriving split merges; the new token's K / V is appended here) and
//                      every shape or type the matrix-core kernel does not take
//   tile kernel        bf16 prompt portions on the matrix cores: 128 queries of one (entry, head) per workgroup
#pragma once
#include "attn_rows.h"
#include "attn_tile.h"
#include "decode_tail.h"
#include "lanes.h"

namespace {

struct BiasedArgs {
  const void* x;            // rows of the projections, row stride ld
  long long ld;
  int o_q, o_k, o_v, o_g;   // column blocks; o_g < 0: no gate
  void* kc;                 // [pages][G][PS][dim]
  void* vc;                 // [pages][G][PS][vdim]
  long long k_sp, v_sp;     // page strides (elements)
  const int* table;         // [slots][tstride] page of each block
  int tstride, shift;
  const int* pos;           // [rows] position of the row's token
  const int* slot;          // [rows]
  void* out;                // [rows][H * vdim], row stride ldo
  long long ldo;
  int H, G, dim, vdim;
  float scale, eps;
  const void* qn;           // [dim] gains of the query and key norms (nullable: no norm); POOL: [H dim], [G dim], one
  const void* kn;           // norm over all heads
  const float* bias;        // [H][nb], the last column for every distance beyond (nullable: none)
  int nb;
  const float* sink;        // [H] (nullable: none)
  int append;               // rows kernel: key `pos` comes from the row's own k / v, which it also stores
  int nsplit, chunk;        // rows kernel: keys per split
  float* ws;                // split partials
  unsigned* cnt;            // [rows * G * subgroups] arrival counters (zero, re-armed)
  const int* tiles;         // tile kernel: [ntiles][4] first row, rows, position of first row, slot
  const int* row_of;        // rows kernel: row index of block b (nullable: b)
  int window, pool, per;    // POOL: tokens seen, tokens of a block, block means a page holds
  unsigned pool_mul;        // ceil(2^20 / pool)
  void* kb;                 // [pages][G][per][dim] block means of keys
  void* vb;                 // [pages][G][per][vdim] ... of values
  long long kb_sp, vb_sp;   // page strides (elements)
  const float* freq;        // [rot / 2] radians per position
  int rot;                  // leading dims of a head that rotate, in pairs (i, i + rot / 2)
  float mul;
};

// blocks that end at or before pos - window
__device__ __forceinline__ int blocks_seen(const BiasedArgs& p, int pos) {
  const int n = pos - p.window + 1;
  return n > 0 ? n / p.pool : 0;
}
// row of the block that ends at position `end`, among a head's means in its page
__device__ __forceinline__ int block_row(const BiasedArgs& p, int end) {
  return (int)((unsigned)(end & ((1 << p.shift) - 1)) * p.pool_mul >> 20);
}
__host__ __device__ __forceinline__ int pool_lds(int rb, int dim, int rot) { return (rb + 1) * dim + rot; }  // floats

template <typename E>
__device__ __forceinline__ float gate_of(float z) {
  if constexpr (sizeof(E) == 4) return 1.f / (1.f + expf(-z));
  else return __builtin_amdgcn_rcpf(1.f + __expf(-z));
}

// ---------------------------------------------------------------------------------------- rows kernel
// Workgroup: (row, kv group g, RB query heads of the group, key split), 4 waves. Each wave walks its own
// KT-key tiles of the split with its own online softmax: LPK lanes share a key's dot products and a value
// row; a wave-private LDS array carries the RB x KT weights between the two layouts. The waves, then the
// splits, merge at the end, where the sink joins.
constexpr int MAX_SPLITS = 256;

template <typename E, int RB, int LP, bool VEC, bool POOL>
__device__ __forceinline__ void rows_body(const BiasedArgs& p, int bx, int by, int sp, int ny) {  // workgroup (bx, by, sp), ny of by
  constexpr int KT = LP >= 64 ? 4 : (LP >= 32 ? 8 : 16);  // keys per tile of a wave
  constexpr int KP = 64 / LP, NPASS = KT / KP;            // keys per pass, passes
  static_assert(KP <= KT, "a pass covers at most one tile");
  constexpr int NP = RB * KT, PPL = (NP + 63) / 64;       // (head, key) pairs, pairs per lane
  __shared__ __attribute__((aligned(16))) float sc[4][KT][RB], als[4][RB];
  __shared__ float wm[4][RB], wl[4][RB];
  __shared__ int s_last;
  extern __shared__ __attribute__((aligned(16))) float merged[];  // [4][RB][vdim] then reused; POOL: + the prepared heads
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int D = p.dim, Vd = p.vdim, Hg = p.H / p.G;
  const int nsub = (Hg + RB - 1) / RB;
  const int row = p.row_of ? p.row_of[bx] : bx;
  const int g = by / nsub, sub = by % nsub;
  const int h0 = g * Hg + sub * RB, nh = min(RB, Hg - sub * RB);
  const int pos = p.pos[row], slot = p.slot[row];
  const int nbs = POOL ? blocks_seen(p, pos) : 0;                 // keys [0, nbs): block means,
  const int first = POOL ? max(0, pos - p.window + 1) : 0;        // [nbs, kv): tokens from here on
  const int kv = pos + 1 - first + nbs;
  const int lo = sp * p.chunk, hi = min(kv, lo + p.chunk);
  const int used = (kv + p.chunk - 1) / p.chunk;  // splits that hold keys
  if (sp >= used) return;
  const int* tbl = p.table + (long long)slot * p.tstride;
  const int pmask = (1 << p.shift) - 1;
  const E* xr = reinterpret_cast<const E*>(p.x) + row * p.ld;
  const E* vn = xr + p.o_v + g * Vd;  // the row's own value
  E* kc = reinterpret_cast<E*>(p.kc);
  E* vc = reinterpret_cast<E*>(p.vc);

  const int ll = lane % LP, jj = lane / LP;
  auto add = [](float x, float y) { return x + y; };
  auto mxf = [](float x, float y) { return fmaxf(x, y); };
  float q[RB][8];
  Raw8<E> kown;  // the row's own key, normed and rounded as the page holds it
  // a tile's keys and values (POOL: the first tile's before the norms; more in flight would cost resident waves)
  Raw8<E> kx[NPASS], vx[NPASS];
  auto fetch = [&](int k0) {
#pragma unroll
    for (int n = 0; n < NPASS; ++n) {
      const int key = min(k0 + n * KP + jj, hi - 1);
      const bool mean = POOL && key < nbs;
      const int at = !POOL ? key : mean ? key * p.pool + p.pool - 1 : key - nbs + first;
      const long long pg = tbl[at >> p.shift];
      const E *kr, *vr;
      if (mean) {
        const long long in = (long long)g * p.per + block_row(p, at);
        kr = reinterpret_cast<const E*>(p.kb) + pg * p.kb_sp + in * D;
        vr = reinterpret_cast<const E*>(p.vb) + pg * p.vb_sp + in * Vd;
      } else {
        const long long in = ((long long)g << p.shift) + (at & pmask);
        kr = kc + pg * p.k_sp + in * D;
        vr = vc + pg * p.v_sp + in * Vd;
      }
      if (!POOL && p.append && key == kv - 1) kx[n] = kown;
      else ld8g<E, VEC>(kr + ll * 8, D - ll * 8, kx[n]);
      ld8g<E, VEC>((p.append && key == kv - 1 ? vn : vr) + ll * 8, Vd - ll * 8, vx[n]);
    }
  };
  if (POOL && lo + wv * KT < hi) fetch(lo + wv * KT);
  if constexpr (POOL) {
    if (p.append) {  // norms over the whole projections, this group's heads normed in LDS, then rotated
      __shared__ float red[2][4];
      float *qs = merged + 4 * RB * Vd, *cs = qs + (RB + 1) * D, *sn = cs + p.rot / 2;  // heads: queries, then the key
      const E *gq = reinterpret_cast<const E*>(p.qn), *gk = reinterpret_cast<const E*>(p.kn);
      float sq = 0.f, sk = 0.f;
      const int nq = p.H * D, nk = p.G * D;
#pragma unroll 2
      for (int c = tid * 8; c < nq; c += 2048) {
        Raw8<E> u;
        ld8g<E, VEC>(xr + p.o_q + c, nq - c, u);
#pragma unroll
        for (int i = 0; i < 8; ++i) sq = fmaf(u.f(i), u.f(i), sq);
      }
      for (int c = tid * 8; c < nk; c += 2048) {
        Raw8<E> u;
        ld8g<E, VEC>(xr + p.o_k + c, nk - c, u);
#pragma unroll
        for (int i = 0; i < 8; ++i) sk = fmaf(u.f(i), u.f(i), sk);
      }
      constexpr int MINE = ((RB + 1) * 8 * LP + 255) / 256;  // this thread's elements of the heads, and their partners
      const int half = p.rot / 2;
      float own[MINE], gain[MINE], other[MINE], gain2[MINE];
#pragma unroll
      for (int j = 0; j < MINE; ++j) {
        const int i = min(tid + 256 * j, (RB + 1) * D - 1), r = i / D, c = i - r * D;
        const int col = r < RB ? (h0 + min(r, nh - 1)) * D + c : g * D + c, turn = c < half ? half : c < 2 * half ? -half : 0;
        const E *xs = xr + (r < RB ? p.o_q : p.o_k) + col, *gs = (r < RB ? gq : gk) + col;
        own[j] = El<E>::ld(xs);
        gain[j] = El<E>::ld(gs);
        other[j] = El<E>::ld(xs + turn);
        gain2[j] = El<E>::ld(gs + turn);
      }
      for (int i = tid; i < half; i += 256) sincosf((float)pos * p.freq[i], sn + i, cs + i);
      sq = lanes_reduce<64>(sq, add);
      sk = lanes_reduce<64>(sk, add);
      if (lane == 0) red[0][wv] = sq, red[1][wv] = sk;
      __syncthreads();
      const float rq = 1.f / sqrtf((red[0][0] + red[0][1] + red[0][2] + red[0][3]) / (float)nq + p.eps);
      const float rk = 1.f / sqrtf((red[1][0] + red[1][1] + red[1][2] + red[1][3]) / (float)nk + p.eps);
#pragma unroll
      for (int j = 0; j < MINE; ++j) {
        const int i = tid + 256 * j, r = i / D, c = i - r * D;
        if (r > RB) break;
        const float n = r < RB ? rq : rk;
        float u = own[j] * n * gain[j];
        if (c < 2 * half) {
          const int f = c < half ? c : c - half;
          u = u * cs[f] + (c < half ? -1.f : 1.f) * (other[j] * n * gain2[j]) * sn[f];
        }
        qs[i] = r < RB ? u * p.scale : u;
      }
      __syncthreads();
#pragma unroll
      for (int r = 0; r <= RB; ++r) {
        const float* u = qs + r * D + ll * 8;
        float v[8];
        if constexpr (VEC) {
          const int o = ll * 8 < D ? 0 : -ll * 8;  // (past the head: in bounds, and zero)
          load8f(u + o, v);
#pragma unroll
          for (int i = 0; i < 8; ++i) v[i] = o ? 0.f : v[i];
        } else {
#pragma unroll
          for (int i = 0; i < 8; ++i) v[i] = ll * 8 + i < D ? u[i] : 0.f;
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
          if (r < RB) q[r < RB ? r : 0][i] = v[i];
          else El<E>::st(kown.v + i, v[i]);
        }
      }
    } else {
#pragma unroll
      for (int r = 0; r < RB; ++r) {
        Raw8<E> x;
        ld8g<E, VEC>(xr + p.o_q + (h0 + min(r, nh - 1)) * D + ll * 8, D - ll * 8, x);
#pragma unroll
        for (int i = 0; i < 8; ++i) q[r][i] = x.f(i) * p.scale;
      }
    }
  } else {
    Raw8<E> x[RB], w, kw;
#pragma unroll
    for (int r = 0; r < RB; ++r) ld8g<E, VEC>(xr + p.o_q + (h0 + min(r, nh - 1)) * D + ll * 8, D - ll * 8, x[r]);
    ld8g<E, VEC>(xr + p.o_k + g * D + ll * 8, D - ll * 8, kown);
    if (p.qn) ld8g<E, VEC>(reinterpret_cast<const E*>(p.qn) + ll * 8, D - ll * 8, w);
    if (p.kn) ld8g<E, VEC>(reinterpret_cast<const E*>(p.kn) + ll * 8, D - ll * 8, kw);
#pragma unroll
    for (int r = 0; r < RB; ++r) {
      float n = 1.f;
      if (p.qn) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) ss = fmaf(x[r].f(i), x[r].f(i), ss);
        n = 1.f / sqrtf(lanes_reduce<LP>(ss, add) / (float)D + p.eps);
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) q[r][i] = x[r].f(i) * n * (p.qn ? w.f(i) : 1.f) * p.scale;
    }
    if (p.kn) {
      float ss = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) ss = fmaf(kown.f(i), kown.f(i), ss);
      const float n = 1.f / sqrtf(lanes_reduce<LP>(ss, add) / (float)D + p.eps);
#pragma unroll
      for (int i = 0; i < 8; ++i) El<E>::st(kown.v + i, kown.f(i) * n * kw.f(i));
    }
  }
  float acc[RB][8];
#pragma unroll
  for (int s = 0; s < RB; ++s)
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[s][i] = 0.f;
  float mx[PPL], l[PPL];  // running maximum and sum of the head this lane's pairs belong to
#pragma unroll
  for (int j = 0; j < PPL; ++j) mx[j] = -INFINITY, l[j] = 0.f;
  for (int k0 = lo + wv * KT; k0 < hi; k0 += 4 * KT) {
    if (!POOL || k0 > lo + wv * KT) fetch(k0);
#pragma unroll
    for (int n = 0; n < NPASS; ++n)  // (the page does not hold the new key yet)
      if (POOL && p.append && min(k0 + n * KP + jj, hi - 1) == kv - 1) kx[n] = kown;
    float bv[PPL];
#pragma unroll
    for (int j = 0; j < PPL; ++j) {
      const int pr = min(lane + 64 * j, NP - KT + lane % KT), s = pr / KT, kt = pr % KT;
      bv[j] = !POOL && p.bias ? p.bias[(long long)(h0 + min(s, nh - 1)) * p.nb + min(max(pos - (k0 + kt), 0), p.nb - 1)] : 0.f;
    }
#pragma unroll
    for (int n = 0; n < NPASS; ++n)
#pragma unroll
      for (int r = 0; r < RB; ++r) {
        float d = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) d = fmaf(q[r][i], kx[n].f(i), d);
        d = lanes_reduce<LP>(d, add);
        const int kt = n * KP + jj;
        if (ll == 0) sc[wv][kt][r] = k0 + kt < hi ? d : -INFINITY;
      }
    wave_sync();
    float e[PPL];
#pragma unroll
    for (int j = 0; j < PPL; ++j) {  // pair (head, key): the KT lanes of a head reduce together
      const int pr = min(lane + 64 * j, NP - KT + lane % KT), s = pr / KT, kt = pr % KT;
      const float x = sc[wv][kt][s] + bv[j];
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
    for (int s = 0; s < RB; ++s) {
      const float al = als[wv][s];
#pragma unroll
      for (int i = 0; i < 8; ++i) acc[s][i] *= al;
    }
#pragma unroll
    for (int n = 0; n < NPASS; ++n) {
      float w[RB];
#pragma unroll
      for (int s = 0; s < RB; ++s) w[s] = sc[wv][n * KP + jj][s];
#pragma unroll
      for (int s = 0; s < RB; ++s)
#pragma unroll
        for (int i = 0; i < 8; ++i) acc[s][i] = fmaf(w[s], vx[n].f(i), acc[s][i]);
    }
    wave_sync();
  }
  // the key lanes of a value row, then the four waves
#pragma unroll
  for (int s = 0; s < RB; ++s)
#pragma unroll
    for (int i = 0; i < 8; ++i)
#pragma unroll
      for (int o = LP; o < 64; o <<= 1) acc[s][i] += __shfl_xor(acc[s][i], o, 64);
  if (jj == 0)
#pragma unroll
    for (int s = 0; s < RB; ++s)
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (ll * 8 + i < Vd) merged[(wv * RB + s) * Vd + ll * 8 + i] = acc[s][i];
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
    const long long pg = tbl[pos >> p.shift], in = ((long long)g << p.shift) + (pos & pmask);
    if (tid < LP)
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (ll * 8 + i < D) kc[pg * p.k_sp + in * D + ll * 8 + i] = kown.v[i];
    for (int c = tid; c < Vd; c += 256) vc[pg * p.v_sp + in * Vd + c] = vn[c];
    if (POOL && (pos + 1) % p.pool == 0 && wv < 2 && lane < LP) {  // it completes a block: wave 0 the keys' mean, wave 1 the values'
      const int n = wv ? Vd : D;
      const E* src = wv ? vc : kc;
      const long long psz = wv ? p.v_sp : p.k_sp;
      float sum[8];
      Raw8<E> u = kown;
      if (wv) ld8g<E, VEC>(vn + ll * 8, n - ll * 8, u);
#pragma unroll
      for (int i = 0; i < 8; ++i) sum[i] = u.f(i);
#pragma unroll 4
      for (int j = 1; j < p.pool; ++j) {
        const int at = pos - j;
        ld8g<E, VEC>(src + tbl[at >> p.shift] * psz + (((long long)g << p.shift) + (at & pmask)) * n + ll * 8, n - ll * 8, u);
#pragma unroll
        for (int i = 0; i < 8; ++i) sum[i] += u.f(i);
      }
      E* dst = (wv ? reinterpret_cast<E*>(p.vb) + pg * p.vb_sp : reinterpret_cast<E*>(p.kb) + pg * p.kb_sp) +
               ((long long)g * p.per + block_row(p, pos)) * n + ll * 8;
#pragma unroll
      for (int i = 0; i < 8; ++i)
        if (ll * 8 + i < n) El<E>::st(dst + i, sum[i] / (float)p.pool);
    }
  }
  // waves -> this split's (m, l, acc)
  const long long blk = (long long)bx * ny + by;
  const int stride = RB * (Vd + 2);
  float* part = p.ws + (blk * p.nsplit + sp) * stride;
  for (int s = wv; s < RB; s += 4) {
    float M = fmaxf(fmaxf(wm[0][s], wm[1][s]), fmaxf(wm[2][s], wm[3][s]));
    float c[4], L = 0.f;
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      c[w] = wm[w][s] == -INFINITY ? 0.f : El<E>::ex(wm[w][s] - M);
      L += c[w] * wl[w][s];
    }
    if (used == 1 && p.sink) L += El<E>::ex(p.sink[h0 + min(s, nh - 1)] - M);
    for (int i = lane; i < Vd; i += 64) {
      float o = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) o += c[w] * merged[(w * RB + s) * Vd + i];
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
    // weights of the splits first (a wave per head), then every thread sums outputs, UZ splits' loads in flight
    const float* base = p.ws + blk * p.nsplit * stride;
    __shared__ float wz[RB][MAX_SPLITS];
    for (int s = wv; s < RB; s += 4) {
      const float* b = base + s * (Vd + 2);
      float M = -INFINITY, L = 0.f;
      for (int z = lane; z < used; z += 64) M = fmaxf(M, b[(long long)z * stride]);
      M = wave_max(M);
      for (int z = lane; z < used; z += 64) {
        const float c = El<E>::ex(b[(long long)z * stride] - M);
        wz[s][z] = c;
        L += c * b[(long long)z * stride + 1];
      }
      L = wave_sum(L);
      if (p.sink) L += El<E>::ex(p.sink[h0 + min(s, nh - 1)] - M);
      L = 1.f / L;
      for (int z = lane; z < used; z += 64) wz[s][z] *= L;
    }
    __syncthreads();
    constexpr int UZ = 16;
    for (int i = tid; i < RB * Vd; i += 256) {
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
  E* orow = reinterpret_cast<E*>(p.out) + row * p.ldo + (long long)h0 * Vd;
  const E* gr = xr + p.o_g + h0 * Vd;
  for (int i = tid; i < nh * Vd; i += 256)
    El<E>::st(orow + i, POOL ? merged[i] * p.mul : p.o_g >= 0 ? merged[i] * gate_of<E>(El<E>::ld(gr + i)) : merged[i]);
}

template <typename E, int RB, int LP, bool VEC, bool POOL>
__global__ void __launch_bounds__(256, sizeof(E) == 2 && LP <= 16 ? 4 : 1) biased_rows_kernel(BiasedArgs p) {
  rows_body<E, RB, LP, VEC, POOL>(p, blockIdx.x, blockIdx.y, blockIdx.z, gridDim.y);
}

// ---------------------------------------------------------------------------------------- tile kernel
// 4 waves of 32 queries of one head. 32-key tiles of K | V double buffered in LDS (the image of attn_tile.h)
// beside the head's bias row (BL; longer rows stay in global memory); S^T = K Q^T leaves a query per lane, and
// P^T feeds O^T += V^T P^T from registers. Tiles beyond the last bucket's edge add one constant.
template <int DK, int DV, bool BL, bool POOL>
__global__ void __launch_bounds__(256, DV > 128 ? 1 : 2) biased_tile_kernel(BiasedArgs p) {
  constexpr int BN = 32, TK = BN * DK * 2, TV = BN * DV * 2, BUF = TK + TV;
  constexpr int KS = DK / 16, NB = DV / 32;
  constexpr int CK = BN * (DK / 8), CV = BN * (DV / 8), NC = CK + CV;  // 16-B chunks per tile
  constexpr int CPT = (NC + 255) / 256;
  extern __shared__ __attribute__((aligned(16))) char smem[];  // [2][K | V], bias row
  const int tid = threadIdx.x, lane = tid & 63, qg = tid >> 6;
  const int l32 = lane & 31, hh = lane >> 5, gi = lane & 15;
  // tiles in their order (the longest first) on every XCD; one with an eighth of the heads shares their K / V in its L2
  const int hx = p.H % 8 ? p.H : p.H / 8, j = p.H % 8 ? (int)blockIdx.x : (int)blockIdx.x >> 3;
  const int ti = j / hx, h = j % hx + (p.H % 8 ? 0 : hx * (blockIdx.x & 7)), g = h / (p.H / p.G);
  const int* tl = p.tiles + ti * 4;
  const int row0 = tl[0], nrow = tl[1], pos0 = tl[2], slot = tl[3];
  const int qi = qg * 32 + l32;
  const bool live = qi < nrow;
  const int row = row0 + min(qi, nrow - 1), pos = pos0 + min(qi, nrow - 1);
  const int kv_hi = pos0 + nrow;                       // keys any query of the tile sees
  const int wave_hi = pos0 + min(qg * 32 + 32, nrow);  // ... any query of this wave
  // POOL: tiles of block means [0, nbt), then tiles of tokens from the first that the tile's first query sees
  const int nbm = POOL ? blocks_seen(p, kv_hi - 1) : 0, nbt = (nbm + BN - 1) / BN;
  const int tt0 = POOL ? max(0, pos0 - p.window + 1) / BN - nbt : 0;  // token tile t holds keys (t + tt0) BN ..
  const int ntiles = (kv_hi + BN - 1) / BN - tt0;
  const int seen = POOL ? blocks_seen(p, pos) : 0;                                   // this lane's query
  const int wave_seen = POOL ? blocks_seen(p, wave_hi - 1) : 0, wave_all = POOL ? blocks_seen(p, pos0 + qg * 32) : 0;
  const int wave_lo = POOL ? pos0 + qg * 32 - p.window + 1 : 0;                      // first token its first query sees
  const bool busy = qg * 32 < nrow;
  const int D = p.dim, Vd = p.vdim;
  const int* tbl = p.table + (long long)slot * p.tstride;
  const bf16_t* kc = reinterpret_cast<const bf16_t*>(p.kc);
  const bf16_t* vc = reinterpret_cast<const bf16_t*>(p.vc);
  const bf16_t* xr = reinterpret_cast<const bf16_t*>(p.x) + row * p.ld;

  // this thread's 16-B chunks of a tile: element offset from the tile's first row, LDS offset
  int off[CPT], ldo[CPT], vrow[CPT], col[POOL ? CPT : 1];  // (col: within the row)
  bool on[CPT];
#pragma unroll
  for (int i = 0; i < CPT; ++i) {
    const int c = tid + 256 * i, cv = c - CK;
    const bool key = c < CK;
    const int r = key ? c / (DK / 8) : cv / (DV / 8), ch = key ? c % (DK / 8) : cv % (DV / 8);
    on[i] = c < NC && ch * 8 < (key ? D : Vd);
    off[i] = on[i] ? r * (key ? D : Vd) + ch * 8 : 0;
    if constexpr (POOL) col[i] = on[i] ? ch * 8 : 0;
    ldo[i] = key ? img_off<DK>(r, ch) : TK + img_off<DV>(r, ch);
    vrow[i] = key ? -1 : r;
  }
  struct Pages { int pg, v[POOL ? CPT : 1]; };  // of a tile (of tokens; of block means: of each chunk's row)
  auto end_of = [&](int t, int i) {          // last position of the block in chunk i's row
    const int c = tid + 256 * i, r = c < CK ? c / (DK / 8) : min(c - CK, CV - 1) / (DV / 8);
    return min(t * BN + r, nbm - 1) * p.pool + p.pool - 1;
  };
  auto page = [&](int tn) {
    Pages r;
    const int t = min(tn, ntiles - 1);
    if (POOL && t < nbt) {
#pragma unroll
      for (int i = 0; i < CPT; ++i) r.v[POOL ? i : 0] = tbl[end_of(t, i) >> p.shift];
    } else {
      r.pg = tbl[(t + tt0) * BN >> p.shift];
    }
    return r;
  };
  auto load = [&](int tn, const Pages& pgs, u32x4 (&st)[CPT]) {  // tile t of these pages (tiles past the end: the last again)
    const int t = min(tn, ntiles - 1);
    if (POOL && t < nbt) {
#pragma unroll
      for (int i = 0; i < CPT; ++i) {
        const bool key = 256 * i + 255 < CK || (256 * i < CK && tid + 256 * i < CK);
        const long long in = (long long)g * p.per + block_row(p, end_of(t, i));
        const bf16_t* base = key ? reinterpret_cast<const bf16_t*>(p.kb) + pgs.v[POOL ? i : 0] * p.kb_sp + in * D
                                 : reinterpret_cast<const bf16_t*>(p.vb) + pgs.v[POOL ? i : 0] * p.vb_sp + in * Vd;
        const u32x4 v = *reinterpret_cast<const u32x4*>(base + col[POOL ? i : 0]);
        st[i] = on[i] && t * BN + vrow[i] < nbm ? v : u32x4{0u, 0u, 0u, 0u};
      }
      return;
    }
    const int pg = pgs.pg, k0 = (t + tt0) * BN;
    const long long o0 = ((long long)g << p.shift) + (k0 & ((1 << p.shift) - 1));
    const bf16_t *kb = kc + pg * p.k_sp + o0 * D, *vb = vc + pg * p.v_sp + o0 * Vd;
#pragma unroll
    for (int i = 0; i < CPT; ++i) {
      const bool key = 256 * i + 255 < CK || (256 * i < CK && tid + 256 * i < CK);
      const u32x4 v = *reinterpret_cast<const u32x4*>((key ? kb : vb) + off[i]);
      st[i] = on[i] && k0 + vrow[i] < kv_hi ? v : u32x4{0u, 0u, 0u, 0u};  // (a value past the last key may be anything)
    }
  };
  auto store = [&](const u32x4 (&st)[CPT], char* buf) {
#pragma unroll
    for (int i = 0; i < CPT; ++i)
      if (256 * i + 255 < NC || tid + 256 * i < NC) *reinterpret_cast<u32x4*>(buf + ldo[i]) = st[i];
  };
  u32x4 st0[CPT], st1[CPT];
  load(0, page(0), st0);
  Pages pg = page(1);
  // the bias row in units of log2
  const float* gb = !POOL && p.bias ? p.bias + (long long)h * p.nb : nullptr;
  float* lb = reinterpret_cast<float*>(smem + 2 * BUF);
  if constexpr (BL)
    for (int i = tid; i < p.nb; i += 256) lb[i] = gb[i] * kLog2e;
  const float far = gb ? gb[p.nb - 1] * kLog2e : 0.f;
  // queries: normed in fp32, rounded once
  bf16x8 qf[KS];
  {
    U16x8 raw[KS];
    float ss = 0.f;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int c = 16 * s + 8 * hh;
      u32x4 v = {0u, 0u, 0u, 0u};
      if (c < D) v = *reinterpret_cast<const u32x4*>(xr + p.o_q + h * D + c);
      raw[s] = __builtin_bit_cast(U16x8, v);
#pragma unroll
      for (int e = 0; e < 8; ++e) ss = fmaf(bf2f(raw[s].v[e]), bf2f(raw[s].v[e]), ss);
    }
    if (!POOL && p.qn) {
      ss += __shfl_xor(ss, 32, 64);
      const float n = 1.f / sqrtf(ss / (float)D + p.eps);
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const int c = 16 * s + 8 * hh;
        float w[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) w[e] = 0.f;
        if (c < D) load8(reinterpret_cast<const bf16_t*>(p.qn) + c, w);
#pragma unroll
        for (int e = 0; e < 8; ++e) raw[s].v[e] = f2bf(bf2f(raw[s].v[e]) * n * w[e]);
      }
    }
#pragma unroll
    for (int s = 0; s < KS; ++s) qf[s] = __builtin_bit_cast(bf16x8, raw[s]);
  }
  const float sl2 = p.scale * kLog2e;

  const int xs = (l32 >> 2) & 3;
  const int kb_e = (l32 >> 3) * 16 * DK + 64 * (l32 & 7) + 16 * (hh ^ xs);
  const int kb_o = (l32 >> 3) * 16 * DK + 64 * (l32 & 7) + 16 * ((2 + hh) ^ xs);
  const int c3 = 2 * ((lane >> 4) & 1) + ((gi & 3) >> 1);
  const int vb_1 = TK + 64 * (4 * hh + (gi >> 2)) + 16 * (c3 ^ hh) + 8 * (gi & 1);
  const int vb_2 = TK + 16 * DV + 64 * (4 * hh + (gi >> 2)) + 16 * (c3 ^ hh ^ 2) + 8 * (gi & 1);

  f32x16 o[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int r = 0; r < 16; ++r) o[b][r] = 0.f;
  float mref = POOL ? -1e30f : -INFINITY, ls = 0.f;  // (POOL: a query may see nothing of the first tiles)

  store(st0, smem);
  load(1, pg, st0);
  pg = page(2);
  __syncthreads();
  // tile t; its successor lies in `next`, the one after that is loaded into `far2` meanwhile
  auto step = [&](int t, const u32x4 (&next)[CPT], u32x4 (&far2)[CPT]) {
    const char* buf = smem + (t & 1) * BUF;
    const bool mean = POOL && t < nbt;
    const int k0 = (mean ? t : t + tt0) * BN;
    load(t + 2, pg, far2);
    pg = page(t + 3);
    // (tiles past the wave's last query, or before its first query's window: staging only)
    if (busy && k0 < (mean ? wave_seen : wave_hi) && (!POOL || mean || k0 + BN > wave_lo)) {
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
      // s[r]: key k0 + (r & 3) + 8 (r >> 2) + 4 hh of this lane's query; log2 of its weight is s a + c
      float a = sl2, c = far;
      const int d0 = pos - k0 - 4 * hh;  // distance of key r = 0
      const bool near = gb && pos0 + qg * 32 - (k0 + BN - 1) < p.nb - 1;
      if (near || !(sl2 > 0.f)) {
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          float bias = 0.f;
          if (gb) {
            const int n = min(max(d0 - ((r & 3) + 8 * (r >> 2)), 0), p.nb - 1);
            if constexpr (BL) bias = lb[n];
            else bias = gb[n] * kLog2e;
          }
          s[r] = fmaf(s[r], sl2, bias);
        }
        a = 1.f;
        c = 0.f;
      }
      if constexpr (POOL) {
        if (mean ? k0 + BN > wave_all : (k0 + BN > pos0 + qg * 32 || k0 < wave_hi - p.window)) {
          const int hi = mean ? seen - k0 - 4 * hh : d0 + 1, lo = mean ? 0 : d0 + 1 - p.window;  // keys [lo, hi) of r
#pragma unroll
          for (int r = 0; r < 16; ++r)
            if ((r & 3) + 8 * (r >> 2) >= hi || (r & 3) + 8 * (r >> 2) < lo) s[r] = -INFINITY;
        }
      } else if (k0 + BN > pos0 + qg * 32) {
#pragma unroll
        for (int r = 0; r < 16; ++r)
          if ((r & 3) + 8 * (r >> 2) > d0) s[r] = -INFINITY;
      }
      float mt = s[0];
#pragma unroll
      for (int r = 1; r < 16; ++r) mt = fmaxf(mt, s[r]);
      mt = fmaf(fmaxf(mt, __shfl_xor(mt, 32, 64)), a, c);
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
      const float off = c - mref;
      float sum = 0.f;
      uint32_t u[8];
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float w0 = __builtin_amdgcn_exp2f(fmaf(s[2 * i], a, off));
        const float w1 = __builtin_amdgcn_exp2f(fmaf(s[2 * i + 1], a, off));
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
    store(next, smem + ((t + 1) & 1) * BUF);
    __syncthreads();
  };
  for (int t = 0; t < ntiles; t += 2) {
    step(t, st0, st1);
    if (t + 1 < ntiles) step(t + 1, st1, st0);
  }
  if (!live) return;
  float l = ls + __shfl_xor(ls, 32, 64);
  if (p.sink) l += __builtin_amdgcn_exp2f(fmaf(p.sink[h], kLog2e, -mref));
  const float n = POOL ? p.mul / l : 1.f / l;
  bf16_t* orow = reinterpret_cast<bf16_t*>(p.out) + row * p.ldo + h * Vd;
  const bf16_t* gr = xr + p.o_g + h * Vd;
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int q4 = 0; q4 < 4; ++q4) {
      const int c = 32 * b + 8 * q4 + 4 * hh;
      if (c < Vd) {
        float y[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = o[b][4 * q4 + e] * n;
        if (!POOL && p.o_g >= 0) {
          const U16x4 z = *reinterpret_cast<const U16x4*>(gr + c);
#pragma unroll
          for (int e = 0; e < 4; ++e) y[e] *= gate_of<bf16_t>(bf2f(z.v[e]));
        }
        *reinterpret_cast<uint2*>(orow + c) = make_uint2(pk_bf16(y[0], y[1]), pk_bf16(y[2], y[3]));
      }
    }
}

template <bool POOL>
size_t rows_lds(const BiasedArgs& p, int rb) {
  return ((size_t)4 * rb * p.vdim + (POOL ? pool_lds(rb, p.dim, p.rot) : 0)) * 4;
}

template <typename E, int RB, int LP, bool VEC, bool POOL>
int rows_go(const BiasedArgs& p, int rows, hipStream_t s) {
  const int Hg = p.H / p.G, nsub = (Hg + RB - 1) / RB;
  const size_t lds = rows_lds<POOL>(p, RB);
  hipLaunchKernelGGL((biased_rows_kernel<E, RB, LP, VEC, POOL>), dim3(rows, p.G * nsub, p.nsplit), dim3(256), lds, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

static int rb_for(int Hg, bool vec) { return vec && Hg > 1 ? 4 : 1; }

template <typename E, bool POOL>
int rows_dispatch(const BiasedArgs& p, int rows, bool vec, hipStream_t s) {
  const int lp = lanes_for(p.dim > p.vdim ? p.dim : p.vdim);
  if (lp > 64) return 10;
  if (!vec) return rows_go<E, 1, 64, false, POOL>(p, rows, s);
  const bool r4 = rb_for(p.H / p.G, vec) == 4;
#define R2(A) (r4 ? rows_go<E, 4, A, true, POOL>(p, rows, s) : rows_go<E, 1, A, true, POOL>(p, rows, s))
  if (lp == 8) return R2(8);
  if (lp == 16) return R2(16);
  if (lp == 32) return R2(32);
  return R2(64);
#undef R2
}

constexpr int MAX_LDS_BIAS = 8192;  // longest bias row that is staged

template <int DK, int DV, bool POOL>
int tile_go(const BiasedArgs& p, int ntiles, hipStream_t s) {
  const bool bl = p.bias && p.nb <= MAX_LDS_BIAS;
  const int lds = 2 * (32 * DK * 2 + 32 * DV * 2) + (bl ? p.nb * 4 : 0);
  auto kern = biased_tile_kernel<DK, DV, false, POOL>;
  if constexpr (!POOL)
    if (bl) kern = biased_tile_kernel<DK, DV, true, false>;
  if (lds > 48 * 1024)
    if (hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess) return 5;
  hipLaunchKernelGGL(kern, dim3(ntiles * p.H), dim3(256), lds, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

template <int DK, bool POOL>
int tile_dv(const BiasedArgs& p, int ntiles, hipStream_t s) {
  if (p.vdim <= 64) return tile_go<DK, 64, POOL>(p, ntiles, s);
  if (p.vdim <= 96) return tile_go<DK, 96, POOL>(p, ntiles, s);
  if (p.vdim <= 128) return tile_go<DK, 128, POOL>(p, ntiles, s);
  return tile_go<DK, 256, POOL>(p, ntiles, s);
}

static bool args_ok(const BiasedArgs& p) {
  const long long ends[4] = {p.o_q + (long long)p.H * p.dim, p.o_k + (long long)p.G * p.dim, p.o_v + (long long)p.G * p.vdim,
                             p.o_g < 0 ? 0 : p.o_g + (long long)p.H * p.vdim};
  for (long long e : ends)
    if (e > p.ld) return false;
  return p.H > 0 && p.G > 0 && p.H % p.G == 0 && p.dim > 0 && p.vdim > 0 && p.shift >= 4 && p.x && p.kc && p.vc && p.table &&
         p.o_q >= 0 && p.o_k >= 0 && p.o_v >= 0 && (!p.bias || p.nb >= 1);
}

static bool vec_ok(const BiasedArgs& p) {
  return p.dim % 8 == 0 && p.vdim % 8 == 0 && p.ld % 8 == 0 && p.o_q % 8 == 0 && p.o_k % 8 == 0 && p.o_v % 8 == 0 &&
         (uintptr_t)p.x % 16 == 0 && (uintptr_t)p.kc % 16 == 0 && (uintptr_t)p.vc % 16 == 0 && p.k_sp % 8 == 0 &&
         p.v_sp % 8 == 0 && (uintptr_t)p.qn % 16 == 0 && (uintptr_t)p.kn % 16 == 0;
}

static bool pool_ok(const BiasedArgs& p) {
  return args_ok(p) && p.window >= 1 && p.pool >= 1 && p.per >= ((1 << p.shift) + p.pool - 1) / p.pool && p.shift <= 10 && p.kb && p.vb &&
         p.pool_mul == (unsigned)(((1 << 20) + p.pool - 1) / p.pool) && p.pool <= (1 << 20) && p.qn && p.kn && p.rot >= 0 &&
         p.rot % 2 == 0 && p.rot <= p.dim && (p.rot == 0 || p.freq) && !p.bias && p.o_g < 0;
}
static bool pool_vec(const BiasedArgs& p) {
  return vec_ok(p) && (uintptr_t)p.kb % 16 == 0 && (uintptr_t)p.vb % 16 == 0 && p.kb_sp % 8 == 0 && p.vb_sp % 8 == 0;
}

// 0: the rows kernel may run. nsplit * chunk must cover the keys of every row (at most max_kv).
static int rows_check(const BiasedArgs& p, int rows, long long ws_floats, long long n_cnt, int max_kv) {
  if (!args_ok(p) || !p.pos || !p.slot || !p.out || rows < 1 || p.nsplit < 1 || p.chunk < 1 || p.nsplit > MAX_SPLITS)
    return 1;
  if ((long long)p.nsplit * p.chunk < max_kv) return 2;
  const int rb = rb_for(p.H / p.G, vec_ok(p)), nsub = (p.H / p.G + rb - 1) / rb;
  if (p.nsplit > 1) {
    const long long blk = (long long)rows * p.G * nsub;
    if (!p.ws || !p.cnt || n_cnt < blk || ws_floats < blk * p.nsplit * rb * (p.vdim + 2)) return 5;
  }
  return 0;
}

// One query token per row.
template <bool POOL>
int rows_entry(const BiasedArgs& p, int dtype, int rows, long long ws_floats, long long n_cnt, int max_kv, hipStream_t s) {
  if (const int rc = rows_check(p, rows, ws_floats, n_cnt, max_kv)) return rc;
  if (dtype == 0) return rows_dispatch<float, POOL>(p, rows, vec_ok(p), s);
  if (dtype == 1) return rows_dispatch<bf16_t, POOL>(p, rows, vec_ok(p), s);
  return 3;
}

// 10: a shape for the rows kernel
template <bool POOL>
int tiles_entry(const BiasedArgs& p, int ntiles, hipStream_t s) {
  if (!args_ok(p) || !p.tiles || !p.out || ntiles < 1) return 1;
  if (!vec_ok(p) || p.dim > 128 || p.vdim > 256 || p.shift < 5 || p.ldo % 4 || (uintptr_t)p.out % 8 ||
      (p.o_g >= 0 && p.o_g % 4))
    return 10;
  if (p.dim <= 32) return tile_dv<32, POOL>(p, ntiles, s);
  if (p.dim <= 64) return tile_dv<64, POOL>(p, ntiles, s);
  if (p.dim <= 96) return tile_dv<96, POOL>(p, ntiles, s);
  return tile_dv<128, POOL>(p, ntiles, s);
}

}  // namespace
