// Mixture of gated experts: router, grouping, expert products.
//
//   s = sigmoid(W_router h); the `top` experts with the largest scores take the token, with weight s;  or
//   s = softmax(W_router h); the `top` experts with the largest s + correction, out of the `keep` of `groups` equal groups
//   of neighbours whose largest such score is largest, with weight s / (their sum + 1e-20). The last `identity` of the
//   outputs have no weights: they pass the token on (norm_residual.hip adds it), and no expert row is made for them.
//   expert(x) = W_down (silu(W_gate x) * (W_up x))
// A weight scales the expert's input -- both first products are linear, so it multiplies their fp32 sums
// before the activation -- or its output (`scale_in` 0). The router (and the shared expert's gate, one
// more row) accumulates in fp32 and is never rounded.
//
//   route   scores, top-k, weights of each token (bf16: matrix cores, 16 tokens per workgroup)
//   group   assignments sorted by expert and cut in row tiles that hold one expert each
//   gemv    expert products of tiles of up to 8 rows: streams the weight rows on the vector units
//           (decode; any dims, fp32 too)
//   gemm    expert products of tiles of up to 128 rows on the matrix cores (prompts)
// Expert weights are stacked: gate-and-up [E][2F][d] (gate rows first), down [E][d][F]. The sorted rows'
// activations are [n][F], their outputs [n][d]; the residual pass (rms_shift.hip) sums a token's outputs
// through `inv`.
#include "common.h"
#include "lanes.h"

#include <type_traits>

namespace {

typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));

template <typename E> __device__ __forceinline__ float lde(const E* p);
template <> __device__ __forceinline__ float lde<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float lde<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <typename E> __device__ __forceinline__ void ste(E* p, float v);
template <> __device__ __forceinline__ void ste<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void ste<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }

__device__ __forceinline__ float sigmoid(float x) { return 1.f / (1.f + expf(-x)); }

struct RouteArgs {
  const void* h;       // [T][d]
  const void* wr;      // [E][d]
  const void* wsg;     // [d] shared expert's gate (nullable)
  int* ids;            // [T][top]
  float* wts;          // [T][top]
  float* sg;           // [T]
  int T, d, E, top;    // E: router outputs, identity experts included
  int softmax, groups, keep;
  const float* fix;    // [E] correction of the choice (softmax; nullable)
};

__device__ __forceinline__ void lds_order() {  // one wave's LDS writes before its later reads
  __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
  __builtin_amdgcn_wave_barrier();
  __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// largest of z[0 .. n) over the wave; ties go to the lower index
__device__ __forceinline__ void wave_argmax(const float* z, int n, int lane, float& best, int& bi) {
  best = -INFINITY;
  bi = 0x7fffffff;
  for (int e = lane; e < n; e += 64)
    if (z[e] > best) best = z[e], bi = e;
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ob = __shfl_xor(best, o, 64);
    const int oi = __shfl_xor(bi, o, 64);
    if (ob > best || (ob == best && oi < bi)) best = ob, bi = oi;
  }
  if (bi >= n) bi = 0;  // (no finite score left)
}

// One wave: softmax scores, corrected choice within the best groups. z: logits, c, w: E floats each (LDS).
__device__ __forceinline__ void pick_softmax(const RouteArgs& p, float* z, float* c, float* w, int t, int lane, int* ids_lds) {
  float mx = -INFINITY, sum = 0.f;
  for (int e = lane; e < p.E; e += 64) mx = fmaxf(mx, z[e]);
  mx = wave_max(mx);
  for (int e = lane; e < p.E; e += 64) sum += expf(z[e] - mx);
  sum = 1.f / wave_sum(sum);
  for (int e = lane; e < p.E; e += 64) {
    const float s = expf(z[e] - mx) * sum;
    z[e] = s;
    c[e] = s + (p.fix ? p.fix[e] : 0.f);
  }
  lds_order();
  if (p.keep < p.groups) {
    const int size = p.E / p.groups;
    for (int g = lane; g < p.groups; g += 64) {
      float best = -INFINITY;
      for (int e = g * size; e < (g + 1) * size; ++e) best = fmaxf(best, c[e]);
      w[g] = best;
    }
    lds_order();
    for (int g = lane; g < p.groups; g += 64) {
      int ahead = 0;  // groups before this one
      for (int j = 0; j < p.groups; ++j) ahead += w[j] > w[g] || (w[j] == w[g] && j < g);
      if (ahead >= p.keep)
        for (int e = g * size; e < (g + 1) * size; ++e) c[e] = -INFINITY;
    }
    lds_order();
  }
  float total = 0.f;
  for (int k = 0; k < p.top; ++k) {
    float best;
    int bi;
    wave_argmax(c, p.E, lane, best, bi);
    total += z[bi];
    if (lane == 0) {
      p.ids[(long long)t * p.top + k] = bi;
      if (ids_lds) ids_lds[t * p.top + k] = bi;
      w[k] = z[bi];
      c[bi] = -INFINITY;
    }
    lds_order();
  }
  for (int k = lane; k < p.top; k += 64) p.wts[(long long)t * p.top + k] = w[k] / (total + 1e-20f);
}

__device__ __forceinline__ float lane_of(float v, int j) {
  return __int_as_float(__builtin_amdgcn_readlane(__float_as_int(v), j));
}

// Both rules for up to 64 outputs, one a lane: choices by rank, all at once. (NaN counts as the least; ties go to the
// lower index, so ranks are distinct.)
__device__ __forceinline__ void pick_lanes(const RouteArgs& p, const float* z, float fix, int t, int lane, int* ids_lds) {
  const bool on = lane < p.E;
  float s = on ? z[lane] : -INFINITY, c;
  if (p.softmax) {
    auto add = [](float a, float b) { return a + b; };
    auto big = [](float a, float b) { return fmaxf(a, b); };
    const float mx = lanes_reduce<64>(s, big), e = on ? expf(s - mx) : 0.f;
    s = e / lanes_reduce<64>(e, add);
    c = on ? s + fix : -INFINITY;
    if (c != c) c = -INFINITY;
    if (p.keep < p.groups) {
      const int size = p.E / p.groups, g = lane / size;
      float best = -INFINITY;
      int ahead = 0;  // groups before this lane's
      for (int j = 0; j < size; ++j) best = fmaxf(best, __shfl(c, g * size + j, 64));
      for (int j = 0; j < p.groups; ++j) {
        const float o = lane_of(best, j * size);
        ahead += o > best || (o == best && j < g);
      }
      if (ahead >= p.keep) c = -INFINITY;
    }
  } else {
    c = s != s ? -INFINITY : s;
  }
  int rank = 0;
  for (int j = 0; j < p.E; ++j) {
    const float o = lane_of(c, j);
    rank += o > c || (o == c && j < lane);
  }
  const bool take = on && rank < p.top;
  float w = sigmoid(s);
  if (p.softmax) w = s / (lanes_reduce<64>(take ? s : 0.f, [](float a, float b) { return a + b; }) + 1e-20f);
  if (take) {
    p.ids[(long long)t * p.top + rank] = lane;
    if (ids_lds) ids_lds[t * p.top + rank] = lane;
    p.wts[(long long)t * p.top + rank] = w;
  }
}

// this lane's correction, requested early
__device__ __forceinline__ float lane_fix(const RouteArgs& p, int lane) { return p.fix && p.E <= 64 && lane < p.E ? p.fix[lane] : 0.f; }

// One wave: the top experts of one token from its logits z[E] (LDS; softmax: E floats each at c and w).
__device__ __forceinline__ void pick(const RouteArgs& p, float* z, float* c, float* w, float fix, int t, int lane, int* ids_lds = nullptr) {
  if (p.E <= 64) return pick_lanes(p, z, fix, t, lane, ids_lds);
  if (p.softmax) return pick_softmax(p, z, c, w, t, lane, ids_lds);
  for (int k = 0; k < p.top; ++k) {
    float best;
    int bi;
    wave_argmax(z, p.E, lane, best, bi);
    if (lane == 0) {
      p.ids[(long long)t * p.top + k] = bi;
      if (ids_lds) ids_lds[t * p.top + k] = bi;
      p.wts[(long long)t * p.top + k] = sigmoid(best);
      z[bi] = -INFINITY;
    }
    lds_order();
  }
}

// any dims and type: one token per workgroup, a wave per expert row
template <typename E>
__global__ void __launch_bounds__(256) route_rows_kernel(RouteArgs p) {
  extern __shared__ float z[];  // [E + 1], softmax: [2][E] more
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, t = blockIdx.x;
  const E* h = reinterpret_cast<const E*>(p.h) + (long long)t * p.d;
  const int n = p.E + (p.wsg ? 1 : 0);
  for (int e = wv; e < n; e += 4) {
    const E* w = e < p.E ? reinterpret_cast<const E*>(p.wr) + (long long)e * p.d : reinterpret_cast<const E*>(p.wsg);
    float s = 0.f;
    for (int i = lane; i < p.d; i += 64) s = fmaf(lde<E>(h + i), lde<E>(w + i), s);
    s = wave_sum(s);
    if (lane == 0) z[e] = s;
  }
  __syncthreads();
  if (wv == 0) pick(p, z, z + n, z + n + p.E, lane_fix(p, lane), t, lane);
  if (threadIdx.x == 64 && p.wsg) p.sg[t] = sigmoid(z[p.E]);
}

struct GroupArgs {
  const int* ids;      // [n]; E and beyond: no expert row (inv -1)
  int n, E, mt;
  int *perm, *inv, *tiles, *ntiles;
};

// n assignments -> perm (sorted position -> assignment), inv (assignment -> sorted position), tiles
// [ntiles][5] (expert, first sorted position, rows <= mt, first tile and tile count of the expert) and
// their count. One workgroup of NT threads;
// sh: 3 E + 2 ints.
template <int NT>
__device__ __forceinline__ void group_rows(const GroupArgs& p, int* sh) {
  const int E = p.E, n = p.n, mt = p.mt, tid = threadIdx.x;
  int *cnt = sh, *off = sh + E, *toff = off + E + 1;
  for (int e = tid; e < E; e += NT) cnt[e] = 0;
  __syncthreads();
  for (int i = tid; i < n; i += NT)
    if (p.ids[i] < E) atomicAdd(&cnt[p.ids[i]], 1);
  __syncthreads();
  if (tid < 64) {  // exclusive sums over the experts, 64 at a time
    int co = 0, to = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
      const int e = e0 + tid, c = e < E ? cnt[e] : 0, t = (c + mt - 1) / mt;
      int cs = c, ts = t;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const int a = __shfl_up(cs, o, 64), b = __shfl_up(ts, o, 64);
        if (tid >= o) cs += a, ts += b;
      }
      if (e < E) off[e] = co + cs - c, toff[e] = to + ts - t;
      co += __shfl(cs, 63, 64);
      to += __shfl(ts, 63, 64);
    }
    if (tid == 0) off[E] = co, toff[E] = to, *p.ntiles = to;
  }
  __syncthreads();
  for (int e = tid; e < E; e += NT) {
    const int c = cnt[e];
    for (int j = 0; j * mt < c; ++j) {
      int* t = p.tiles + (toff[e] + j) * 5;
      t[0] = e;
      t[1] = off[e] + j * mt;
      t[2] = min(mt, c - j * mt);
      t[3] = toff[e];
      t[4] = (c + mt - 1) / mt;
    }
    cnt[e] = off[e];
  }
  __syncthreads();
  for (int i = tid; i < n; i += NT) {  // (the order within an expert does not matter: rows are independent)
    const int e = p.ids[i], pos = e < E ? atomicAdd(&cnt[e], 1) : -1;
    if (pos >= 0) p.perm[pos] = i;
    p.inv[i] = pos;
  }
}

__global__ void __launch_bounds__(1024) group_kernel(GroupArgs p) {
  extern __shared__ int sh[];
  group_rows<1024>(p, sh);
}

// bf16: 16 tokens per workgroup, the K range cut over NW waves, 64 experts at a time. GROUP: the launch is
// one workgroup, which also groups its assignments (the decode step)
template <int NW, bool GROUP>
__global__ void __launch_bounds__(NW * 64) route_mfma_kernel(RouteArgs p, GroupArgs gr) {
  // z[16][zs], softmax: two more of them; part[NW][16][64] (then group_rows'), ids
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int n = p.E + (p.wsg ? 1 : 0), zs = (n + 63) / 64 * 64, zr = 16 * zs;
  float *z = lds, *part = lds + (p.softmax ? 3 : 1) * zr;
  int* sids = reinterpret_cast<int*>(part + NW * 1024);  // GROUP: [T * top]
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, r16 = lane & 15, g = lane >> 4;
  const int t0 = blockIdx.x * 16, d = p.d;
  const bf16_t* h = reinterpret_cast<const bf16_t*>(p.h) + (long long)min(t0 + r16, p.T - 1) * d;
  const int nk = (d + 31) / 32;
  const float fix = lane_fix(p, lane);
  for (int e0 = 0; e0 < n; e0 += 64) {
    const bf16_t* w[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int e = min(e0 + 16 * i + r16, n - 1);
      w[i] = e < p.E ? reinterpret_cast<const bf16_t*>(p.wr) + (long long)e * d : reinterpret_cast<const bf16_t*>(p.wsg);
    }
    const int nt = min(4, (n - e0 + 15) / 16);
    f32x4 acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
    auto steps = [&](auto ntc) {
      constexpr int NTC = decltype(ntc)::value, AH = NTC > 2 ? 4 : 8;  // k steps whose loads fly together
      for (int k0 = wv * 2; k0 < nk; k0 += NW * AH) {  // 64 columns at a time: whole cache lines of every row
        u32x4 a[AH][NTC], b[AH];
#pragma unroll
        for (int j = 0; j < AH; ++j) {  // (no load is conditional; columns past d multiply zeros)
          const int c = (k0 + (j & 1) + (j >> 1) * NW * 2) * 32 + g * 8, cc = min(c, d - 8);
          const uint32_t keep = c < d ? ~0u : 0u;
          b[j] = *reinterpret_cast<const u32x4*>(h + cc) & u32x4{keep, keep, keep, keep};
#pragma unroll
          for (int i = 0; i < NTC; ++i) a[j][i] = *reinterpret_cast<const u32x4*>(w[i] + cc);
        }
        asm volatile("" ::: "memory");
#pragma unroll
        for (int j = 0; j < AH; ++j)
#pragma unroll
          for (int i = 0; i < NTC; ++i)
            acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a[j][i]), __builtin_bit_cast(bf16x8, b[j]),
                                                             acc[i], 0, 0, 0);
      }
    };
    if (nt == 1) steps(std::integral_constant<int, 1>{});
    else if (nt == 2) steps(std::integral_constant<int, 2>{});
    else steps(std::integral_constant<int, 4>{});
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) part[(wv * 16 + r16) * 64 + i * 16 + g * 4 + r] = acc[i][r];
    __syncthreads();
    for (int i = tid; i < 1024; i += NW * 64) {
      float s = 0.f;
#pragma unroll
      for (int w8 = 0; w8 < NW; ++w8) s += part[w8 * 1024 + i];
      z[(i >> 6) * zs + e0 + (i & 63)] = s;
    }
  }
  __syncthreads();
  for (int r = wv; r < 16; r += NW) {
    if (t0 + r >= p.T) break;
    if (p.wsg && lane == 0) p.sg[t0 + r] = sigmoid(z[r * zs + p.E]);
    pick(p, z + r * zs, z + zr + r * zs, z + 2 * zr + r * zs, fix, t0 + r, lane, GROUP ? sids : nullptr);
  }
  if constexpr (GROUP) {
    __syncthreads();
    gr.ids = sids;
    group_rows<NW * 64>(gr, reinterpret_cast<int*>(part));
  }
}

struct ExpertArgs {
  const void* x;        // gate-up: [T][K] token rows; down: [n][K] sorted rows
  const void* w;        // [E][2N or N][K]
  void* y;              // [n][N] sorted rows
  const int* perm;
  const float* wts;     // [n] by assignment
  const int* tiles;
  const int* ntiles;
  int top, N, K, up, scale;  // up: gate-and-up (x gathered by token, silu product); scale: the weight applies here
  // gemv: a shared expert beside them, `tokens` rows in order, without a weight (ws null: none)
  const void* xs;       // [tokens][Ks]
  const void* ws;       // [2Ns or Ns][Ks]
  void* ys;             // [tokens][Ns]
  int tokens, Ns, Ks;
};

// ------------------------------------------------------------------------------------------------ gemv
// Workgroup: one tile (<= MT rows of one expert, or of the shared one: the first tiles) x 4 waves, a wave streams two
// weight rows (gate and up of one output, or two outputs); the activation rows of a K chunk are staged in LDS for the four.
template <typename E, int MT, bool VEC>
__global__ void __launch_bounds__(256) expert_gemv_kernel(ExpertArgs p) {
  constexpr int KC = 2048, EPL = 16 / (int)sizeof(E), NL = KC / (64 * EPL);  // elements per lane and load
  extern __shared__ __attribute__((aligned(16))) char raw[];
  E* xs = reinterpret_cast<E*>(raw);  // [MT][KC]
  const int nsh = p.ws ? (p.tokens + MT - 1) / MT : 0;
  const bool sh = (int)blockIdx.y < nsh;
  const int tile = (int)blockIdx.y - nsh, N = sh ? p.Ns : p.N, K = sh ? p.Ks : p.K;
  if ((!sh && tile >= *p.ntiles) || (int)blockIdx.x * (p.up ? 4 : 8) >= N) return;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int* tl = p.tiles + (sh ? 0 : tile) * 5;
  const int ex = sh ? 0 : tl[0], lo = sh ? blockIdx.y * MT : tl[1], nr = sh ? min(MT, p.tokens - lo) : tl[2];
  const int n0 = p.up ? blockIdx.x * 4 + wv : (blockIdx.x * 4 + wv) * 2;
  const int rows = p.up ? 2 * N : N;
  const int ra = min(n0, N - 1), rb = p.up ? N + ra : min(n0 + 1, N - 1);
  const E* w = reinterpret_cast<const E*>(sh ? p.ws : p.w);
  const E* wa = w + ((long long)ex * rows + ra) * K;
  const E* wb = w + ((long long)ex * rows + rb) * K;
  float acc[2][MT];
#pragma unroll
  for (int r = 0; r < MT; ++r) acc[0][r] = acc[1][r] = 0.f;
  for (int k0 = 0; k0 < K; k0 += KC) {
    const int kn = min(KC, K - k0);
    u32x4 va[NL], vb[NL];
    if constexpr (VEC) {
#pragma unroll
      for (int i = 0; i < NL; ++i) {
        const int k = (i * 64 + lane) * EPL;
        if (k < kn) {
          va[i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(wa + k0 + k));
          vb[i] = __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(wb + k0 + k));
        }
      }
    }
    __syncthreads();
    for (int r = 0; r < nr; ++r) {
      const long long src = p.up && !sh ? p.perm[lo + r] / p.top : lo + r;
      const E* x = reinterpret_cast<const E*>(sh ? p.xs : p.x) + src * K + k0;
      if constexpr (VEC) {
        for (int i = tid * EPL; i < kn; i += 256 * EPL)
          *reinterpret_cast<u32x4*>(xs + r * KC + i) = *reinterpret_cast<const u32x4*>(x + i);
      } else {
        for (int i = tid; i < kn; i += 256) xs[r * KC + i] = x[i];
      }
    }
    __syncthreads();
    if constexpr (VEC) {
#pragma unroll
      for (int i = 0; i < NL; ++i) {
        const int k = (i * 64 + lane) * EPL;
        if (k < kn) {
#pragma unroll
          for (int r = 0; r < MT; ++r)
            if (r < nr) {
              const u32x4 x = *reinterpret_cast<const u32x4*>(xs + r * KC + k);
#pragma unroll
              for (int e = 0; e < 4; ++e) {
                if constexpr (sizeof(E) == 2) {
                  acc[0][r] = dot2_acc<0>(va[i][e], x[e], acc[0][r]);
                  acc[1][r] = dot2_acc<0>(vb[i][e], x[e], acc[1][r]);
                } else {
                  acc[0][r] = fmaf(__uint_as_float(va[i][e]), __uint_as_float(x[e]), acc[0][r]);
                  acc[1][r] = fmaf(__uint_as_float(vb[i][e]), __uint_as_float(x[e]), acc[1][r]);
                }
              }
            }
        }
      }
    } else {
      for (int k = lane; k < kn; k += 64) {
        const float a = lde<E>(wa + k0 + k), b = lde<E>(wb + k0 + k);
#pragma unroll
        for (int r = 0; r < MT; ++r)
          if (r < nr) {
            const float x = lde<E>(xs + r * KC + k);
            acc[0][r] = fmaf(a, x, acc[0][r]);
            acc[1][r] = fmaf(b, x, acc[1][r]);
          }
      }
    }
  }
#pragma unroll
  for (int r = 0; r < MT; ++r) {
    if (r >= nr) break;
    float a = wave_sum(acc[0][r]), b = wave_sum(acc[1][r]);
    if (lane) continue;
    if (p.scale && !sh) {
      const float s = p.wts[p.perm[lo + r]];
      a *= s;
      b *= s;
    }
    E* y = reinterpret_cast<E*>(sh ? p.ys : p.y) + (long long)(lo + r) * N;
    if (p.up) {
      if (n0 < N) ste<E>(y + n0, a * sigmoid(a) * b);
    } else {
      if (n0 < N) ste<E>(y + n0, a);
      if (n0 + 1 < N) ste<E>(y + n0 + 1, b);
    }
  }
}

// ------------------------------------------------------------------------------------------------ gemm
// bf16, 128 rows x 256 weight rows x 64 per step, 8 waves of 64 x 64 (32x32x16 tiles); weights are the A
// operand, so a lane holds one activation row and runs of four outputs. up: a workgroup covers 128 gate
// and the matching 128 up rows, each wave 32 of both.
constexpr int GBK = 64, GN = 256, GM = 128, GEMM_LDS = 2 * (GN + GM) * GBK * 2;

template <bool UP>
__global__ void __launch_bounds__(512, 2) expert_gemm_kernel(ExpertArgs p) {
  constexpr int BK = GBK;
  extern __shared__ __attribute__((aligned(16))) bf16_t gl[];  // [2][GN + GM][BK]: weight rows, then activation rows
  bf16_t *const sw[2] = {gl, gl + (GN + GM) * BK}, *const sx[2] = {gl + GN * BK, gl + (2 * GN + GM) * BK};
  // order: an XCD works a contiguous run of (expert, weight block, row tile), so the row tiles that share a
  // weight block are on one XCD at one time
  const int nt = *p.ntiles, nb = (p.N + (UP ? 127 : 255)) / (UP ? 128 : 256);
  if ((int)blockIdx.x >= nt * nb) return;
  const int id = xcd_remap(blockIdx.x, nt * nb);
  const int* t0 = p.tiles + id / nb * 5;
  const int in = id - t0[3] * nb, tile = t0[3] + in % t0[4], bn = in / t0[4];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, l32 = lane & 31, hh = lane >> 5;
  const int wn = wv >> 1, wm = wv & 1;
  const int* tl = p.tiles + tile * 5;
  const int ex = tl[0], lo = tl[1], nr = tl[2], K = p.K, N = p.N;
  const int n0 = bn * (UP ? 128 : 256);
  // staging: thread tid owns 16-B chunk tid % 8 of rows tid / 8 + 64 i
  const int ch = tid & 7, sr = tid >> 3;
  const bf16_t *wp[4], *xp[2];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = sr + 64 * i;
    long long wr;
    if constexpr (UP) wr = (r < 128 ? 0 : N) + min(n0 + (r & 127), N - 1);
    else wr = min(n0 + r, N - 1);
    wp[i] = reinterpret_cast<const bf16_t*>(p.w) + ((long long)ex * (UP ? 2 * N : N) + wr) * K;
  }
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    const int r = sr + 64 * i, xr = lo + min(r, nr - 1);
    const long long src = UP ? p.perm[xr] / p.top : xr;
    xp[i] = reinterpret_cast<const bf16_t*>(p.x) + src * K;
  }
  // Two k steps in flight in registers (a step's products alone do not cover a trip past L2). No load or
  // store of the loop is conditional -- a branch between them would make every wait a full drain: loads
  // past K repeat valid columns, and such columns of the activation are stored as zeros.
  u32x4 ra[2][4], rb[2][2];
  auto load = [&](int t, u32x4 (&rw)[4], u32x4 (&rx)[2]) {
    const int k = min(t * BK + ch * 8, K - 8);
#pragma unroll
    for (int i = 0; i < 4; ++i) rw[i] = *reinterpret_cast<const u32x4*>(wp[i] + k);
#pragma unroll
    for (int i = 0; i < 2; ++i) rx[i] = *reinterpret_cast<const u32x4*>(xp[i] + k);
  };
  const int so = sr * BK + ((ch ^ ((sr >> 1) & 7)) << 3);  // 16 rows x one chunk, or 2 x 8: all 64 banks
  auto store = [&](int t, int b, const u32x4 (&rw)[4], const u32x4 (&rx)[2]) {
    const uint32_t keep = t * BK + ch * 8 < K ? ~0u : 0u;
#pragma unroll
    for (int i = 0; i < 4; ++i) *reinterpret_cast<u32x4*>(sw[b] + so + 64 * i * BK) = rw[i];
#pragma unroll
    for (int i = 0; i < 2; ++i) *reinterpret_cast<u32x4*>(sx[b] + so + 64 * i * BK) = rx[i] & u32x4{keep, keep, keep, keep};
  };
  f32x16 acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 16; ++r) acc[i][j][r] = 0.f;
  int ar[2], br[2];
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    ar[i] = (UP ? i * 128 + wn * 32 : wn * 64 + i * 32) + l32;
    br[i] = wm * 64 + i * 32 + l32;
  }
  const int nk = ((K + BK - 1) / BK + 1) & ~1;  // (an odd count's extra step multiplies zeros)
  const bool live = __builtin_amdgcn_readfirstlane(wm) * 64 < nr;
  // step t: LDS buffer t & 1 holds it, register set (t + 1) & 1 the next, the other set is requested
  auto step = [&](int t, auto par) {
    constexpr int b = decltype(par)::value;
    load(t + 2, ra[b], rb[b]);
    asm volatile("" ::: "memory");
    if (live) {
      bf16x8 a[2][2], x[2][2];
      auto frag = [&](int s, int f) {
#pragma unroll
        for (int i = 0; i < 2; ++i) {
          a[f][i] = *reinterpret_cast<const bf16x8*>(sw[b] + ar[i] * BK + (((2 * s + hh) ^ ((ar[i] >> 1) & 7)) << 3));
          x[f][i] = *reinterpret_cast<const bf16x8*>(sx[b] + br[i] * BK + (((2 * s + hh) ^ ((br[i] >> 1) & 7)) << 3));
        }
      };
      frag(0, 0);
      __builtin_amdgcn_sched_group_barrier(0x100, 4, 0);
#pragma unroll
      for (int s = 0; s < BK / 16; ++s) {  // fragments one sub-step ahead of their products
        if (s + 1 < BK / 16) {
          frag(s + 1, (s + 1) & 1);
          __builtin_amdgcn_sched_group_barrier(0x100, 4, 0);
        }
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
          for (int j = 0; j < 2; ++j)
            acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(a[s & 1][i], x[s & 1][j], acc[i][j], 0, 0, 0);
        __builtin_amdgcn_sched_group_barrier(0x8, 4, 0);
      }
    }
    asm volatile("" ::: "memory");
    store(t + 1, b ^ 1, ra[b ^ 1], rb[b ^ 1]);
    __syncthreads();
  };
  load(0, ra[0], rb[0]);
  store(0, 0, ra[0], rb[0]);
  load(1, ra[1], rb[1]);
  __syncthreads();
  for (int t = 0; t < nk; t += 2) {
    step(t, std::integral_constant<int, 0>{});
    step(t + 1, std::integral_constant<int, 1>{});
  }
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int r = br[j];
    if (r >= nr) continue;
    const float s = p.scale ? p.wts[p.perm[lo + r]] : 1.f;
    bf16_t* y = reinterpret_cast<bf16_t*>(p.y) + (long long)(lo + r) * N;
#pragma unroll
    for (int i = 0; i < (UP ? 1 : 2); ++i)
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int n = n0 + (UP ? wn * 32 : wn * 64 + i * 32) + 8 * q + 4 * hh;
        if (n >= N) continue;  // (N % 4 == 0)
        float o[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          if constexpr (UP) {
            const float gt = acc[0][j][4 * q + e] * s, up = acc[1][j][4 * q + e] * s;
            o[e] = gt * __builtin_amdgcn_rcpf(1.f + __expf(-gt)) * up;
          } else {
            o[e] = acc[i][j][4 * q + e] * s;
          }
        }
        *reinterpret_cast<uint2*>(y + n) = make_uint2(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]));
      }
  }
}

template <typename E, bool VEC>
int gemv_go(const ExpertArgs& a, int mt, int max_tiles, hipStream_t s) {
  const int n = a.ws && a.Ns > a.N ? a.Ns : a.N;
  const dim3 g((n + (a.up ? 4 : 8) - 1) / (a.up ? 4 : 8), max_tiles + (a.ws ? (a.tokens + mt - 1) / mt : 0));
#define GO(M)                                                                                                  \
  do {                                                                                                         \
    constexpr int lds = M * 2048 * (int)sizeof(E);                                                             \
    auto kern = expert_gemv_kernel<E, M, VEC>;                                                                 \
    if (lds > 48 * 1024 &&                                                                                     \
        hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess) \
      return 5;                                                                                                \
    hipLaunchKernelGGL(kern, g, dim3(256), lds, s, a);                                                         \
  } while (0)
  if (mt == 1) GO(1);
  else if (mt == 2) GO(2);
  else if (mt == 4) GO(4);
  else if (mt == 8) GO(8);
  else return 6;
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

bool al16(const void* p) { return (uintptr_t)p % 16 == 0; }

template <int NW, bool GROUP>
int route_lds(const RouteArgs& a) {
  const int zs = (a.E + (a.wsg ? 1 : 0) + 63) / 64 * 64;
  return ((a.softmax ? 3 : 1) * 16 * zs + NW * 1024 + (GROUP ? a.T * a.top : 0)) * 4;
}
constexpr int MAX_LDS = 160 * 1024;

// softmax routers: equal groups, enough experts in the kept ones
bool route_ok(const RouteArgs& a) {
  return a.T >= 1 && a.d >= 1 && a.E >= 1 && a.E <= 1024 && a.top >= 1 && a.top <= a.E && a.h && a.wr && a.ids && a.wts && (!a.wsg || a.sg) &&
         (!a.softmax || (a.groups >= 1 && a.E % a.groups == 0 && a.keep >= 1 && a.keep <= a.groups && a.top <= a.E / a.groups * a.keep));
}

template <int NW, bool GROUP>
int route_go(const RouteArgs& a, const GroupArgs& g, hipStream_t s) {
  const int lds = route_lds<NW, GROUP>(a);
  auto kern = route_mfma_kernel<NW, GROUP>;
  if (lds > 48 * 1024 && hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess)
    return 5;
  hipLaunchKernelGGL(kern, dim3((a.T + 15) / 16), dim3(NW * 64), lds, s, a, g);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

}  // namespace

// dtype: 0 fp32, 1 bf16
KCA_API int kca_moe_route(int dtype, const void* h, const void* wr, const void* wsg, void* ids, void* wts, void* sg,
                          int T, int d, int E, int top, int softmax, const void* fix, int groups, int keep, hipStream_t s) {
  const RouteArgs a{h, wr, wsg, (int*)ids, (float*)wts, (float*)sg, T, d, E, top, softmax, groups, keep, (const float*)fix};
  if (!route_ok(a)) return 1;
  if (dtype == 1 && d % 8 == 0 && al16(h) && al16(wr) && al16(wsg)) {
    if (T <= 1024 && route_lds<16, false>(a) <= MAX_LDS) return route_go<16, false>(a, GroupArgs{}, s);
    if (route_lds<8, false>(a) <= MAX_LDS) return route_go<8, false>(a, GroupArgs{}, s);
  }
  const int lds = ((softmax ? 3 : 1) * E + 1) * 4;
  if (dtype == 1) hipLaunchKernelGGL(route_rows_kernel<bf16_t>, dim3(T), dim3(256), lds, s, a);
  else if (dtype == 0) hipLaunchKernelGGL(route_rows_kernel<float>, dim3(T), dim3(256), lds, s, a);
  else return 3;
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

static bool group_ok(const GroupArgs& g, int max_tiles) {
  return g.n >= 1 && g.E >= 1 && g.E <= 1024 && g.mt >= 1 && g.ids && g.perm && g.inv && g.tiles && g.ntiles &&
         max_tiles >= (g.E < g.n ? g.E : g.n) + g.n / g.mt;
}

// tiles: [max_tiles][5] with max_tiles >= min(E, n) + n / mt
KCA_API int kca_moe_group(const void* ids, int n, int E, int mt, void* perm, void* inv, void* tiles, int max_tiles,
                          void* ntiles, hipStream_t s) {
  const GroupArgs g{(const int*)ids, n, E, mt, (int*)perm, (int*)inv, (int*)tiles, (int*)ntiles};
  if (!group_ok(g, max_tiles)) return 1;
  hipLaunchKernelGGL(group_kernel, dim3(1), dim3(1024), (3 * E + 2) * 4, s, g);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

// Both in one launch: bf16, at most 16 tokens (10: shape outside it). E: router outputs, the first `real` with weights
KCA_API int kca_moe_route_group(const void* h, const void* wr, const void* wsg, void* ids, void* wts, void* sg, int T,
                                int d, int E, int real, int top, int softmax, const void* fix, int groups, int keep, int mt, void* perm,
                                void* inv, void* tiles, int max_tiles, void* ntiles, hipStream_t s) {
  const RouteArgs a{h, wr, wsg, (int*)ids, (float*)wts, (float*)sg, T, d, E, top, softmax, groups, keep, (const float*)fix};
  if (!route_ok(a) || real < 1 || real > E) return 1;
  if (T > 16 || top > 64 || d % 8 || !al16(h) || !al16(wr) || !al16(wsg) || route_lds<16, true>(a) > MAX_LDS) return 10;
  const GroupArgs g{(const int*)ids, T * top, real, mt, (int*)perm, (int*)inv, (int*)tiles, (int*)ntiles};
  if (!group_ok(g, max_tiles)) return 1;
  return route_go<16, true>(a, g, s);
}

// One expert product of every tile. mt: the tiles' row limit (1, 2, 4, 8: gemv; 128: gemm, bf16 with
// K % 8 == 0 and N % 4 == 0). ws: a shared expert's product over all tokens beside them (gemv; nullable).
KCA_API int kca_moe_expert(int dtype, const void* x, const void* w, void* y, const void* perm, const void* wts,
                           const void* tiles, const void* ntiles, int max_tiles, int mt, int top, int N, int K, int up,
                           int scale, const void* xs, const void* ws, void* ys, int tokens, int Ns, int Ks, hipStream_t s) {
  if (max_tiles < 1 || max_tiles > 32767 || N < 1 || K < 1 || top < 1 || !x || !w || !y || !perm || !wts || !tiles || !ntiles) return 1;
  if (ws && (!xs || !ys || tokens < 1 || tokens > 32767 || Ns < 1 || Ks < 1 || mt == 128)) return 1;
  const ExpertArgs a{x, w, y, (const int*)perm, (const float*)wts, (const int*)tiles, (const int*)ntiles, top, N, K, up, scale,
                     xs, ws, ys, tokens, Ns, Ks};
  if (mt == 128) {
    if (dtype != 1 || K % 8 || N % 4 || !al16(x) || !al16(w) || (uintptr_t)y % 8) return 10;
    const void* kern = up ? (const void*)expert_gemm_kernel<true> : (const void*)expert_gemm_kernel<false>;
    if (hipFuncSetAttribute(kern, hipFuncAttributeMaxDynamicSharedMemorySize, GEMM_LDS) != hipSuccess) return 5;
    if (up) hipLaunchKernelGGL(expert_gemm_kernel<true>, dim3((N + 127) / 128 * max_tiles), dim3(512), GEMM_LDS, s, a);
    else hipLaunchKernelGGL(expert_gemm_kernel<false>, dim3((N + 255) / 256 * max_tiles), dim3(512), GEMM_LDS, s, a);
    return hipGetLastError() == hipSuccess ? 0 : 4;
  }
  const int v = dtype == 1 ? 8 : 4;
  const bool vec = K % v == 0 && al16(x) && al16(w) && (!ws || (Ks % v == 0 && al16(xs) && al16(ws)));
  if (dtype == 0) return vec ? gemv_go<float, true>(a, mt, max_tiles, s) : gemv_go<float, false>(a, mt, max_tiles, s);
  if (dtype == 1) return vec ? gemv_go<bf16_t, true>(a, mt, max_tiles, s) : gemv_go<bf16_t, false>(a, mt, max_tiles, s);
  return 3;
}
