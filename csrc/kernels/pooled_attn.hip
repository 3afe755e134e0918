// Sliding-window attention that sees what lies before its window as block means (biased_attn.h, POOL), behind query and
// key norms over all heads at once and a rotation:
//   q <- R(pos) (q / rms(q) * qn),  k <- R(pos) (k / rms(k) * kn)       rms over the whole projection
//   keys of a query at pos: the tokens (pos - window, pos] and the means of whole blocks that end at or before pos - window
//   o = mul * sum_j w_j v_j / (exp(sink_h) + sum_j w_j),  w_j = exp(q . k_j * scale)
//
//   prep kernel        norms and rotation of every row of a batch: q in place, k and v into their pages
//   mean kernel        means of the blocks that a batch's rows complete, from the pages
//   rows, tile kernels biased_attn.h. A batch of single tokens is one launch of the rows kernel, which norms, rotates,
//                      appends and completes blocks itself (a block that ends at pos is seen from pos + window on).
#include "biased_attn.h"

namespace {

// One row per workgroup. V elements per access (V > 1: head sizes and half the rotated dims are multiples of V).
template <typename E, int V>
__global__ void __launch_bounds__(256) prep_kernel(BiasedArgs p) {
  struct alignas(sizeof(E) * V) Pack { E v[V]; };
  extern __shared__ __attribute__((aligned(16))) char lds[];
  __shared__ float red[2][4];
  const int tid = threadIdx.x, t = blockIdx.x, D = p.dim, nq = p.H * D, nk = p.G * D, nv = p.G * p.vdim, half = p.rot / 2;
  float *cs = reinterpret_cast<float*>(lds), *sn = cs + half;
  E* raw = reinterpret_cast<E*>(lds + ((half * 8 + 15) & ~15));  // q | k as projected
  E* x = reinterpret_cast<E*>(const_cast<void*>(p.x)) + (long long)t * p.ld;
  const int pos = p.pos[t], in_page = pos & ((1 << p.shift) - 1);
  const long long pg = p.table[(long long)p.slot[t] * p.tstride + (pos >> p.shift)];
  float sq = 0.f, sk = 0.f;
  for (int c = tid * V; c < nq + nk; c += 256 * V) {
    const bool key = c >= nq;
    const Pack u = *reinterpret_cast<const Pack*>(x + (key ? p.o_k + c - nq : p.o_q + c));
    *reinterpret_cast<Pack*>(raw + c) = u;
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < V; ++e) s = fmaf(El<E>::ld(u.v + e), El<E>::ld(u.v + e), s);
    if (key) sk += s;
    else sq += s;
  }
  E* vc = reinterpret_cast<E*>(p.vc) + pg * p.v_sp;
  for (int c = tid * V; c < nv; c += 256 * V) {
    const int g = c / p.vdim, e = c - g * p.vdim;
    *reinterpret_cast<Pack*>(vc + (((long long)g << p.shift) + in_page) * p.vdim + e) = *reinterpret_cast<const Pack*>(x + p.o_v + c);
  }
  for (int i = tid; i < half; i += 256) sincosf((float)pos * p.freq[i], sn + i, cs + i);
  auto add = [](float a, float b) { return a + b; };
  sq = lanes_reduce<64>(sq, add);
  sk = lanes_reduce<64>(sk, add);
  if ((tid & 63) == 0) red[0][tid >> 6] = sq, red[1][tid >> 6] = sk;
  __syncthreads();
  const float rq = 1.f / sqrtf((red[0][0] + red[0][1] + red[0][2] + red[0][3]) / (float)nq + p.eps);
  const float rk = 1.f / sqrtf((red[1][0] + red[1][1] + red[1][2] + red[1][3]) / (float)nk + p.eps);
  E* kc = reinterpret_cast<E*>(p.kc) + pg * p.k_sp;
  for (int c = tid * V; c < nq + nk; c += 256 * V) {
    const bool key = c >= nq;
    const int c0 = key ? c - nq : c, hd = c0 / D, e0 = c0 - hd * D;  // (V elements of one head, on one side of its halves)
    const E* gain = reinterpret_cast<const E*>(key ? p.kn : p.qn) + c0;
    const int other = e0 >= 2 * half ? 0 : e0 < half ? half : -half;
    const Pack a = *reinterpret_cast<const Pack*>(raw + c), b = *reinterpret_cast<const Pack*>(raw + c + other);
    const Pack ga = *reinterpret_cast<const Pack*>(gain), gb = *reinterpret_cast<const Pack*>(gain + other);
    const float n = key ? rk : rq, sign = e0 < half ? -1.f : 1.f;
    const int f0 = e0 < half ? e0 : e0 - half;
    Pack y;
#pragma unroll
    for (int e = 0; e < V; ++e) {
      float u = El<E>::ld(a.v + e) * n * El<E>::ld(ga.v + e);
      if (other) u = u * cs[f0 + e] + sign * (El<E>::ld(b.v + e) * n * El<E>::ld(gb.v + e)) * sn[f0 + e];
      El<E>::st(y.v + e, u);
    }
    *reinterpret_cast<Pack*>(key ? kc + (((long long)hd << p.shift) + in_page) * D + e0 : x + p.o_q + c0) = y;
  }
}

// 16 rows per workgroup: every row that completes a block, all heads' means
constexpr int MEAN_ROWS = 16;
template <typename E, int V>
__global__ void __launch_bounds__(256) mean_kernel(BiasedArgs p, int T) {
  struct alignas(sizeof(E) * V) Pack { E v[V]; };
  const int D = p.dim, nk = p.G * D, n = nk + p.G * p.vdim, pmask = (1 << p.shift) - 1;
  for (int t = blockIdx.x * MEAN_ROWS; t < min(T, (int)(blockIdx.x + 1) * MEAN_ROWS); ++t) {
    const int pos = p.pos[t];
    if ((pos + 1) % p.pool) continue;
    const int* tbl = p.table + (long long)p.slot[t] * p.tstride;
    for (int c = threadIdx.x * V; c < n; c += 256 * V) {
      const bool key = c < nk;
      const int c0 = key ? c : c - nk, sz = key ? D : p.vdim, g = c0 / sz, e0 = c0 - g * sz;
      const E* src = reinterpret_cast<const E*>(key ? p.kc : p.vc) + e0;
      const long long sp = key ? p.k_sp : p.v_sp;
      float s[V];
#pragma unroll
      for (int e = 0; e < V; ++e) s[e] = 0.f;
#pragma unroll 4
      for (int j = p.pool - 1; j >= 0; --j) {
        const int at = pos - j;
        const Pack u = *reinterpret_cast<const Pack*>(src + tbl[at >> p.shift] * sp + (((long long)g << p.shift) + (at & pmask)) * sz);
#pragma unroll
        for (int e = 0; e < V; ++e) s[e] += El<E>::ld(u.v + e);
      }
      Pack y;
#pragma unroll
      for (int e = 0; e < V; ++e) El<E>::st(y.v + e, s[e] / (float)p.pool);
      const long long pg = tbl[pos >> p.shift];
      E* dst = key ? reinterpret_cast<E*>(p.kb) + pg * p.kb_sp : reinterpret_cast<E*>(p.vb) + pg * p.vb_sp;
      *reinterpret_cast<Pack*>(dst + ((long long)g * p.per + block_row(p, pos)) * sz + e0) = y;
    }
  }
}

template <typename E, int V>
int prep_go(const BiasedArgs& p, int T, hipStream_t s) {
  const int lds = ((p.rot * 4 + 15) & ~15) + (p.H + p.G) * p.dim * (int)sizeof(E);
  auto kern = prep_kernel<E, V>;
  if (lds > 160 * 1024 - 256) return 10;
  if (lds > 48 * 1024 && hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, lds) != hipSuccess) return 5;
  hipLaunchKernelGGL(kern, dim3(T), dim3(256), lds, s, p);
  if (hipGetLastError() != hipSuccess) return 4;
  hipLaunchKernelGGL((mean_kernel<E, V>), dim3((T + MEAN_ROWS - 1) / MEAN_ROWS), dim3(256), 0, s, p, T);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

}  // namespace

// Mirrored by ops/biased_attention.py
KCA_API int kca_pooled_attn_abi() { return (int)sizeof(BiasedArgs); }

// Queries of T rows in place, their K / V into the pages, and the means of the blocks they complete
KCA_API int kca_pooled_prep(const BiasedArgs* in, int dtype, int T, hipStream_t s) {
  const BiasedArgs& p = *in;
  if (!pool_ok(p) || !p.pos || !p.slot || T < 1) return 1;
  const bool vec = pool_vec(p) && (p.rot / 2) % 8 == 0;
  if (dtype == 0) return vec ? prep_go<float, 4>(p, T, s) : prep_go<float, 1>(p, T, s);
  if (dtype == 1) return vec ? prep_go<bf16_t, 8>(p, T, s) : prep_go<bf16_t, 1>(p, T, s);
  return 3;
}

KCA_API int kca_pooled_rows(const BiasedArgs* in, int dtype, int rows, long long ws_floats, long long n_cnt, int max_kv, hipStream_t s) {
  if (!pool_ok(*in) || (vec_ok(*in) && !pool_vec(*in))) return 1;
  return rows_entry<true>(*in, dtype, rows, ws_floats, n_cnt, max_kv, s);
}

KCA_API int kca_pooled_tiles(const BiasedArgs* in, int ntiles, hipStream_t s) {
  if (!pool_ok(*in) || !pool_vec(*in)) return 1;
  return tiles_entry<true>(*in, ntiles, s);
}
