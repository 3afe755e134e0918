// Causal attention over the paged cache with a bias by distance, a sink and an output gate:
//   q <- N(q; qn), k <- N(k; kn)                      RMS norms per head (optional)
//   w_j = exp(q . k_j * scale + bias[h][min(pos - j, nb - 1)])
//   o = sum_j w_j v_j / (exp(sink_h) + sum_j w_j) * sigmoid(g)
// Query heads share key / value heads in groups. K pages [G][PS][dim] hold normed keys, V pages [G][PS][vdim].
// q / k / v / g are column blocks of one projection buffer. Norms, scores, weights and the gate are fp32.
//
//   append kernel      K (normed) / V of new tokens into their pages
//   rows, tile kernels biased_attn.h
#include "biased_attn.h"

namespace {

// V elements per access (V > 1: head sizes, rows and pools are multiples of V); NL lanes per (token, head)
template <typename E, int V, int NL>
__global__ void __launch_bounds__(256) append_kernel(BiasedArgs p, int T) {
  struct alignas(sizeof(E) * V) Pack { E v[V]; };
  const int i = (int)(((long long)blockIdx.x * 256 + threadIdx.x) / NL), lane = threadIdx.x % NL;
  if (i >= T * 2 * p.G) return;  // (whole groups of NL lanes)
  const int t = i / (2 * p.G), hd = i - t * 2 * p.G;
  const bool key = hd < p.G;
  const int g = key ? hd : hd - p.G, sz = key ? p.dim : p.vdim;
  const int ps = p.pos[t], in_page = ps & ((1 << p.shift) - 1);
  const long long pg = p.table[(long long)p.slot[t] * p.tstride + (ps >> p.shift)];
  const E* src = reinterpret_cast<const E*>(p.x) + (long long)t * p.ld + (key ? p.o_k : p.o_v) + g * sz;
  E* dst = (key ? reinterpret_cast<E*>(p.kc) + pg * p.k_sp : reinterpret_cast<E*>(p.vc) + pg * p.v_sp) +
           (((long long)g << p.shift) + in_page) * sz;
  const E* gain = reinterpret_cast<const E*>(p.kn);
  float n = 1.f;
  const bool norm = key && gain;
  if (norm) {
    float ss = 0.f;
    for (int c = lane * V; c < sz; c += NL * V) {
      const Pack u = *reinterpret_cast<const Pack*>(src + c);
#pragma unroll
      for (int e = 0; e < V; ++e) ss = fmaf(El<E>::ld(u.v + e), El<E>::ld(u.v + e), ss);
    }
    ss = lanes_reduce<NL>(ss, [](float a, float b) { return a + b; });
    n = 1.f / sqrtf(ss / (float)sz + p.eps);
  }
  for (int c = lane * V; c < sz; c += NL * V) {
    Pack u = *reinterpret_cast<const Pack*>(src + c);
    if (norm) {
      const Pack w = *reinterpret_cast<const Pack*>(gain + c);
#pragma unroll
      for (int e = 0; e < V; ++e) El<E>::st(u.v + e, El<E>::ld(u.v + e) * n * El<E>::ld(w.v + e));
    }
    *reinterpret_cast<Pack*>(dst + c) = u;
  }
}

template <typename E>
int append_go(const BiasedArgs& p, int T, bool vec, hipStream_t s) {
  constexpr int V = sizeof(E) == 2 ? 8 : 4;
  const long long n = (long long)T * 2 * p.G;
  const int lanes = ((p.dim > p.vdim ? p.dim : p.vdim) + V - 1) / V;
#define GO(W, NL) hipLaunchKernelGGL((append_kernel<E, W, NL>), dim3((unsigned)((n * NL + 255) / 256)), dim3(256), 0, s, p, T)
  if (!vec) GO(1, 64);
  else if (lanes <= 8) GO(V, 8);
  else if (lanes <= 16) GO(V, 16);
  else if (lanes <= 32) GO(V, 32);
  else GO(V, 64);
#undef GO
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

}  // namespace

// Mirrored by ops/biased_attention.py (checked by kca_biased_attn_abi)
struct KcaBiasedAttn {
  BiasedArgs a;
};
KCA_API int kca_biased_attn_abi() { return (int)sizeof(KcaBiasedAttn); }

// K / V of T tokens into their pages
KCA_API int kca_biased_append(const KcaBiasedAttn* in, int dtype, int T, hipStream_t s) {
  const BiasedArgs& p = in->a;
  if (!args_ok(p) || !p.pos || !p.slot || T < 1 || (long long)T * 2 * p.G > 0x7fffffff) return 1;
  if (dtype == 0) return append_go<float>(p, T, vec_ok(p), s);
  if (dtype == 1) return append_go<bf16_t>(p, T, vec_ok(p), s);
  return 3;
}

KCA_API int kca_biased_rows(const KcaBiasedAttn* in, int dtype, int rows, long long ws_floats, long long n_cnt, int max_kv,
                            hipStream_t s) {
  return rows_entry<false>(in->a, dtype, rows, ws_floats, n_cnt, max_kv, s);
}

KCA_API int kca_biased_tiles(const KcaBiasedAttn* in, int ntiles, hipStream_t s) { return tiles_entry<false>(in->a, ntiles, s); }
