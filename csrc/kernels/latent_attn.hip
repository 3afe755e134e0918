// Latent attention (latent_attn.h) in any size, fp32 or bf16:
//
//   prep kernel    norms both latents of new tokens, rotates the shared key part, stores the cache rows
//   head_mm        per-head products (W_uk^T q)
//   rows kernel    one query token and head per workgroup over the paged latents -> partial softmax
//   merge kernel   merges the partials of a (row, head) and applies W_uv
#include "latent_attn.h"

namespace {
using latent::ld;
using latent::rot;

template <typename E> __device__ __forceinline__ float ex(float x);
template <> __device__ __forceinline__ float ex<float>(float x) { return expf(x); }
template <> __device__ __forceinline__ float ex<bf16_t>(float x) { return __expf(x); }

// bf16 rows in multiples of 8 (at most 2048 of either latent): a thread keeps its elements between the passes
__global__ void __launch_bounds__(256) latent_prep_vec_kernel(LatentArgs a) {
  __shared__ float red[8];
  const int t = blockIdx.x, tid = threadIdx.x, pos = a.pos[t], c = tid * 8;
  const bf16_t* xq = reinterpret_cast<const bf16_t*>(a.x) + (long long)t * a.ld + a.o_q;
  const bf16_t* xk = reinterpret_cast<const bf16_t*>(a.x) + (long long)t * a.ld + a.o_kv;
  const long long pg = a.table[(long long)a.slot[t] * a.tstride + (pos >> a.shift)];
  float q[8], k[8], gq[8], gk[8], sq = 0.f, sk = 0.f;
  const int tq = c < a.Q ? c : 0, tk = c < a.C ? c : 0;
  load8(xq + tq, q);
  load8(xk + tk, k);
  load8(reinterpret_cast<const bf16_t*>(a.gq) + tq, gq);
  load8(reinterpret_cast<const bf16_t*>(a.gk) + tk, gk);
#pragma unroll
  for (int e = 0; e < 8; ++e) sq = fmaf(q[e], q[e], sq), sk = fmaf(k[e], k[e], sk);
  sq = wave_sum(c < a.Q ? sq : 0.f);
  sk = wave_sum(c < a.C ? sk : 0.f);
  if ((tid & 63) == 0) red[tid >> 6] = sq, red[4 + (tid >> 6)] = sk;
  bf16_t* row = reinterpret_cast<bf16_t*>(a.kc) + pg * a.k_sp + (long long)(pos & ((1 << a.shift) - 1)) * (a.C + a.R);
  for (int i = tid - 192; i >= 0 && i < a.R; i += 64) latent::st<bf16_t>(row + a.C + i, rot<bf16_t>(xk + a.C, i, pos, a.freq, a.nr));
  __syncthreads();
  const float nq = 1.f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.Q + a.eps);
  const float nk = 1.f / sqrtf((red[4] + red[5] + red[6] + red[7]) / (float)a.C + a.eps);
#pragma unroll
  for (int e = 0; e < 8; ++e) q[e] *= nq * gq[e], k[e] *= nk * gk[e];
  if (c < a.Q) store8(reinterpret_cast<bf16_t*>(a.cq) + (long long)t * a.Q + c, q);
  if (c < a.C) store8(row + c, k);
}

template <typename E>
__global__ void __launch_bounds__(256) latent_prep_kernel(LatentArgs a) {
  __shared__ float red[2][4];
  const int t = blockIdx.x, tid = threadIdx.x, pos = a.pos[t];
  const E* xq = reinterpret_cast<const E*>(a.x) + (long long)t * a.ld + a.o_q;
  const E* xk = reinterpret_cast<const E*>(a.x) + (long long)t * a.ld + a.o_kv;
  float sq = 0.f, sk = 0.f;
  for (int i = tid; i < a.Q; i += 256) { const float v = ld<E>(xq + i); sq = fmaf(v, v, sq); }
  for (int i = tid; i < a.C; i += 256) { const float v = ld<E>(xk + i); sk = fmaf(v, v, sk); }
  const float nq = 1.f / sqrtf(block_sum(sq, red[0]) / (float)a.Q + a.eps);
  const float nk = 1.f / sqrtf(block_sum(sk, red[1]) / (float)a.C + a.eps);
  E* cq = reinterpret_cast<E*>(a.cq) + (long long)t * a.Q;
  for (int i = tid; i < a.Q; i += 256)
    latent::st<E>(cq + i, ld<E>(xq + i) * nq * ld<E>(reinterpret_cast<const E*>(a.gq) + i));
  const long long pg = a.table[(long long)a.slot[t] * a.tstride + (pos >> a.shift)];
  E* row = reinterpret_cast<E*>(a.kc) + pg * a.k_sp + (long long)(pos & ((1 << a.shift) - 1)) * (a.C + a.R);
  for (int i = tid; i < a.C; i += 256)
    latent::st<E>(row + i, ld<E>(xk + i) * nk * ld<E>(reinterpret_cast<const E*>(a.gk) + i));
  for (int i = tid; i < a.R; i += 256) latent::st<E>(row + a.C + i, rot<E>(xk + a.C, i, pos, a.freq, a.nr));
}

// y[b][h][n] = sum_k x[row_of[b]][h][k] w[h][n][k]
template <typename E>
__global__ void __launch_bounds__(256) head_mm_kernel(const E* x, long long ldx, int hx, const E* w, E* y, long long ldy,
                                                      int hy, int N, int K, const int* row_of) {
  extern __shared__ float xs[];
  const int b = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int row = row_of ? row_of[b] : b;
  const E* xr = x + row * ldx + (long long)h * hx;
  for (int i = tid; i < K; i += 256) xs[i] = ld<E>(xr + i);
  __syncthreads();
  for (int n = tid; n < N; n += 256) {
    const E* wr = w + ((long long)h * N + n) * K;
    float s = 0.f;
    for (int k = 0; k < K; ++k) s = fmaf(xs[k], ld<E>(wr + k), s);
    latent::st<E>(y + b * ldy + (long long)h * hy + n, s);
  }
}

// tiles of 64 keys: a wave scores 16 of them, then every thread sums its latent columns
template <typename E, int NC>
__global__ void __launch_bounds__(256) latent_rows_kernel(LatentArgs a) {
  extern __shared__ float q[];  // [C + R]
  __shared__ float sc[64];
  const int b = blockIdx.x, h = blockIdx.y, sp = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int row = a.row_of ? a.row_of[b] : b, pos = a.pos[row], kv = pos + 1, KL = a.C + a.R;
  const int lo = sp * a.chunk, hi = min(kv, lo + a.chunk);
  if (lo >= kv) return;
  const E* qa = reinterpret_cast<const E*>(a.qa) + ((long long)b * a.H + h) * a.C;
  const E* qr = reinterpret_cast<const E*>(a.q) + ((long long)row * a.H + h) * (a.D + a.R) + a.D;
  for (int i = tid; i < KL; i += 256) q[i] = (i < a.C ? ld<E>(qa + i) : rot<E>(qr, i - a.C, pos, a.freq, a.nr)) * a.scale;
  __syncthreads();
  const int* tbl = a.table + (long long)a.slot[row] * a.tstride;
  const int pmask = (1 << a.shift) - 1;
  const E* kc = reinterpret_cast<const E*>(a.kc);
  float m = -INFINITY, l = 0.f, acc[NC];
#pragma unroll
  for (int i = 0; i < NC; ++i) acc[i] = 0.f;
  for (int k0 = lo; k0 < hi; k0 += 64) {
    for (int j = wv * 16; j < wv * 16 + 16; ++j) {
      const int key = k0 + j;
      float s = -INFINITY;
      if (key < hi) {
        const E* kr = kc + (long long)tbl[key >> a.shift] * a.k_sp + (long long)(key & pmask) * KL;
        float d = 0.f;
        for (int i = lane; i < KL; i += 64) d = fmaf(q[i], ld<E>(kr + i), d);
        s = wave_sum(d);
      }
      if (lane == 0) sc[j] = s;
    }
    __syncthreads();
    const float s = sc[lane], mn = fmaxf(m, wave_max(s)), e = ex<E>(s - mn), al = ex<E>(m - mn);
    l = l * al + wave_sum(e);
    m = mn;
    __syncthreads();
    if (wv == 0) sc[lane] = e;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NC; ++i) acc[i] *= al;
    const int n = min(64, hi - k0);
    for (int j = 0; j < n; ++j) {
      const int key = k0 + j;
      const E* kr = kc + (long long)tbl[key >> a.shift] * a.k_sp + (long long)(key & pmask) * KL;
      const float w = sc[j];
#pragma unroll
      for (int i = 0; i < NC; ++i)
        if (tid + 256 * i < a.C) acc[i] = fmaf(w, ld<E>(kr + tid + 256 * i), acc[i]);
    }
    __syncthreads();
  }
  float* part = a.part + (((long long)b * a.H + h) * a.nsplit + sp) * (a.C + 4);
  if (tid == 0) part[0] = m, part[1] = l;
#pragma unroll
  for (int i = 0; i < NC; ++i)
    if (tid + 256 * i < a.C) part[4 + tid + 256 * i] = acc[i];
}

template <typename E>
__global__ void __launch_bounds__(256) latent_merge_kernel(LatentArgs a) {
  extern __shared__ float o[];  // [C]
  const int b = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int row = a.row_of ? a.row_of[b] : b, used = (a.pos[row] + a.chunk) / a.chunk;
  const float sink = ld<E>(reinterpret_cast<const E*>(a.sink) + h);
  const int st = a.C + 4;
  const float* part = a.part + ((long long)b * a.H + h) * a.nsplit * st;
  float M = sink;
  for (int z = 0; z < used; ++z) M = fmaxf(M, part[(long long)z * st]);
  float L = ex<E>(sink - M);
  for (int z = 0; z < used; ++z) L += part[(long long)z * st + 1] * ex<E>(part[(long long)z * st] - M);
  for (int c = tid; c < a.C; c += 256) {
    float v = 0.f;
    for (int z = 0; z < used; ++z) v = fmaf(ex<E>(part[(long long)z * st] - M), part[(long long)z * st + 4 + c], v);
    o[c] = v / L;
  }
  __syncthreads();
  E* out = reinterpret_cast<E*>(a.out) + row * a.ldo + (long long)h * a.E;
  for (int e = wv; e < a.E; e += 4) {
    const E* w = reinterpret_cast<const E*>(a.wuv) + ((long long)h * a.E + e) * a.C;
    float s = 0.f;
    for (int c = lane; c < a.C; c += 64) s = fmaf(o[c], ld<E>(w + c), s);
    s = wave_sum(s);
    if (lane == 0) latent::st<E>(out + e, s);
  }
}

template <typename E>
int rows_go(const LatentArgs& a, int rows, hipStream_t s) {
  const size_t lds = (size_t)(a.C + a.R) * 4;
  const dim3 g(rows, a.H, a.nsplit);
  if (a.C <= 256) hipLaunchKernelGGL((latent_rows_kernel<E, 1>), g, dim3(256), lds, s, a);
  else if (a.C <= 512) hipLaunchKernelGGL((latent_rows_kernel<E, 2>), g, dim3(256), lds, s, a);
  else if (a.C <= 1024) hipLaunchKernelGGL((latent_rows_kernel<E, 4>), g, dim3(256), lds, s, a);
  else return 10;
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

}  // namespace

// Mirrored by ops/latent_attention.py
KCA_API int kca_latent_abi() { return (int)sizeof(LatentArgs); }

// dtype: 0 fp32, 1 bf16. T tokens' latents into their pages, normed query latents into a.cq
KCA_API int kca_latent_prep(const LatentArgs* in, int dtype, int T, hipStream_t s) {
  const LatentArgs& a = *in;
  if (!latent_args_ok(a) || T < 1 || !a.x || !a.cq || !a.gq || !a.gk) return 1;
  if (dtype == 0) hipLaunchKernelGGL((latent_prep_kernel<float>), dim3(T), dim3(256), 0, s, a);
  else if (dtype == 1) {
    const uintptr_t al = (uintptr_t)a.x | (uintptr_t)a.cq | (uintptr_t)a.kc | (uintptr_t)a.gq | (uintptr_t)a.gk;
    if ((a.Q | a.C | a.R | a.o_q | a.o_kv) % 8 == 0 && a.ld % 8 == 0 && a.k_sp % 8 == 0 && al % 16 == 0 && a.Q <= 2048 && a.C <= 2048)
      hipLaunchKernelGGL(latent_prep_vec_kernel, dim3(T), dim3(256), 0, s, a);
    else hipLaunchKernelGGL((latent_prep_kernel<bf16_t>), dim3(T), dim3(256), 0, s, a);
  } else return 3;
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

// y[b][h][n] = sum_k x[row_of[b]][h][k] w[h][n][k]
KCA_API int kca_head_mm(int dtype, const void* x, long long ldx, int hx, const void* w, void* y, long long ldy, int hy,
                        int B, int H, int N, int K, const void* row_of, hipStream_t s) {
  if (!x || !w || !y || B < 1 || H < 1 || H > 65535 || N < 1 || K < 1 || K > 8192) return 1;
  const dim3 g(B, H);
  if (dtype == 0)
    hipLaunchKernelGGL((head_mm_kernel<float>), g, dim3(256), K * 4, s, (const float*)x, ldx, hx, (const float*)w, (float*)y,
                       ldy, hy, N, K, (const int*)row_of);
  else if (dtype == 1)
    hipLaunchKernelGGL((head_mm_kernel<bf16_t>), g, dim3(256), K * 4, s, (const bf16_t*)x, ldx, hx, (const bf16_t*)w,
                       (bf16_t*)y, ldy, hy, N, K, (const int*)row_of);
  else return 3;
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

// partial softmaxes of `rows` query tokens (a.qa in block order); nsplit * chunk covers max_kv keys
KCA_API int kca_latent_rows(const LatentArgs* in, int dtype, int rows, int max_kv, hipStream_t s) {
  const LatentArgs& a = *in;
  if (!latent_args_ok(a) || rows < 1 || !a.q || !a.qa || !a.part || a.nsplit < 1 || a.nsplit > 65535 || a.chunk < 1 || a.H > 65535)
    return 1;
  if ((long long)a.nsplit * a.chunk < max_kv) return 2;
  if (dtype == 0) return rows_go<float>(a, rows, s);
  if (dtype == 1) return rows_go<bf16_t>(a, rows, s);
  return 3;
}

// a.out of those rows
KCA_API int kca_latent_merge(const LatentArgs* in, int dtype, int rows, hipStream_t s) {
  const LatentArgs& a = *in;
  if (!latent_args_ok(a) || rows < 1 || !a.part || !a.out || !a.wuv || !a.sink || a.chunk < 1 || a.H > 65535) return 1;
  const dim3 g(rows, a.H);
  if (dtype == 0) hipLaunchKernelGGL((latent_merge_kernel<float>), g, dim3(256), a.C * 4, s, a);
  else if (dtype == 1) hipLaunchKernelGGL((latent_merge_kernel<bf16_t>), g, dim3(256), a.C * 4, s, a);
  else return 3;
  return hipGetLastError() == hipSuccess ? 0 : 4;
}
