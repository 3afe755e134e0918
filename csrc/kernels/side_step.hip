// One decoded token per row through two mixers of the same projection rows in one launch: windowed attention over block
// means (pooled_attn.hip) in the first workgroups, a matrix memory (matrix_memory.hip) in the rest. Neither fills the
// chip or its memory at small batches, so they run side by side. bf16, usual head sizes.
#include "biased_attn.h"
#include "matrix_memory.h"

namespace {

struct SideArgs {
  BiasedArgs a;
  MemArgs m;
  int rows, na;  // tokens; workgroups of the attention
};

template <int LP, int R>
__global__ void __launch_bounds__(256, 4) side_step_kernel(SideArgs p) {
  __shared__ float red[16];
  extern __shared__ __attribute__((aligned(16))) float merged[];
  // the memory's workgroups first: they are few and start their state's loads at once
  const int nm = p.rows * p.m.H, b = (int)blockIdx.x;
  if (b < nm) {
    step_body<bf16_t, R, 4>(p.m, b / p.m.H, b % p.m.H, merged, red);
  } else {
    const int i = b - nm, ny = p.a.G * ((p.a.H / p.a.G + 3) / 4);
    rows_body<bf16_t, 4, LP, true, true>(p.a, i / ny % p.rows, i % ny, i / ny / p.rows, ny);
  }
}

template <int LP, int R>
int side_go(const SideArgs& p, hipStream_t s) {
  size_t lds = rows_lds<true>(p.a, 4);
  if (lds < (size_t)p.m.dv * 4) lds = (size_t)p.m.dv * 4;
  if (lds > 48 * 1024) return 10;
  hipLaunchKernelGGL((side_step_kernel<LP, R>), dim3(p.na + p.rows * p.m.H), dim3(256), lds, s, p);
  return hipGetLastError() == hipSuccess ? 0 : 4;
}

}  // namespace

// Mirrored by ops/side_step.py
KCA_API int kca_side_step_abi() { return (int)sizeof(SideArgs); }

// 10: sizes for two launches
KCA_API int kca_side_step(const BiasedArgs* attn, const MemArgs* mem, int rows, long long ws_floats, long long n_cnt, int max_kv,
                          hipStream_t s) {
  SideArgs p{*attn, *mem, rows, 0};
  const BiasedArgs& a = p.a;
  if (!pool_ok(a) || !mem_ok(p.m) || !p.m.out || !a.append || a.row_of) return 1;
  if (!pool_vec(a) || a.H / a.G < 2 || a.dim > 128 || a.vdim > 128 || p.m.dk > 128 || p.m.dk < 33 || !wide(p.m)) return 10;
  if (const int rc = rows_check(a, rows, ws_floats, n_cnt, max_kv)) return rc;
  const long long n = (long long)rows * a.G * ((a.H / a.G + 3) / 4) * a.nsplit;
  if (n + (long long)rows * p.m.H > 0x7fffffff) return 1;
  p.na = (int)n;
  const int lp = lanes_for(a.dim > a.vdim ? a.dim : a.vdim);
  if (p.m.dk <= 64) return lp == 8 ? side_go<8, 4>(p, s) : side_go<16, 4>(p, s);
  return lp == 8 ? side_go<8, 8>(p, s) : side_go<16, 8>(p, s);
}
