// The residual row update of layers whose sublayers run side by side: two branches that join through norms of their
// own, a plain addend, and the norm the next reader wants, in one pass over the row.
//   new = (keep ? x : 0) + coef (rms(a) wa + rms(b) wb) + f;   x <- new;   h = rms(new) hw
// (a, b, f and h each optional; hw is a vector, or one number for all columns).  All sums fp32.
#include "seq_common.h"
#include "row_vec.h"
#include "fls_seq.h"

#define RB_PIECES 8                // 256 VE columns a piece; that many pieces of a and b stay in registers

// one block per row
template <typename TO, int VE>
__global__ __launch_bounds__(256) void residual_branches_kernel(float* __restrict__ x, int ldx, int keep, const float* __restrict__ a,
                                                                int lda, const float* __restrict__ wa, const float* __restrict__ b,
                                                                int ldb, const float* __restrict__ wb, float coef,
                                                                const float* __restrict__ f, int ldf_, TO* __restrict__ h, int ldh,
                                                                const float* __restrict__ hw, int hw_one, int D, float eps) {
  __shared__ float red[8];
  const int r = blockIdx.x;
  const int wave = threadIdx.x >> 6;
  float* xr = x + (size_t)r * ldx;
  const float* ar = a != nullptr ? a + (size_t)r * lda : nullptr;
  const float* br = a != nullptr ? b + (size_t)r * ldb : nullptr;
  const float* fr = f != nullptr ? f + (size_t)r * ldf_ : nullptr;
  const int np = (D + 256 * VE - 1) / (256 * VE);
  RowVec<VE> av[RB_PIECES], bv[RB_PIECES];
  float rsa = 0.f, rsb = 0.f;
  if (ar != nullptr) {
    float sa = 0.f, sb = 0.f;
#pragma unroll
    for (int k = 0; k < RB_PIECES; ++k) {
      const int c = (threadIdx.x + 256 * k) * VE;
      if (c < D) {
        av[k] = row_load<VE>(ar + c);
        bv[k] = row_load<VE>(br + c);
#pragma unroll
        for (int i = 0; i < VE; ++i) { sa += av[k].v[i] * av[k].v[i]; sb += bv[k].v[i] * bv[k].v[i]; }
      }
    }
    for (int k = RB_PIECES; k < np; ++k) {
      const int c = (threadIdx.x + 256 * k) * VE;
      if (c < D) {
        const RowVec<VE> ta = row_load<VE>(ar + c), tb = row_load<VE>(br + c);
#pragma unroll
        for (int i = 0; i < VE; ++i) { sa += ta.v[i] * ta.v[i]; sb += tb.v[i] * tb.v[i]; }
      }
    }
    sa = wave_sum(sa);
    sb = wave_sum(sb);
    if ((threadIdx.x & 63) == 0) { red[wave] = sa; red[4 + wave] = sb; }
    __syncthreads();
    rsa = coef / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)D + eps);
    rsb = coef / sqrtf((red[4] + red[5] + red[6] + red[7]) / (float)D + eps);
    __syncthreads();
  }
  float ss = 0.f;
  // one piece of the row; returns the new entries
  auto piece = [&](int c, const RowVec<VE>& pa, const RowVec<VE>& pb) -> RowVec<VE> {
    RowVec<VE> n;
    if (keep) n = row_load<VE>(xr + c);
    else {
#pragma unroll
      for (int i = 0; i < VE; ++i) n.v[i] = 0.f;
    }
    if (ar != nullptr) {
      const RowVec<VE> qa = row_load<VE>(wa + c), qb = row_load<VE>(wb + c);
#pragma unroll
      for (int i = 0; i < VE; ++i) n.v[i] += pa.v[i] * rsa * qa.v[i] + pb.v[i] * rsb * qb.v[i];
    }
    if (fr != nullptr) {
      const RowVec<VE> q = row_load<VE>(fr + c);
#pragma unroll
      for (int i = 0; i < VE; ++i) n.v[i] += q.v[i];
    }
    row_store<VE>(xr + c, n);
#pragma unroll
    for (int i = 0; i < VE; ++i) ss += n.v[i] * n.v[i];
    return n;
  };
#pragma unroll
  for (int k = 0; k < RB_PIECES; ++k) {
    const int c = (threadIdx.x + 256 * k) * VE;
    if (c < D) av[k] = piece(c, av[k], bv[k]);       // (from here on av holds the new entries)
  }
  for (int k = RB_PIECES; k < np; ++k) {
    const int c = (threadIdx.x + 256 * k) * VE;
    if (c >= D) break;
    RowVec<VE> ta, tb;
    if (ar != nullptr) { ta = row_load<VE>(ar + c); tb = row_load<VE>(br + c); }
    piece(c, ta, tb);
  }
  if (h == nullptr) return;
  ss = wave_sum(ss);
  if ((threadIdx.x & 63) == 0) red[wave] = ss;
  __syncthreads();
  const float rs = 1.f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)D + eps);
  TO* hr = h + (size_t)r * ldh;
  const float g1 = hw_one ? hw[0] : 0.f;
  auto out = [&](int c, RowVec<VE> n) {
#pragma unroll
    for (int i = 0; i < VE; ++i) n.v[i] *= rs * (hw_one ? g1 : hw[c + i]);
    row_store<VE>(hr + c, n);
  };
#pragma unroll
  for (int k = 0; k < RB_PIECES; ++k) {
    const int c = (threadIdx.x + 256 * k) * VE;
    if (c < D) out(c, av[k]);
  }
  for (int k = RB_PIECES; k < np; ++k) {             // (a thread re-reads only what it wrote itself)
    const int c = (threadIdx.x + 256 * k) * VE;
    if (c >= D) break;
    out(c, row_load<VE>(xr + c));
  }
}

extern "C" int fls_seq_residual_branches(float* x, int ldx, int keep, const float* a, int lda, const float* wa, const float* b,
                                         int ldb, const float* wb, float coef, const float* f, int ldf, void* h, int th, int ldh,
                                         const float* hw, int hw_one, int rows, int D, float eps, fls_stream_t s) {
  if (rows <= 0) return 0;
  if (D < 1 || x == nullptr || (a == nullptr) != (b == nullptr) || (a != nullptr && (wa == nullptr || wb == nullptr)) ||
      (h != nullptr && hw == nullptr))
    return -1;
  auto al = [](const void* p, int ld, int es) { return p == nullptr || ((uintptr_t)p % (4 * es) == 0 && ld % 4 == 0); };
  const int vec = D % 4 == 0 && al(x, ldx, 4) && al(a, lda, 4) && al(b, ldb, 4) && al(wa, 0, 4) && al(wb, 0, 4) && al(f, ldf, 4) &&
                  al(h, ldh, th == 1 ? 2 : 4);
  hipStream_t st = (hipStream_t)s;
#define RB_GO(TO, VV) hipLaunchKernelGGL((residual_branches_kernel<TO, VV>), dim3(rows), dim3(256), 0, st, x, ldx, keep, a, lda, wa, b, ldb, \
                                         wb, coef, f, ldf, (TO*)h, ldh, hw, hw_one, D, eps)
  if (th == 1) { if (vec) RB_GO(bf16_t, 4); else RB_GO(bf16_t, 1); }
  else { if (vec) RB_GO(float, 4); else RB_GO(float, 1); }
#undef RB_GO
  SEQ_LAUNCH_CHECK();
  return 0;
}
