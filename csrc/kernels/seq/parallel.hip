// Layers whose mixer and feed-forward run side by side on one row, each with a norm and a per-channel scale of its own, and the
// input rows of a latent attention.  One block per row (or row and column piece), fp32 sums.
#include "seq_common.h"
#include "row_vec.h"
#include "fls_seq.h"

static inline bool vec4_ok(const void* p, int ld, int es) { return p == nullptr || ((uintptr_t)p % (4 * es) == 0 && ld % 4 == 0); }

// ------------------------------------------------------------------- two norms of one row
// x (+= add first), then h1 = x rs w1 and h2 = x rs w2 with rs = 1 / sqrt(mean(x^2) + eps): the row is read once
#define RP_PIECES 8                // 256 VE columns a piece; that many pieces stay in registers
template <typename TO, int VE>
__global__ __launch_bounds__(256) void rmsnorm_pair_kernel(float* __restrict__ x, int ldx, const float* __restrict__ add, int ldadd,
                                                           const float* __restrict__ w1, TO* __restrict__ h1, int ld1,
                                                           const float* __restrict__ w2, TO* __restrict__ h2, int ld2, int D,
                                                           float eps) {
  __shared__ float red[4];
  const int r = blockIdx.x;
  float* xr = x + (size_t)r * ldx;
  const float* ar = add != nullptr ? add + (size_t)r * ldadd : nullptr;
  const int np = (D + 256 * VE - 1) / (256 * VE);
  RowVec<VE> v[RP_PIECES];
  float ss = 0.f;
  auto piece = [&](int c) -> RowVec<VE> {
    RowVec<VE> n = row_load<VE>(xr + c);
    if (ar != nullptr) {
      const RowVec<VE> q = row_load<VE>(ar + c);
#pragma unroll
      for (int i = 0; i < VE; ++i) n.v[i] += q.v[i];
      row_store<VE>(xr + c, n);
    }
#pragma unroll
    for (int i = 0; i < VE; ++i) ss += n.v[i] * n.v[i];
    return n;
  };
#pragma unroll
  for (int k = 0; k < RP_PIECES; ++k) {
    const int c = (threadIdx.x + 256 * k) * VE;
    if (c < D) v[k] = piece(c);
  }
  for (int k = RP_PIECES; k < np; ++k) {
    const int c = (threadIdx.x + 256 * k) * VE;
    if (c < D) piece(c);
  }
  ss = block_sum_256(ss, red);
  const float rs = 1.f / sqrtf(ss / (float)D + eps);
  auto out = [&](int c, const RowVec<VE>& n) {
    RowVec<VE> a = row_load<VE>(w1 + c);
#pragma unroll
    for (int i = 0; i < VE; ++i) a.v[i] *= n.v[i] * rs;
    row_store<VE>(h1 + (size_t)r * ld1 + c, a);
    if (h2 != nullptr) {
      RowVec<VE> b = row_load<VE>(w2 + c);
#pragma unroll
      for (int i = 0; i < VE; ++i) b.v[i] *= n.v[i] * rs;
      row_store<VE>(h2 + (size_t)r * ld2 + c, b);
    }
  };
#pragma unroll
  for (int k = 0; k < RP_PIECES; ++k) {
    const int c = (threadIdx.x + 256 * k) * VE;
    if (c < D) out(c, v[k]);
  }
  for (int k = RP_PIECES; k < np; ++k) {             // (a thread re-reads only what it wrote itself)
    const int c = (threadIdx.x + 256 * k) * VE;
    if (c < D) out(c, row_load<VE>(xr + c));
  }
}

extern "C" int fls_seq_rmsnorm_pair(float* x, int ldx, const float* add, int ldadd, const float* w1, void* h1, int ld1,
                                    const float* w2, void* h2, int ld2, int th, int rows, int D, float eps, fls_stream_t s) {
  if (rows <= 0) return 0;
  if (D < 1 || w1 == nullptr || h1 == nullptr || (w2 == nullptr) != (h2 == nullptr)) return -1;
  const int es = th == 1 ? 2 : 4;
  const bool vec = D % 4 == 0 && vec4_ok(x, ldx, 4) && vec4_ok(add, ldadd, 4) && vec4_ok(w1, 0, 4) && vec4_ok(w2, 0, 4) &&
                   vec4_ok(h1, ld1, es) && vec4_ok(h2, ld2, es);
  hipStream_t st = (hipStream_t)s;
#define RP_GO(TO, VV) hipLaunchKernelGGL((rmsnorm_pair_kernel<TO, VV>), dim3(rows), dim3(256), 0, st, x, ldx, add, ldadd, w1, (TO*)h1, ld1, w2, \
                                         (TO*)h2, ld2, D, eps)
  if (th == 1) { if (vec) RP_GO(bf16_t, 4); else RP_GO(bf16_t, 1); }
  else { if (vec) RP_GO(float, 4); else RP_GO(float, 1); }
#undef RP_GO
  SEQ_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------- the residual update of both sublayers
// x += a wa + f wb: f a row of its own, or the weighted sum of the rows of the token's experts (identity experts: the row h
// that went in), which so never exists in memory
template <typename TH, int VE>
__global__ __launch_bounds__(256) void parallel_update_kernel(float* __restrict__ x, int ldx, const float* __restrict__ a, int lda,
                                                              const float* __restrict__ wa, const float* __restrict__ b, int ldb,
                                                              const float* __restrict__ wb, const float* __restrict__ y, int ldy,
                                                              const int* __restrict__ dest, const float* __restrict__ w,
                                                              const int* __restrict__ ids, int top, int E,
                                                              const TH* __restrict__ h, int ldh, int D) {
  const int t = blockIdx.x;
  const int c = (blockIdx.y * 256 + threadIdx.x) * VE;
  if (c >= D) return;
  RowVec<VE> n = row_load<VE>(x + (size_t)t * ldx + c);
  {
    const RowVec<VE> av = row_load<VE>(a + (size_t)t * lda + c), s = row_load<VE>(wa + c);
#pragma unroll
    for (int i = 0; i < VE; ++i) n.v[i] += av.v[i] * s.v[i];
  }
  if (wb != nullptr) {
    RowVec<VE> f;
    if (dest != nullptr) {
#pragma unroll
      for (int i = 0; i < VE; ++i) f.v[i] = 0.f;
      for (int k = 0; k < top; ++k) {
        const size_t at = (size_t)t * top + k;
        const float wk = w[at];
        const RowVec<VE> q = ids[at] < E ? row_load<VE>(y + (size_t)dest[at] * ldy + c) : row_load<VE>(h + (size_t)t * ldh + c);
#pragma unroll
        for (int i = 0; i < VE; ++i) f.v[i] += wk * q.v[i];
      }
    } else {
      f = row_load<VE>(b + (size_t)t * ldb + c);
    }
    const RowVec<VE> s = row_load<VE>(wb + c);
#pragma unroll
    for (int i = 0; i < VE; ++i) n.v[i] += f.v[i] * s.v[i];
  }
  row_store<VE>(x + (size_t)t * ldx + c, n);
}

extern "C" int fls_seq_parallel_update(float* x, int ldx, const float* a, int lda, const float* wa, const float* b, int ldb,
                                       const float* wb, const float* y, int ldy, const int* dest, const float* w, const int* ids,
                                       int top, int E, const void* h, int th, int ldh, int rows, int D, fls_stream_t s) {
  if (rows <= 0) return 0;
  if (D < 1 || a == nullptr || wa == nullptr) return -1;
  if (dest != nullptr && (b != nullptr || wb == nullptr || y == nullptr || w == nullptr || ids == nullptr || h == nullptr || top < 1)) return -1;
  if (dest == nullptr && (b == nullptr) != (wb == nullptr)) return -1;
  const bool vec = D % 4 == 0 && vec4_ok(x, ldx, 4) && vec4_ok(a, lda, 4) && vec4_ok(wa, 0, 4) && vec4_ok(b, ldb, 4) && vec4_ok(wb, 0, 4) &&
                   vec4_ok(y, ldy, 4) && vec4_ok(h, ldh, th == 1 ? 2 : 4);
  hipStream_t st = (hipStream_t)s;
#define PU_GO(TH, VV)                                                                                                                    \
  hipLaunchKernelGGL((parallel_update_kernel<TH, VV>), dim3(rows, (D + 256 * VV - 1) / (256 * VV)), dim3(256), 0, st, x, ldx, a, lda, wa, b, \
                     ldb, wb, y, ldy, dest, w, ids, top, E, (const TH*)h, ldh, D)
  if (th == 1) { if (vec) PU_GO(bf16_t, 4); else PU_GO(bf16_t, 1); }
  else { if (vec) PU_GO(float, 4); else PU_GO(float, 1); }
#undef PU_GO
  SEQ_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------- rows of a latent attention
// one block per row of z = [query latent (qr) | latent (r) | rotated key part (dr) | ...]: both latents' statistics at once, the
// normed query latent to cq, the normed latent and the rotated key part to the row's place in the pool
template <typename TO, int VE>
__global__ __launch_bounds__(256) void latent_rows_kernel(const float* __restrict__ z, int ldz, int qr, int r, int dr,
                                                          const float* __restrict__ qw, const float* __restrict__ kw, float eps,
                                                          const float* __restrict__ freqs, int rot, const int* __restrict__ tok_pos,
                                                          const int* __restrict__ kv_slot, TO* __restrict__ cq, int ldcq,
                                                          TO* __restrict__ pool, int pw) {
  __shared__ float red[8];
  const int t = blockIdx.x;
  const float* zq = z + (size_t)t * ldz;
  const float* zk = zq + qr;
  const float* zr = zk + r;
  TO* prow = pool + (size_t)kv_slot[t] * pw;
  float sq = 0.f, sk = 0.f;
  for (int c = threadIdx.x * VE; c < qr; c += 256 * VE) {
    const RowVec<VE> v = row_load<VE>(zq + c);
#pragma unroll
    for (int i = 0; i < VE; ++i) sq += v.v[i] * v.v[i];
  }
  for (int c = threadIdx.x * VE; c < r; c += 256 * VE) {
    const RowVec<VE> v = row_load<VE>(zk + c);
#pragma unroll
    for (int i = 0; i < VE; ++i) sk += v.v[i] * v.v[i];
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((threadIdx.x & 63) == 0) { red[threadIdx.x >> 6] = sq; red[4 + (threadIdx.x >> 6)] = sk; }
  // (the rotation needs no statistic: it goes on while the others arrive)
  const float pos = rot > 0 ? (float)tok_pos[t] : 0.f;
  const int hr = rot >> 1;
  for (int c = threadIdx.x; c < dr; c += 256) {
    float v = zr[c];
    if (c < rot) {
      const bool second = c >= hr;
      const float ang = pos * freqs[second ? c - hr : c], cs = cosf(ang), sn = sinf(ang);
      v = second ? v * cs + zr[c - hr] * sn : v * cs - zr[c + hr] * sn;
    }
    stf(prow + r, c, v);
  }
  __syncthreads();
  const float rk = 1.f / sqrtf((red[4] + red[5] + red[6] + red[7]) / (float)r + eps);
  for (int c = threadIdx.x * VE; c < r; c += 256 * VE) {
    RowVec<VE> v = row_load<VE>(zk + c);
    const RowVec<VE> w = row_load<VE>(kw + c);
#pragma unroll
    for (int i = 0; i < VE; ++i) v.v[i] *= rk * w.v[i];
    row_store<VE>(prow + c, v);
  }
  if (qr > 0) {
    const float rq = 1.f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)qr + eps);
    for (int c = threadIdx.x * VE; c < qr; c += 256 * VE) {
      RowVec<VE> v = row_load<VE>(zq + c);
      const RowVec<VE> w = row_load<VE>(qw + c);
#pragma unroll
      for (int i = 0; i < VE; ++i) v.v[i] *= rq * w.v[i];
      row_store<VE>(cq + (size_t)t * ldcq + c, v);
    }
  }
}

extern "C" int fls_seq_latent_rows(const float* z, int ldz, int qr, int r, int dr, const float* qw, const float* kw, float eps,
                                   const float* freqs, int rot, const int* tok_pos, const int* kv_slot, void* cq, int ldcq,
                                   void* pool, int pw, int tp, int T, fls_stream_t s) {
  if (T <= 0) return 0;
  if (r < 1 || qr < 0 || dr < 0 || rot < 0 || rot > dr || (rot & 1) || (rot > 0 && freqs == nullptr) || pw < r + dr || ldz < qr + r + dr ||
      (qr > 0 && (qw == nullptr || cq == nullptr || ldcq < qr)))
    return -1;
  const int es = tp == 1 ? 2 : 4;
  const bool vec = qr % 4 == 0 && r % 4 == 0 && vec4_ok(z, ldz, 4) && vec4_ok(qw, 0, 4) && vec4_ok(kw, 0, 4) && vec4_ok(cq, ldcq, es) &&
                   vec4_ok(pool, pw, es);
  hipStream_t st = (hipStream_t)s;
#define LR_GO(TO, VV) hipLaunchKernelGGL((latent_rows_kernel<TO, VV>), dim3(T), dim3(256), 0, st, z, ldz, qr, r, dr, qw, kw, eps, freqs, rot, \
                                         tok_pos, kv_slot, (TO*)cq, ldcq, (TO*)pool, pw)
  if (tp == 1) { if (vec) LR_GO(bf16_t, 4); else LR_GO(bf16_t, 1); }
  else { if (vec) LR_GO(float, 4); else LR_GO(float, 1); }
#undef LR_GO
  SEQ_LAUNCH_CHECK();
  return 0;
}
