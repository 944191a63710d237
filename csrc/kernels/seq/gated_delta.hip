// Gated delta rule with a decay per head and key channel: per head a state S [key i, value c] in fp32,
//   S <- diag(g) S;   u = sigmoid(beta) (v - S^T k);   S <- S + k u^T;   o = S^T q
// with unit q and k (q scaled).  With S' = diag(g) S one pass over the state gives both  p1 = S'^T k  and  p2 = S'^T q, and
// o = p2 + u (q . k), so the state is read and written once per token.
//
// The value columns of S do not depend on each other.  Sixteen lanes share a column: lane n of them holds its rows
// 64 m + 4 n .. + 3 in registers, CN columns' worth, and the sums over the key channel are DPP adds inside those sixteen
// lanes (no LDS, no barrier).  The state lies transposed in memory ([value][key]), so the sixteen lanes read a column as
// 256-byte pieces.
//
// A block takes WAVES * 4 * CN columns of one (head, request) and walks the request's rows TT at a time.  The factors of the
// TT rows are made by the whole block, sixteen lanes a row: q and k divided by their lengths, q . k, the decays, into LDS as
// fp32; the next TT rows' loads are issued before the walk and land behind it.
//   prompts (WAVES = 4): the raw o goes to an fp32 matrix; gated_delta_out_kernel finishes whole heads;
//   one row per request (FUSED): a block owns all columns of its head, so norm, weight and gate follow in the same launch.
// A request whose step starts at position 0 starts from zeros without reading its slot.
#include "seq_common.h"
#include "fls_seq.h"

template <int RPL, int CN, int WAVES, int TT, bool FUSED, typename TO>
__global__ __launch_bounds__(64 * WAVES) void gated_delta_kernel(const float* __restrict__ qkv, int ldq, const float* __restrict__ beta,
                                                                 int ldb, const float* __restrict__ decay, int ldd,
                                                                 const float* __restrict__ gate, int ldg,
                                                                 const float* __restrict__ norm_w, float* __restrict__ state,
                                                                 TO* __restrict__ out, int ldo, const int* __restrict__ cu,
                                                                 const int* __restrict__ pos0, const int* __restrict__ slot, int H,
                                                                 int G, int d, int dv, float q_scale, float unit_eps, float norm_eps,
                                                                 int vec) {
  constexpr int DP = 16 * RPL;                       // rows of the state, padded: past d they stay zero
  constexpr int COLS = WAVES * 4 * CN;
  constexpr int NV = (TT * COLS + 64 * WAVES - 1) / (64 * WAVES);
  __shared__ __attribute__((aligned(16))) float sk[TT][DP], sq[TT][DP], sg[TT][DP];
  __shared__ float sv[TT][COLS], sb[TT], sqk[TT];
  __shared__ float so[FUSED ? COLS : 1];
  const int h = blockIdx.y, s = blockIdx.z, hq = h / (H / G);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int ns = lane & 15, lc = (wave * 4 + (lane >> 4)) * CN;      // this lane's rows; its first column inside the block
  const int c0 = blockIdx.x * COLS;
  const int a0 = cu[s], a1 = cu[s + 1];
  float* sp = state + ((size_t)slot[s] * H + h) * dv * d;
  float S[CN][RPL];
#pragma unroll
  for (int c = 0; c < CN; ++c)
#pragma unroll
    for (int x = 0; x < RPL; ++x) S[c][x] = 0.f;
  if (pos0[s] > 0) {
#pragma unroll
    for (int c = 0; c < CN; ++c) {
      const int col = c0 + lc + c;
      if (col >= dv) continue;
#pragma unroll
      for (int m = 0; m < RPL / 4; ++m) {
        const int i0 = 64 * m + 4 * ns;
        const float* p = sp + (size_t)col * d + i0;
        if (vec) {
          if (i0 < d) {
            const float4 v = *reinterpret_cast<const float4*>(p);
            S[c][4 * m] = v.x; S[c][4 * m + 1] = v.y; S[c][4 * m + 2] = v.z; S[c][4 * m + 3] = v.w;
          }
        } else {
#pragma unroll
          for (int x = 0; x < 4; ++x) if (i0 + x < d) S[c][4 * m + x] = p[x];
        }
      }
    }
  }
  // staging: sixteen threads a row (row tid / 16 of the TT), each the same channels as its state rows; one round ahead
  const int wrow = tid >> 4;
  float nq[RPL], nk[RPL], ng[RPL], nv[NV], nb = 0.f;
#pragma unroll
  for (int x = 0; x < RPL; ++x) { nq[x] = 0.f; nk[x] = 0.f; ng[x] = 0.f; }
  auto load = [&](int t0) {
    const int t = t0 + wrow;
    if (wrow < TT && t < a1) {
      const float* qp = qkv + (size_t)t * ldq + (size_t)hq * d;
      const float* kp = qp + (size_t)G * d;
      const float* gp = decay + (size_t)t * ldd + (size_t)h * d;
#pragma unroll
      for (int m = 0; m < RPL / 4; ++m) {
        const int i0 = 64 * m + 4 * ns;
        if (vec) {
          if (i0 < d) {
            const float4 a = *reinterpret_cast<const float4*>(qp + i0), b = *reinterpret_cast<const float4*>(kp + i0),
                         g4 = *reinterpret_cast<const float4*>(gp + i0);
            nq[4 * m] = a.x; nq[4 * m + 1] = a.y; nq[4 * m + 2] = a.z; nq[4 * m + 3] = a.w;
            nk[4 * m] = b.x; nk[4 * m + 1] = b.y; nk[4 * m + 2] = b.z; nk[4 * m + 3] = b.w;
            ng[4 * m] = g4.x; ng[4 * m + 1] = g4.y; ng[4 * m + 2] = g4.z; ng[4 * m + 3] = g4.w;
          }
        } else {
#pragma unroll
          for (int x = 0; x < 4; ++x)
            if (i0 + x < d) { nq[4 * m + x] = qp[i0 + x]; nk[4 * m + x] = kp[i0 + x]; ng[4 * m + x] = gp[i0 + x]; }
        }
      }
      if (ns == 0) nb = beta[(size_t)t * ldb + h];
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int e = tid + 64 * WAVES * x, tt = e / COLS, c = e % COLS;
      nv[x] = tt < TT && t0 + tt < a1 && c0 + c < dv ? qkv[(size_t)(t0 + tt) * ldq + (size_t)2 * G * d + (size_t)h * dv + c0 + c] : 0.f;
    }
  };
  load(a0);
  for (int t0 = a0; t0 < a1; t0 += TT) {
    const int rows = min(TT, a1 - t0);
    __syncthreads();                                 // (the last round's readers are done)
    if (wrow < TT) {                                 // (uniform over a row of 16 lanes: all of them take part in the sums)
      float qq = 0.f, kk = 0.f, qk = 0.f;
#pragma unroll
      for (int x = 0; x < RPL; ++x) { qq += nq[x] * nq[x]; kk += nk[x] * nk[x]; qk += nq[x] * nk[x]; }
      qq = row16_sum(qq); kk = row16_sum(kk); qk = row16_sum(qk);
      const float rq = q_scale / sqrtf(qq + unit_eps), rk = 1.f / sqrtf(kk + unit_eps);
#pragma unroll
      for (int m = 0; m < RPL / 4; ++m) {
        const int i0 = 64 * m + 4 * ns;
        *reinterpret_cast<float4*>(&sq[wrow][i0]) = make_float4(nq[4 * m] * rq, nq[4 * m + 1] * rq, nq[4 * m + 2] * rq, nq[4 * m + 3] * rq);
        *reinterpret_cast<float4*>(&sk[wrow][i0]) = make_float4(nk[4 * m] * rk, nk[4 * m + 1] * rk, nk[4 * m + 2] * rk, nk[4 * m + 3] * rk);
        *reinterpret_cast<float4*>(&sg[wrow][i0]) = make_float4(ng[4 * m], ng[4 * m + 1], ng[4 * m + 2], ng[4 * m + 3]);
      }
      if (ns == 0) { sb[wrow] = sigmoid_f(nb); sqk[wrow] = qk * rq * rk; }
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int e = tid + 64 * WAVES * x;
      if (e < TT * COLS) sv[e / COLS][e % COLS] = nv[x];
    }
    __syncthreads();
    load(t0 + TT);
#pragma unroll 1
    for (int j = 0; j < rows; ++j) {                 // (no barrier in here: a lane's columns are its own)
      float p1[CN], p2[CN];
      float kf[RPL];
#pragma unroll
      for (int c = 0; c < CN; ++c) { p1[c] = 0.f; p2[c] = 0.f; }
#pragma unroll
      for (int m = 0; m < RPL / 4; ++m) {
        const float4 k4 = *reinterpret_cast<const float4*>(&sk[j][64 * m + 4 * ns]);
        const float4 q4 = *reinterpret_cast<const float4*>(&sq[j][64 * m + 4 * ns]);
        const float4 g4 = *reinterpret_cast<const float4*>(&sg[j][64 * m + 4 * ns]);
        kf[4 * m] = k4.x; kf[4 * m + 1] = k4.y; kf[4 * m + 2] = k4.z; kf[4 * m + 3] = k4.w;
        const float gf[4] = {g4.x, g4.y, g4.z, g4.w}, qf[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
        for (int c = 0; c < CN; ++c)
#pragma unroll
          for (int x = 0; x < 4; ++x) {
            S[c][4 * m + x] *= gf[x];
            p1[c] += kf[4 * m + x] * S[c][4 * m + x];
            p2[c] += qf[x] * S[c][4 * m + x];
          }
      }
      const float bj = sb[j], qkj = sqk[j];
#pragma unroll
      for (int c = 0; c < CN; ++c) { p1[c] = row16_sum(p1[c]); p2[c] = row16_sum(p2[c]); }
#pragma unroll
      for (int c = 0; c < CN; ++c) {
        const float u = bj * (sv[j][lc + c] - p1[c]);
#pragma unroll
        for (int x = 0; x < RPL; ++x) S[c][x] += kf[x] * u;
        p2[c] += u * qkj;
      }
      if constexpr (FUSED) {
        if (ns == 0) {
#pragma unroll
          for (int c = 0; c < CN; ++c) so[lc + c] = c0 + lc + c < dv ? p2[c] : 0.f;
        }
        __syncthreads();                             // (rows is the same for the whole block)
        float ss = 0.f;
        for (int c = lane; c < dv; c += 64) ss += so[c] * so[c];
        const float rs = 1.f / sqrtf(wave_sum(ss) / (float)dv + norm_eps);
        for (int c = tid; c < dv; c += 64 * WAVES)
          stf(out + (size_t)(t0 + j) * ldo + (size_t)h * dv, c,
              so[c] * rs * norm_w[c] * sigmoid_f(gate[(size_t)(t0 + j) * ldg + (size_t)h * dv + c]));
        __syncthreads();
      } else {
        if (ns == 0) {
#pragma unroll
          for (int c = 0; c < CN; ++c)
            if (c0 + lc + c < dv) stf(out + (size_t)(t0 + j) * ldo + (size_t)h * dv, c0 + lc + c, p2[c]);
        }
      }
    }
  }
#pragma unroll
  for (int c = 0; c < CN; ++c) {
    const int col = c0 + lc + c;
    if (col >= dv) continue;
#pragma unroll
    for (int m = 0; m < RPL / 4; ++m) {
      const int i0 = 64 * m + 4 * ns;
      float* p = sp + (size_t)col * d + i0;
      if (vec) {
        if (i0 < d) *reinterpret_cast<float4*>(p) = make_float4(S[c][4 * m], S[c][4 * m + 1], S[c][4 * m + 2], S[c][4 * m + 3]);
      } else {
#pragma unroll
        for (int x = 0; x < 4; ++x) if (i0 + x < d) p[x] = S[c][4 * m + x];
      }
    }
  }
}

// one wave per (row, head): o over its root mean square in the head, weight, gate
template <typename TO>
__global__ __launch_bounds__(256) void gated_delta_out_kernel(const float* __restrict__ raw, const float* __restrict__ gate, int ldg,
                                                              const float* __restrict__ norm_w, TO* __restrict__ out, int ldo, int H,
                                                              int dv, float norm_eps, int items) {
  const int lane = threadIdx.x & 63;
  const int item = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= items) return;
  const int t = item / H, h = item % H;
  const float* o = raw + (size_t)t * H * dv + (size_t)h * dv;
  float v[8], ss = 0.f;
#pragma unroll
  for (int e = 0; e < 8; ++e) { const int c = lane + 64 * e; v[e] = c < dv ? o[c] : 0.f; ss += v[e] * v[e]; }
  const float rs = 1.f / sqrtf(wave_sum(ss) / (float)dv + norm_eps);
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    const int c = lane + 64 * e;
    if (c < dv) stf(out + (size_t)t * ldo + (size_t)h * dv, c, v[e] * rs * norm_w[c] * sigmoid_f(gate[(size_t)t * ldg + (size_t)h * dv + c]));
  }
}

extern "C" int fls_seq_gated_delta_scan(const float* qkv, int ldq, const float* beta, int ldb, const float* decay, int ldd,
                                        const float* gate, int ldg, const float* norm_w, float* state, float* raw, void* out, int to,
                                        int ldo, const int* cu, const int* pos0, const int* slot, int T, int B, int one_row_each,
                                        int H, int G, int d, int dv, float q_scale, float unit_eps, float norm_eps, fls_stream_t s) {
  if (T <= 0 || B <= 0) return 0;
  if (d < 1 || d > 256 || dv < 1 || dv > 512 || H < 1 || G < 1 || H % G) return -1;
  const int vec = d % 4 == 0 && ldq % 4 == 0 && ldd % 4 == 0 && (uintptr_t)qkv % 16 == 0 && (uintptr_t)decay % 16 == 0 &&
                  (uintptr_t)state % 16 == 0;
  hipStream_t st = (hipStream_t)s;
  const int rpl = d <= 64 ? 4 : (d <= 128 ? 8 : 16);
#define GD_ARGS qkv, ldq, beta, ldb, decay, ldd, gate, ldg, norm_w, state
#define GD_TAIL cu, pos0, slot, H, G, d, dv, q_scale, unit_eps, norm_eps, vec
  if (one_row_each && T == B) {                      // decoding: a head's columns in one block, finished there
    int cn = 1;
    while (32 * cn < dv) cn *= 2;
    if (rpl * cn <= 64) {
#define GD_F_(R, C, TO_) hipLaunchKernelGGL((gated_delta_kernel<R, C, 8, 1, true, TO_>), dim3(1, H, B), dim3(512), 0, st, GD_ARGS, (TO_*)out, ldo, GD_TAIL)
#define GD_F(R, C) do { if (to == 1) GD_F_(R, C, bf16_t); else GD_F_(R, C, float); } while (0)
      if (rpl == 4) { if (cn == 1) GD_F(4, 1); else if (cn == 2) GD_F(4, 2); else if (cn == 4) GD_F(4, 4); else if (cn == 8) GD_F(4, 8); else GD_F(4, 16); }
      else if (rpl == 8) { if (cn == 1) GD_F(8, 1); else if (cn == 2) GD_F(8, 2); else if (cn == 4) GD_F(8, 4); else GD_F(8, 8); }
      else { if (cn == 1) GD_F(16, 1); else if (cn == 2) GD_F(16, 2); else GD_F(16, 4); }
#undef GD_F
#undef GD_F_
      SEQ_LAUNCH_CHECK();
      return 0;
    }
  }
  if (raw == nullptr) return -1;
  // as many columns a lane as still leave the chip two waves per SIMD: the factors read from LDS serve them all
  int cn = rpl == 16 ? 2 : 4;
  while (cn > 1 && (long long)H * B * ((dv + 16 * cn - 1) / (16 * cn)) * 4 < 2048) cn /= 2;
#define GD_P(R, C) hipLaunchKernelGGL((gated_delta_kernel<R, C, 4, 16, false, float>), dim3((dv + 16 * C - 1) / (16 * C), H, B), dim3(256), 0, st, \
                                      GD_ARGS, raw, H * dv, GD_TAIL)
  if (rpl == 4) { if (cn == 1) GD_P(4, 1); else if (cn == 2) GD_P(4, 2); else GD_P(4, 4); }
  else if (rpl == 8) { if (cn == 1) GD_P(8, 1); else if (cn == 2) GD_P(8, 2); else GD_P(8, 4); }
  else { if (cn == 1) GD_P(16, 1); else GD_P(16, 2); }
#undef GD_P
#undef GD_ARGS
#undef GD_TAIL
  SEQ_LAUNCH_CHECK();
  const int items = T * H;
  if (to == 1) hipLaunchKernelGGL((gated_delta_out_kernel<bf16_t>), dim3((items + 3) / 4), dim3(256), 0, st, raw, gate, ldg, norm_w, (bf16_t*)out, ldo, H, dv, norm_eps, items);
  else hipLaunchKernelGGL((gated_delta_out_kernel<float>), dim3((items + 3) / 4), dim3(256), 0, st, raw, gate, ldg, norm_w, (float*)out, ldo, H, dv, norm_eps, items);
  SEQ_LAUNCH_CHECK();
  return 0;
}
