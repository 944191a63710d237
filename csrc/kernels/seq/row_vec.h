// VE neighbouring entries of a row as one load or store (VE = 4: 16 bytes of fp32, 8 of bf16; VE = 1: any alignment).
#pragma once
#include "seq_common.h"

template <int VE> struct RowVec { float v[VE]; };
template <int VE>
__device__ __forceinline__ RowVec<VE> row_load(const float* p) {
  RowVec<VE> r;
  if constexpr (VE == 4) {
    const float4 q = *reinterpret_cast<const float4*>(p);
    r.v[0] = q.x; r.v[1] = q.y; r.v[2] = q.z; r.v[3] = q.w;
  } else {
    r.v[0] = p[0];
  }
  return r;
}
template <int VE>
__device__ __forceinline__ void row_store(float* p, const RowVec<VE>& r) {
  if constexpr (VE == 4) *reinterpret_cast<float4*>(p) = make_float4(r.v[0], r.v[1], r.v[2], r.v[3]);
  else p[0] = r.v[0];
}
template <int VE>
__device__ __forceinline__ void row_store(bf16_t* p, const RowVec<VE>& r) {
  if constexpr (VE == 4) {
    const bf16_t e[4] = {f_to_bf16(r.v[0]), f_to_bf16(r.v[1]), f_to_bf16(r.v[2]), f_to_bf16(r.v[3])};
    *reinterpret_cast<uint2*>(p) = *reinterpret_cast<const uint2*>(e);
  } else {
    p[0] = f_to_bf16(r.v[0]);
  }
}
template <int VE>
__device__ __forceinline__ RowVec<VE> row_load(const bf16_t* p) {
  RowVec<VE> r;
  if constexpr (VE == 4) {
    const uint2 q = *reinterpret_cast<const uint2*>(p);
    r.v[0] = __uint_as_float(q.x << 16); r.v[1] = __uint_as_float(q.x & 0xffff0000u);
    r.v[2] = __uint_as_float(q.y << 16); r.v[3] = __uint_as_float(q.y & 0xffff0000u);
  } else {
    r.v[0] = bf16_to_f(p[0]);
  }
  return r;
}
