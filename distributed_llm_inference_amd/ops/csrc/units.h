// V consecutive fp32 entries of a row at a time: one 16-byte access (V = 4, aligned) or one element (V = 1, any layout).
#pragma once
#include "common.h"

namespace dlia {

template <int V> struct Unit { float v[V]; };
template <int V> __device__ __forceinline__ Unit<V> ldu(const float* p) {
  Unit<V> u;
  if constexpr (V == 4) {
    const f32x4 t = *reinterpret_cast<const f32x4*>(p);
    u.v[0] = t.x; u.v[1] = t.y; u.v[2] = t.z; u.v[3] = t.w;
  } else {
    u.v[0] = p[0];
  }
  return u;
}
template <int V> __device__ __forceinline__ void stu(float* p, const Unit<V>& u) {
  if constexpr (V == 4) *reinterpret_cast<f32x4*>(p) = f32x4{u.v[0], u.v[1], u.v[2], u.v[3]};
  else p[0] = u.v[0];
}
template <int V> __device__ __forceinline__ void stu(bf16* p, const Unit<V>& u) {
  if constexpr (V == 4) *reinterpret_cast<u32x2*>(p) = u32x2{pack_bf16(u.v[0], u.v[1]), pack_bf16(u.v[2], u.v[3])};
  else p[0] = (bf16)u.v[0];
}

}  // namespace dlia
