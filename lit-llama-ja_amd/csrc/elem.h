// Element access of kernels that run in both activation types: bf16 (raw bits) and fp32.
#pragma once
#include "common.h"

namespace llj {

// element access of the activation type: bf16 (the reference's rounding points) or fp32 (none)
template <typename T>
__device__ __forceinline__ float ldv(const T* p, size_t i) {
  if constexpr (sizeof(T) == 2) return bf2f(p[i]);
  else return p[i];
}
template <typename T>
__device__ __forceinline__ void stv(T* p, size_t i, float v) {
  if constexpr (sizeof(T) == 2) p[i] = f2bf(v);
  else p[i] = v;
}
template <typename T>
__device__ __forceinline__ float rnd(float v) {
  if constexpr (sizeof(T) == 2) return round_bf(v);
  else return v;
}

// 8 consecutive elements as fp32 (16-byte aligned)
__device__ __forceinline__ void ld8(const bf16_t* p, float (&o)[8]) {
  const uint4 v = *reinterpret_cast<const uint4*>(p);
  const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    o[2 * i] = bflo(w[i]);
    o[2 * i + 1] = bfhi(w[i]);
  }
}
__device__ __forceinline__ void ld8(const float* p, float (&o)[8]) {
  const float4 a = reinterpret_cast<const float4*>(p)[0], b = reinterpret_cast<const float4*>(p)[1];
  o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w;
  o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
}
__device__ __forceinline__ void st8(bf16_t* p, const float (&v)[8]) {
  *reinterpret_cast<uint4*>(p) = make_uint4(pack2bf(v[0], v[1]), pack2bf(v[2], v[3]), pack2bf(v[4], v[5]), pack2bf(v[6], v[7]));
}
__device__ __forceinline__ void st8(float* p, const float (&v)[8]) {
  reinterpret_cast<float4*>(p)[0] = make_float4(v[0], v[1], v[2], v[3]);
  reinterpret_cast<float4*>(p)[1] = make_float4(v[4], v[5], v[6], v[7]);
}

// clamped gated unit: g * sigmoid(alpha g) * (u + 1), g = min(g, limit), u = clamp(u, -limit, limit)
__device__ __forceinline__ float clamped_glu(float g, float u, float limit, float alpha) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g / (1.f + expf(-alpha * g)) * (u + 1.f);
}

}  // namespace llj

#define LLJ_DT(dt, CALL_BF16, CALL_F32) \
  do {                                 \
    if ((dt) == 0) CALL_BF16;          \
    else CALL_F32;                     \
  } while (0)
