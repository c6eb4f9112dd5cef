// kh_tile.h — the 16x16 matrix-core tile of the layer-list models (kh_lgemm.h, kh_latent.h), written once for the two
// storage types they run in: bf16 (v_mfma_f32_16x16x32_bf16, one instruction per 64-byte k-block) and fp32
// (v_mfma_f32_16x16x4_f32, four instructions per 64-byte k-block: exact fp32).
//
// A FRAGMENT is 16 bytes per lane: lane (i = l & 15, h = l >> 4) holds row i, bytes [16 h, 16 h + 16) of a 64-byte
// k-block of that row - 8 bf16 or 4 fp32 - for either operand, so loads and LDS layouts do not depend on the type.
// Result: lane (j, h) holds elements (m = 4 h + 0..3, n = j), m from the first operand, n from the second.
#pragma once
#include "kh_common.h"

namespace khm {
typedef __bf16 bf16;
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));

template <class T>
struct Tile;
template <>
struct Tile<bf16> {
  typedef bf16x8 frag;
  typedef bf16x4 quad;
  static constexpr int N = 8;  // elements of a 16-byte fragment
  static __device__ __forceinline__ f32x4 mma(const frag& a, const frag& b, f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0);
  }
};
template <>
struct Tile<float> {
  typedef f32x4 frag;
  typedef f32x4 quad;
  static constexpr int N = 4;
  static __device__ __forceinline__ f32x4 mma(const frag& a, const frag& b, f32x4 c) {
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, c, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, c, 0, 0, 0);
  }
};

template <class T>
__device__ __forceinline__ typename Tile<T>::quad to_quad(f32x4 v) {
  typename Tile<T>::quad q;
  q.x = (T)v.x;
  q.y = (T)v.y;
  q.z = (T)v.z;
  q.w = (T)v.w;
  return q;
}

__device__ __forceinline__ float sigmoid1(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float silu1(float z) { return z * sigmoid1(z); }
// Gated unit of a feed-forward: gate times sigmoid(alpha gate) times (up + shift), both sides limited first.  SwiGLU is
// {INFINITY, 1, 0}.
struct GateAct {
  float limit, alpha, shift;
};
__device__ __forceinline__ float gated1(const GateAct& c, float g, float u) {
  g = fminf(g, c.limit);
  u = fminf(fmaxf(u, -c.limit), c.limit);
  return g * sigmoid1(c.alpha * g) * (u + c.shift);
}
// log(1 + e^z) without overflow
__device__ __forceinline__ float softplus1(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
}  // namespace khm
