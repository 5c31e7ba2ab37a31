// Where an attention cache keeps its elements, and small device pieces the attention kernels share
// (w4a32_pooled_attention.hip, w4a32_latent_attention.hip).
#pragma once

#include "w4a32_layered.h"
#include "w4a32_layered_kernels.h"

namespace w4 {

__device__ __forceinline__ int pooled_visible(int p, int window, int pool) {
  const int before = p - window + 1;  // tokens that lie before the window
  return pool > 0 && before > 0 ? before / pool : 0;
}

// element (entry, dim) of a kv head's keys / values
__device__ __forceinline__ size_t k_at(int entry, int d, int D) {
  return (size_t)(entry >> 5) * (32 * D) + (size_t)((d >> 3) * 32 + (entry & 31)) * 8 + (d & 7);
}
__device__ __forceinline__ int v_pos(int o) { return (o & 16) + 8 * ((o >> 2) & 1) + 4 * ((o >> 3) & 1) + (o & 3); }
__device__ __forceinline__ size_t v_at(int entry, int d, int D) {
  return (size_t)(entry >> 5) * (32 * D) + (size_t)d * 32 + v_pos(entry & 31);
}

__device__ __forceinline__ f32x16 mfma_bf16(bf16x8 a, bf16x8 b, f32x16 c) {
  return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0);
}

// component d of a rotated vector at position p, whose partner is component d + rot / 2 or d - rot / 2; tables
// [rows][rot / 2]
__device__ __forceinline__ float rotated(float x, float partner, int d, int rot, size_t p, const float* __restrict__ sin_t,
                                         const float* __restrict__ cos_t) {
  const int half = rot / 2, i = d < half ? d : d - half;
  const float c = cos_t[p * half + i], s = sin_t[p * half + i];
  return d < half ? x * c - partner * s : x * c + partner * s;
}
__device__ __forceinline__ int rot_partner(int d, int rot) { return d < rot / 2 ? d + rot / 2 : d - rot / 2; }

// eight consecutive elements as they come from memory, and as f32
template <typename T>
struct Eight;
template <>
struct Eight<__bf16> {
  u32x4 v;
  __device__ __forceinline__ void load(const __bf16* p) { v = *reinterpret_cast<const u32x4*>(p); }
  __device__ __forceinline__ float get(int e) const {
    return __uint_as_float(e & 1 ? v[e >> 1] & 0xFFFF0000u : v[e >> 1] << 16);
  }
  __device__ __forceinline__ void set(float4 a, float4 b) {  // values that are bf16 already
    v[0] = (__float_as_uint(a.x) >> 16) | (__float_as_uint(a.y) & 0xFFFF0000u);
    v[1] = (__float_as_uint(a.z) >> 16) | (__float_as_uint(a.w) & 0xFFFF0000u);
    v[2] = (__float_as_uint(b.x) >> 16) | (__float_as_uint(b.y) & 0xFFFF0000u);
    v[3] = (__float_as_uint(b.z) >> 16) | (__float_as_uint(b.w) & 0xFFFF0000u);
  }
};
template <>
struct Eight<float> {
  f32x4 a, b;
  __device__ __forceinline__ void load(const float* p) {
    a = *reinterpret_cast<const f32x4*>(p);
    b = *reinterpret_cast<const f32x4*>(p + 4);
  }
  __device__ __forceinline__ float get(int e) const { return e < 4 ? a[e] : b[e - 4]; }
  __device__ __forceinline__ void set(float4 x, float4 y) {
    a = f32x4{x.x, x.y, x.z, x.w};
    b = f32x4{y.x, y.y, y.z, y.w};
  }
};

}  // namespace w4
