// Four elements at a time, whatever the dtype.
#pragma once
#include "common.h"

template <typename Tag>
struct vec4 {
  typedef typename elem<Tag>::T T;
  typedef f32x4 F;
  static __device__ __forceinline__ F unpack(const u32x2 &r) {
    if constexpr (__is_same(Tag, bf16_tag)) {
      return F{u2f(r[0] << 16), u2f(r[0] & 0xffff0000u), u2f(r[1] << 16), u2f(r[1] & 0xffff0000u)};
    } else {
      return F{f16_bits_to_f32((uint16_t)(r[0] & 0xffffu)), f16_bits_to_f32((uint16_t)(r[0] >> 16)),
               f16_bits_to_f32((uint16_t)(r[1] & 0xffffu)), f16_bits_to_f32((uint16_t)(r[1] >> 16))};
    }
  }
  // as it lies in memory, so that many can be on their way before the first is used
  typedef u32x2 R;
  static __device__ __forceinline__ R raw(const T *p) { return *reinterpret_cast<const u32x2 *>(p); }
  static __device__ __forceinline__ F load(const T *p) { return unpack(raw(p)); }
  static __device__ __forceinline__ void store(T *p, const F &f) {
    const float a = f[0], b = f[1], c = f[2], d = f[3];
    *reinterpret_cast<u32x2 *>(p) = u32x2{(uint32_t)elem<Tag>::st(a) | ((uint32_t)elem<Tag>::st(b) << 16),
                                          (uint32_t)elem<Tag>::st(c) | ((uint32_t)elem<Tag>::st(d) << 16)};
  }
};
template <>
struct vec4<f32_tag> {
  typedef float T;
  typedef f32x4 F;
  typedef f32x4 R;
  static __device__ __forceinline__ F unpack(const R &r) { return r; }
  static __device__ __forceinline__ R raw(const T *p) { return *reinterpret_cast<const f32x4 *>(p); }
  static __device__ __forceinline__ F load(const T *p) { return raw(p); }
  static __device__ __forceinline__ void store(T *p, const F &f) { *reinterpret_cast<f32x4 *>(p) = f; }
};
