// Shared helpers of the latent attention kernels (K14).
#pragma once
#include "common.h"

#include <type_traits>
#include <utility>

typedef __attribute__((ext_vector_type(8))) __bf16 mv_bf16x8;
typedef __attribute__((ext_vector_type(8))) _Float16 mv_f16x8;

template <typename Tag>
__device__ __forceinline__ f32x4 mfma16x16x32(const u32x4 &a, const u32x4 &b, const f32x4 &c) {
  if constexpr (__is_same(Tag, bf16_tag))
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(mv_bf16x8, a), __builtin_bit_cast(mv_bf16x8, b), c, 0, 0, 0);
  else
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(mv_f16x8, a), __builtin_bit_cast(mv_f16x8, b), c, 0, 0, 0);
}

// two fp32 -> two 16-bit values in one register (one conversion instruction)
template <typename Tag>
__device__ __forceinline__ uint32_t pack_pair(float lo, float hi) {
  if constexpr (__is_same(Tag, bf16_tag))
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(f32x2{lo, hi}, bf16x2_t));
  else
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(f32x2{lo, hi}, f16x2_t));
}
template <typename Tag>
__device__ __forceinline__ u32x2 pack_quad(const f32x4 &v) { return u32x2{pack_pair<Tag>(v[0], v[1]), pack_pair<Tag>(v[2], v[3])}; }

// one 16-byte vector of a row
template <typename Tag>
__device__ __forceinline__ void load_vec_row(const typename elem<Tag>::T *p, float (&f)[elem<Tag>::VEC]) {
  const u32x4 raw = *reinterpret_cast<const u32x4 *>(p);
  if constexpr (elem<Tag>::VEC == 8) {
    unpack8<Tag>(raw, f);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) f[i] = u2f(raw[i]);
  }
}
template <typename Tag>
__device__ __forceinline__ void store_vec_row(typename elem<Tag>::T *p, const float (&f)[elem<Tag>::VEC]) {
  u32x4 raw;
  if constexpr (elem<Tag>::VEC == 8) {
    raw = pack8<Tag>(f);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) raw[i] = f2u(f[i]);
  }
  *reinterpret_cast<u32x4 *>(p) = raw;
}

// ---- hand-counted LDS reads.  The compiler puts a wait for every outstanding LDS-DMA in front of an LDS read it can see, since
// the transfer might write what is read; with tiles in flight to OTHER buffers that wait is the whole memory latency.  These
// reads are opaque to it and are retired by counted waits that name the fragment as an operand, so that no use moves above its
// wait.  LDS operations complete in order, so a count of one's own newer reads is safe beside LDS operations of the compiler's;
// scalar loads share the counter out of order and must not be outstanding.
__device__ __forceinline__ uint32_t lds_address(const void *p) {
  return (uint32_t)(uintptr_t)(__attribute__((address_space(3))) const char *)p;
}
template <int OFF>
__device__ __forceinline__ void lds_read128(u32x4 &d, uint32_t a) {
  asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(d) : "v"(a), "i"(OFF) : "memory");
}
template <int OFF>
__device__ __forceinline__ void lds_read32(float &d, uint32_t a) {
  asm volatile("ds_read_b32 %0, %1 offset:%2" : "=v"(d) : "v"(a), "i"(OFF) : "memory");
}
template <int OFF>
__device__ __forceinline__ void lds_read64_tr(u32x2 &d, uint32_t a) {
  asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(d) : "v"(a), "i"(OFF) : "memory");
}
template <int N, typename V>
__device__ __forceinline__ void lds_wait(V &a) {
  asm volatile("s_waitcnt lgkmcnt(%1)" : "+v"(a) : "n"(N));
}
template <int N, typename V>
__device__ __forceinline__ void lds_wait(V &a, V &b) {
  asm volatile("s_waitcnt lgkmcnt(%2)" : "+v"(a), "+v"(b) : "n"(N));
}
// the registers count as written here: loads into them are waited for now, not (with everything newer) at their first use
template <int N>
__device__ __forceinline__ void settle(u32x4 (&v)[N]) {
#pragma unroll
  for (int i = 0; i < N; ++i) asm volatile("" : "+v"(v[i]));
}
// workgroup barrier that leaves transfers to LDS in flight (__syncthreads waits for all of them)
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }
// compile-time loop: f(integral_constant<int, 0>) ... f(integral_constant<int, N - 1>)
template <typename F, int... I>
__device__ __forceinline__ void static_for_impl(F &&f, std::integer_sequence<int, I...>) {
  (f(std::integral_constant<int, I>{}), ...);
}
template <int N, typename F>
__device__ __forceinline__ void static_for(F &&f) {
  static_for_impl(f, std::make_integer_sequence<int, N>{});
}

// let kernel K use the CU's whole LDS (once per process)
template <auto K>
static inline int mv_allow_lds() {
  static const hipError_t rc = hipFuncSetAttribute((const void *)K, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  return mv_check_hip(rc);
}

// vector-ALU forms (every dtype and size)
int mv_latent_decode_simple_launch(const void *q, const void *plane, const int32_t *tables, int64_t table_stride,
                                   const int32_t *lens, void *out, int batch, int heads, int kv_cols, int rot_cols,
                                   int block_size, int max_blocks, int64_t num_blocks, int window, float scale, int dtype,
                                   hipStream_t stream);
int mv_latent_prefill_simple_launch(const MvLatentPrefillArgs &a, int dtype, hipStream_t stream);
// matrix-core forms; MV_E_SHAPE when they do not apply
size_t mv_latent_decode_mfma_workspace(int batch, int heads, int kv_cols, int rot_cols, int block_size, int max_blocks, int window);
int mv_latent_decode_mfma_launch(const void *q, const void *plane, const int32_t *tables, int64_t table_stride,
                                 const int32_t *lens, void *out, int batch, int heads, int kv_cols, int rot_cols,
                                 int block_size, int max_blocks, int64_t num_blocks, int window, float scale, void *workspace,
                                 size_t workspace_bytes, int dtype, hipStream_t stream);
int mv_latent_prefill_mfma_launch(const MvLatentPrefillArgs &a, int dtype, hipStream_t stream);
