// Shared helpers of the latent attention kernels (K14).
#pragma once
#include "common.h"

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
