// Shared device helpers for the gfx950 kernels of libmvhip.so.
// wave = 64 lanes everywhere; "row" = one 16-lane DPP row.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

#include "../../include/mvhip.h"

#define MV_WAVE 64
// explicit address spaces for accesses through pointers whose provenance the compiler cannot see (pointers read from
// memory, pointers carried in structs): without them such accesses become flat_ instructions
#define MV_AS1 __attribute__((address_space(1)))
#define MV_AS3 __attribute__((address_space(3)))

typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2_t;
typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
typedef __attribute__((ext_vector_type(2))) uint32_t u32x2;
typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(2))) float f32x2;

typedef __attribute__((ext_vector_type(2))) _Float16 f16x2_t;

// NOTE: never __builtin_bit_cast an ext-vector ELEMENT lvalue (v[i]) directly: clang
// (ROCm 7.2) reads the vector's first element for every i.  Go through these by-value helpers.
__device__ __forceinline__ float u2f(uint32_t u) { return __builtin_bit_cast(float, u); }
__device__ __forceinline__ uint32_t f2u(float f) { return __builtin_bit_cast(uint32_t, f); }
__device__ __forceinline__ bf16x2_t u2bf2(uint32_t u) { return __builtin_bit_cast(bf16x2_t, u); }
__device__ __forceinline__ f16x2_t u2h2(uint32_t u) { return __builtin_bit_cast(f16x2_t, u); }

struct bf16_tag {};
struct f16_tag {};
struct f32_tag {};

// ---- scalar conversions -------------------------------------------------
__device__ __forceinline__ float bf16_bits_to_f32(uint32_t hi16) {
  return __builtin_bit_cast(float, hi16 << 16);
}
// round-to-nearest-even, NaN preserved (v_cvt_pk_bf16_f32 on gfx950)
__device__ __forceinline__ uint16_t f32_to_bf16_bits(float f) {
  __bf16 b = (__bf16)f;
  return __builtin_bit_cast(uint16_t, b);
}
__device__ __forceinline__ float f16_bits_to_f32(uint16_t h) {
  return (float)__builtin_bit_cast(_Float16, h);
}
__device__ __forceinline__ uint16_t f32_to_f16_bits(float f) {
  _Float16 h = (_Float16)f;
  return __builtin_bit_cast(uint16_t, h);
}

// Element traits: T = storage type, 16-byte vector holds VEC elements.
template <typename Tag> struct elem;
template <> struct elem<bf16_tag> {
  typedef uint16_t T;
  static constexpr int VEC = 8;
  static __device__ __forceinline__ float ld(uint16_t v) { return bf16_bits_to_f32(v); }
  static __device__ __forceinline__ uint16_t st(float f) { return f32_to_bf16_bits(f); }
};
template <> struct elem<f16_tag> {
  typedef uint16_t T;
  static constexpr int VEC = 8;
  static __device__ __forceinline__ float ld(uint16_t v) { return f16_bits_to_f32(v); }
  static __device__ __forceinline__ uint16_t st(float f) { return f32_to_f16_bits(f); }
};
template <> struct elem<f32_tag> {
  typedef float T;
  static constexpr int VEC = 4;
  static __device__ __forceinline__ float ld(float v) { return v; }
  static __device__ __forceinline__ float st(float f) { return f; }
};

// Unpack one 16-byte vector (8 x 16-bit) into 8 floats.
template <typename Tag>
__device__ __forceinline__ void unpack8(const u32x4 &v, float (&f)[8]) {
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    if constexpr (__is_same(Tag, bf16_tag)) {
      f[2 * i] = u2f(v[i] << 16);
      f[2 * i + 1] = u2f(v[i] & 0xffff0000u);
    } else {
      f[2 * i] = f16_bits_to_f32((uint16_t)(v[i] & 0xffffu));
      f[2 * i + 1] = f16_bits_to_f32((uint16_t)(v[i] >> 16));
    }
  }
}
template <typename Tag>
__device__ __forceinline__ u32x4 pack8(const float (&f)[8]) {
  u32x4 v;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    uint32_t lo = elem<Tag>::st(f[2 * i]);
    uint32_t hi = elem<Tag>::st(f[2 * i + 1]);
    v[i] = lo | (hi << 16);
  }
  return v;
}

// ---- cross-lane ----------------------------------------------------------
// DPP row rotate within each 16-lane row; ctrl = 0x120 + n (row_ror:n).
template <int N>
__device__ __forceinline__ float row_ror(float x) {
  int xi = __builtin_bit_cast(int, x);
  int r = __builtin_amdgcn_update_dpp(0, xi, 0x120 + N, 0xf, 0xf, false);
  return __builtin_bit_cast(float, r);
}
// Sum over the 16 lanes of a DPP row; every lane of the row gets the total.
__device__ __forceinline__ float row16_sum(float x) {
  x += row_ror<8>(x);
  x += row_ror<4>(x);
  x += row_ror<2>(x);
  x += row_ror<1>(x);
  return x;
}
__device__ __forceinline__ float row16_max(float x) {
  x = fmaxf(x, row_ror<8>(x));
  x = fmaxf(x, row_ror<4>(x));
  x = fmaxf(x, row_ror<2>(x));
  x = fmaxf(x, row_ror<1>(x));
  return x;
}
// Full 64-lane reductions (every lane gets the result).
__device__ __forceinline__ float wave_sum(float x) {
  x = row16_sum(x);
  x += __shfl_xor(x, 16, 64);
  x += __shfl_xor(x, 32, 64);
  return x;
}
__device__ __forceinline__ float wave_max(float x) {
  x = row16_max(x);
  x = fmaxf(x, __shfl_xor(x, 16, 64));
  x = fmaxf(x, __shfl_xor(x, 32, 64));
  return x;
}

// tanh form of gelu: 0.5 z (1 + tanh(u)) = z / (1 + exp(-2 u)), u = sqrt(2/pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gelu_tanh(float z) {
  const float u2 = 1.5957691216057308f * (z + 0.044715f * z * z * z);
  return z / (1.0f + expf(-u2));
}

// 0.5 z (1 + erf(z / sqrt(2))).  16-bit operands: erfc by Abramowitz & Stegun 7.1.26 (absolute error 1.5e-7), hardware exponential
// and reciprocal; max(z, 0) - |z| / 2 erfc(|z| / sqrt(2)) holds on both sides
template <typename Tag>
__device__ __forceinline__ float gelu_erf(float z) {
  if constexpr (__is_same(Tag, f32_tag)) {
    return 0.5f * z * (1.0f + erff(z * 0.7071067811865476f));
  } else {
    const float a = fabsf(z), t = __builtin_amdgcn_rcpf(fmaf(0.3275911f * 0.7071067811865476f, a, 1.0f));
    const float poly = t * fmaf(t, fmaf(t, fmaf(t, fmaf(t, 1.061405429f, -1.453152027f), 1.421413741f), -0.284496736f), 0.254829592f);
    return fmaxf(z, 0.f) - 0.5f * a * poly * __builtin_amdgcn_exp2f(-0.7213475204444817f * a * a);   // exp(-z^2 / 2)
  }
}
// 16-bit operands: hardware exponential and reciprocal (1 ulp of fp32 each)
template <typename Tag>
__device__ __forceinline__ float sigmoid_of(float z) {
  if constexpr (__is_same(Tag, f32_tag)) return 1.0f / (1.0f + expf(-z));
  else return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z));
}

// clamped gate: g = min(gate, limit), u = clamp(up, -limit, limit): g sigmoid(alpha g) (u + 1)
__device__ __forceinline__ float clamped_glu(float gate, float up, float limit, float alpha) {
  const float g = fminf(gate, limit), u = fminf(fmaxf(up, -limit), limit);
  return g / (1.0f + expf(-alpha * g)) * (u + 1.0f);
}

// act(gate) * up on the fp32 accumulators of a gated projection.  gelu, clamped, relu: fp32 throughout.  silu: the rounding points
// of the unfused pair (GEMM -> dtype, silu -> dtype, product in fp32; the caller rounds it)
template <typename Tag>
__device__ __forceinline__ float gated_act(float gate, float up, const MvGateAct &a) {
  if (a.kind == MV_ACT_GELU) return __fmul_rn(gelu_tanh(gate), up);
  if (a.kind == MV_ACT_CLAMPED) return clamped_glu(gate, up, a.limit, a.alpha);
  if (a.kind == MV_ACT_RELU) return __fmul_rn(fmaxf(gate, 0.f), up);
  const float gt = elem<Tag>::ld(elem<Tag>::st(gate)), ut = elem<Tag>::ld(elem<Tag>::st(up));
  float sl = gt / (1.0f + expf(-gt));                        // rmsnorm.hip: silu_and_mul_kernel
  sl = elem<Tag>::ld(elem<Tag>::st(sl));
  return __fmul_rn(sl, ut);
}

// ---- rotary embedding ------------------------------------------------------
// A head row of D elements lies on LPT = D / VEC adjacent lanes, VEC per lane (sub = lane within the row).  Two layouts:
//   halves (NeoX):  dim i pairs with dim i + D/2, i < D/2; the partner sits LPT/2 lanes away; cos / sin [max_pos, D/2]
//   interleaved:    dim 2i pairs with dim 2i + 1, i < pairs, in the same lane; dims from 2 * pairs on pass unchanged;
//                   cos / sin [max_pos, pairs]
template <int D, int VEC>
__device__ __forceinline__ void rot_factors(const float *cos, const float *sin, int64_t pos, bool pos_ok, int sub,
                                            int pairs, bool interleaved, float (&cs)[VEC], float (&sn)[VEC]) {
  constexpr int HALF = D / VEC / 2;
  if (interleaved) {
    // (clamped addresses and a select behind the loads: no branch around each of them)
    const int64_t base = pos_ok ? pos * pairs : 0;
#pragma unroll
    for (int j = 0; j < VEC; j += 2) {
      const int i = (sub * VEC + j) >> 1;
      float c = 1.0f, s = 0.0f;
      if (pairs > 0) {   // (uniform)
        const int ic = i < pairs ? i : pairs - 1;
        c = cos[base + ic], s = sin[base + ic];
      }
      const bool ok = pos_ok && i < pairs;
      cs[j] = cs[j + 1] = ok ? c : 1.0f;
      sn[j] = sn[j + 1] = ok ? s : 0.0f;
    }
  } else {
    const int i0 = (sub % HALF) * VEC;
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      cs[j] = pos_ok ? cos[pos * (D / 2) + i0 + j] : 1.0f;
      sn[j] = pos_ok ? sin[pos * (D / 2) + i0 + j] : 0.0f;
    }
  }
}
// y = rotation of x; every product and sum rounded on its own
template <int D, int VEC>
__device__ __forceinline__ void rot_apply(const float (&x)[VEC], const float (&cs)[VEC], const float (&sn)[VEC], int sub,
                                          bool interleaved, float (&y)[VEC]) {
  constexpr int LPT = D / VEC, HALF = LPT / 2;
  if (interleaved) {
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      const float a = __fmul_rn(x[j], cs[j]), b = __fmul_rn(x[j ^ 1], sn[j]);
      y[j] = (j & 1) ? __fadd_rn(a, b) : __fsub_rn(a, b);
    }
  } else {
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      float other;
      if constexpr (LPT == 16) other = row_ror<8>(x[j]);
      else other = __shfl_xor(x[j], HALF, 64);
      const float a = __fmul_rn(x[j], cs[j]), b = __fmul_rn(other, sn[j]);
      y[j] = sub < HALF ? __fsub_rn(a, b) : __fadd_rn(a, b);
    }
  }
}

// ---- host-side helpers ------------------------------------------------------
static inline int mv_check_act(const MvGateAct *a) {
  if (!a) return MV_E_NULLPTR;
  if (a->kind < MV_ACT_SILU || a->kind > MV_ACT_RELU) return MV_E_RANGE;
  return a->kind == MV_ACT_CLAMPED && !(a->limit > 0.f) ? MV_E_RANGE : MV_OK;
}
static inline int mv_check_hip(hipError_t e) { return e == hipSuccess ? 0 : (int)e; }
static inline bool mv_aligned16(const void *p) { return (((uintptr_t)p) & 15u) == 0; }

// ---- what a query sees and how its scores become weights (MvAttnOpts) --------------------------------------------------
struct AttnMask {
  int window = 0, keep_first = 0;   // window > 0: key j of position i if i - j < window or j < keep_first
  float softcap = 0.f, out_scale = 1.f;
  const void *sink = nullptr;       // [heads] of dtype: one more term of the denominator
  const void *gate = nullptr;       // a row of [heads * D] per query: the output is multiplied by its sigmoid
  int64_t gate_stride = 0;
};
// what an output element is multiplied by
template <typename Tag>
__device__ __forceinline__ float attn_factor(const AttnMask &m, int64_t row, int col) {
  if (!m.gate) return m.out_scale;
  return m.out_scale * sigmoid_of<Tag>(elem<Tag>::ld(((const typename elem<Tag>::T *)m.gate)[row * m.gate_stride + col]));
}
static inline AttnMask mv_attn_mask(const MvAttnOpts *o) {
  AttnMask m;
  if (o) {
    m.window = o->window, m.keep_first = o->window > 0 ? o->keep_first : 0, m.softcap = o->softcap, m.sink = o->sink;
    if (o->out_scale != 0.f) m.out_scale = o->out_scale;
    m.gate = o->gate, m.gate_stride = o->gate_stride;
  }
  return m;
}
static inline int mv_check_mask(const MvAttnOpts *o) {
  if (!o) return MV_OK;
  if (o->chunk < 0 || o->window < 0 || o->keep_first < 0 || (o->chunk > 0 && o->window > 0)) return MV_E_SHAPE;
  if (o->gate && (!mv_aligned16(o->gate) || (o->gate_stride & 7))) return MV_E_ALIGN;
  return o->softcap < 0.f ? MV_E_RANGE : MV_OK;
}
// most keys that one query reads, in whole units; 0 = no bound
static inline int64_t mv_attn_span(const MvAttnOpts *o, int unit) {
  if (!o) return 0;
  if (o->chunk > 0) return (int64_t)o->chunk + unit;   // (a chunk's edge inside a unit)
  if (o->window > 0) return (int64_t)o->window + unit + ((int64_t)o->keep_first + unit - 1) / unit * unit;
  return 0;
}
// cap * tanh(s / cap) in log2 units: `raw` an unscaled score, to_cap = scale / cap, cap_log2 = cap * log2(e)
template <typename Tag>
__device__ __forceinline__ float capped_log2(float raw, float to_cap, float cap_log2) {
  const float z = raw * to_cap;
  if constexpr (__is_same(Tag, f32_tag)) return cap_log2 * tanhf(z);
  // 1 - 2 / (exp(2 z) + 1): hardware exponential and reciprocal, about 1e-7 of the cap
  const float e = __builtin_amdgcn_exp2f(z * 2.8853900817779268f);
  return cap_log2 * (1.f - 2.f * __builtin_amdgcn_rcpf(e + 1.f));
}

// rotary / window options of the attention entry points (NULL = none)
static inline bool mv_needs_tables(const MvAttnOpts *o) { return !(o && o->interleaved && o->rot_pairs == 0); }
static inline int mv_check_rot(const MvAttnOpts *o, int head_dim) {
  if (!o) return MV_OK;
  if (o->norm_dim < 0 || o->norm_dim > head_dim) return MV_E_SHAPE;
  if (o->interleaved) return (o->rot_pairs < 0 || o->rot_pairs > head_dim / 2) ? MV_E_SHAPE : MV_OK;
  return (o->rot_pairs != 0 && o->rot_pairs != head_dim / 2) ? MV_E_SHAPE : MV_OK;   // halves: whole rows only
}

#define MV_LAUNCH_CHECK()                       \
  do {                                          \
    hipError_t _e = hipGetLastError();          \
    if (_e != hipSuccess) return (int)_e;       \
  } while (0)

#define MV_DISPATCH_DTYPE(dtype, ...)                     \
  switch (dtype) {                                        \
    case MV_BF16: { typedef bf16_tag Tag; __VA_ARGS__; } break; \
    case MV_F16:  { typedef f16_tag Tag;  __VA_ARGS__; } break; \
    case MV_F32:  { typedef f32_tag Tag;  __VA_ARGS__; } break; \
    default: return MV_E_DTYPE;                           \
  }
