// Shared helpers of the state space kernels (K15).
#pragma once
#include "latent.h"

__device__ __forceinline__ float silu_f32(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// chunked form (16-bit); MV_E_SHAPE when it does not apply
int mv_ssm_chunk_launch(const MvSsmArgs &a, int dtype, hipStream_t stream);
