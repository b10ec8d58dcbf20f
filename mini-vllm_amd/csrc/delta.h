// Shared helpers of the gated delta rule kernels (K16).
#pragma once
#include "ssm.h"

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }
// log of the decay factor: -exp(a_log) * softplus(a + bias)
__device__ __forceinline__ float decay_log(float rate, float a, float bias) { return -rate * softplus_f32(a + bias); }

// chunked form (16-bit); MV_E_SHAPE when it does not apply
size_t mv_delta_chunk_workspace(int n_seqs, int total_q, int heads, int p, int n);
int mv_delta_chunk_launch(const MvDeltaArgs &a, int dtype, hipStream_t stream);
int mv_delta_scalar_launch(const MvDeltaArgs &a, hipStream_t stream);   // (from the above: bf16, one decay per head)
