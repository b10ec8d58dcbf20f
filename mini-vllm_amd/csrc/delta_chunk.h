// Shared by the chunked forms of the gated delta rule (K16): delta_chunk.hip, delta_scalar.hip.
#pragma once
#include "delta.h"

namespace {

constexpr int L = 64;              // tokens per chunk

typedef bf16_tag B16;

__device__ __forceinline__ void split8(const float (&f)[8], u32x4 &hi, u32x4 &lo) {
  float rest[8];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    hi[i] = pack_pair<B16>(f[2 * i], f[2 * i + 1]);
    rest[2 * i] = f[2 * i] - u2f(hi[i] << 16);
    rest[2 * i + 1] = f[2 * i + 1] - u2f(hi[i] & 0xffff0000u);
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) lo[i] = pack_pair<B16>(rest[2 * i], rest[2 * i + 1]);
}
__device__ __forceinline__ void split44(const f32x4 &a, const f32x4 &b, u32x4 &hi, u32x4 &lo) {
  const float f[8] = {a[0], a[1], a[2], a[3], b[0], b[1], b[2], b[3]};
  split8(f, hi, lo);
}
__device__ __forceinline__ f32x4 mfma3(const u32x4 &ah, const u32x4 &al, const u32x4 &bh, const u32x4 &bl, f32x4 c) {
  c = mfma16x16x32<B16>(ah, bh, c);
  c = mfma16x16x32<B16>(ah, bl, c);
  return mfma16x16x32<B16>(al, bh, c);
}
// softplus in hardware exponential and logarithm: an absolute error of about 1e-7
__device__ __forceinline__ float softplus_fast(float z) {
  return fmaxf(z, 0.f) + 0.6931471805599453f * __builtin_amdgcn_logf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * fabsf(z)));
}

struct DeltaPrep {
  MvDeltaArgs a;
  char *ws;
};

// chunk slot -> sequence (its slots start at cu_q / L + its number)
__device__ __forceinline__ int chunk_sequence(const MvDeltaArgs &p, int slot) {
  int seq = 0;
  for (int hi = p.n_seqs; hi - seq > 1;) {
    const int mid = (seq + hi) >> 1;
    if (p.cu_q[mid] / L + mid <= slot) seq = mid;
    else hi = mid;
  }
  return seq;
}
inline int64_t chunk_slots(int n_seqs, int total_q) { return (int64_t)total_q / L + n_seqs; }

// the ten blocks of 16 x 16 tokens on and below the diagonal, dealt over the waves
__device__ __forceinline__ void block_place(int idx, int &I, int &J) {
  I = idx < 4 ? 3 : idx < 7 ? 2 : idx < 9 ? 1 : 0, J = idx < 4 ? 3 - idx : idx < 7 ? 6 - idx : idx < 9 ? 8 - idx : 0;
}

// an accumulator as half of an operand, high parts and rests
__device__ __forceinline__ void split4(const f32x4 &f, u32x2 &hi, u32x2 &lo) {
  hi = pack_quad<B16>(f);
  f32x4 rest;
#pragma unroll
  for (int e = 0; e < 2; ++e) {
    rest[2 * e] = f[2 * e] - u2f(hi[e] << 16);
    rest[2 * e + 1] = f[2 * e + 1] - u2f(hi[e] & 0xffff0000u);
  }
  lo = pack_quad<B16>(rest);
}

constexpr int TS = L + 4;   // row stride of A and T in LDS
// operands of a lower triangular matrix of L x L tokens: (token tile, step of 32 tokens) 0 0, 1 0, 2 0, 2 1, 3 0, 3 1
constexpr int kTriangle = 6;
__host__ __device__ constexpr int triangle(int it, int s) { return it < 2 ? it : 2 * it - 2 + s; }

// T = (1 + A)^-1 diag(beta), in place of -A in LDS (-A is there, behind a barrier; so is T afterwards), by the first four waves.  T's entries are
// at most 1, since no factor 1 - beta k k^T of the recurrence lengthens a vector.
__device__ __forceinline__ void solve_chunk(float *ts, const float *bt, int wave, int lane) {
  const int r16 = lane & 15, g = lane >> 4;
  // A wave inverts a diagonal block, a column in each of 16 lanes, into one of the blocks above the diagonal, which nothing uses ..
  auto inverse = [&](int I) { return ts + (I < 3 ? 16 * (I + 1) : 16 * TS + 32); };
  if (wave < 4 && lane < 16) {
    const float *d = ts + 16 * wave * TS + 16 * wave;
    float *to = inverse(wave), x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float a = i == r16 ? 1.f : 0.f, b = 0.f;
#pragma unroll
      for (int j = 0; j < i; j += 4) {   // (zeros from column i on)
        const f32x4 t = *(const f32x4 *)(d + i * TS + j);
        a = fmaf(t[0], x[j], a);
        if (j + 1 < i) b = fmaf(t[1], x[j + 1], b);
        if (j + 2 < i) a = fmaf(t[2], x[j + 2], a);
        if (j + 3 < i) b = fmaf(t[3], x[j + 3], b);
      }
      x[i] = a + b;
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) to[i * TS + r16] = x[i];
  }
  __syncthreads();
  // .. and then a wave a column of blocks, from the diagonal down: T_IJ = T_II sum_{J <= K < I} (-A_IK) T_KJ.  Accumulators are the
  // right operand of the next product, whose keys are 4 g + step.
  f32x4 t[4];
  if (wave < 4) {
    auto product = [&](const float *block, const f32x4 &right, f32x4 acc) {
      const f32x4 left = *(const f32x4 *)(block + r16 * TS + 4 * g);
#pragma unroll
      for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(left[e], right[e], acc, 0, 0, 0);
      return acc;
    };
#pragma unroll
    for (int I = 0; I < 4; ++I) {
      t[I] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (I < wave) continue;
      if (I == wave) {
#pragma unroll
        for (int e = 0; e < 4; ++e) t[I][e] = inverse(I)[(4 * g + e) * TS + r16];
        continue;
      }
      f32x4 sum = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int K = 0; K < I; ++K)
        if (K >= wave) sum = product(ts + 16 * I * TS + 16 * K, t[K], sum);
      t[I] = product(inverse(I), sum, t[I]);
    }
  }
  __syncthreads();   // every wave has read A
  if (wave < 4) {
    const float beta = bt[16 * wave + r16];
#pragma unroll
    for (int I = 0; I < 4; ++I)
      if (I >= wave) {
#pragma unroll
        for (int e = 0; e < 4; ++e) ts[(16 * I + 4 * g + e) * TS + 16 * wave + r16] = t[I][e] * beta;
      }
  }
  __syncthreads();
}

// rows of T as an operand of either side: row r16 of a token tile, tokens 16 (e >> 2) + 4 g + (e & 3) of a step of 32
__device__ __forceinline__ void solution_operand(const float *ts, int m, int lane, u32x4 &hi, u32x4 &lo) {
  const int it = m < 2 ? m : 2 + (m - 2) / 2, s = m < 2 ? 0 : m & 1;
  const float *row = ts + (16 * it + (lane & 15)) * TS + 32 * s + 4 * (lane >> 4);
  const f32x4 a = *(const f32x4 *)row;
  f32x4 b = {0.f, 0.f, 0.f, 0.f};
  if (2 * s + 1 <= it) b = *(const f32x4 *)(row + 16);
  split44(a, b, hi, lo);
}

}  // namespace
