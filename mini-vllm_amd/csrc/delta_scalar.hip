// K16 — gated delta rule of prompts in chunks where a head has one decay (bf16 operands, fp32 state).
//
// With r_i the running sum of the log decays in a chunk, the decays leave the products over channels: with the factors f_i, g_i that scale k
// and q to their lengths, S the state ahead of the chunk and T as in delta_chunk.hip,
//     A_ij = beta_i f_i f_j e^{r_i - r_j} (k_i k_j)      U = T R,  R_i = v_i - e^{r_i} f_i (k_i S)
//     B_ij = g_i f_j e^{r_i - r_j} (q_i k_j)             o_i = e^{r_i} g_i (q_i S) + sum_{j <= i} B_ij u_j
//     S <- e^{r_last} S + sum_j k_j (e^{r_last - r_j} f_j u_j)^T
// so k and q enter every product as they are in memory (exact in bf16) and only T, B, S and U are sums of two bf16 numbers.  Two launches:
//   prepare: T, B and three factors per token, one workgroup per (chunk, head), 25 KiB of workspace;
//   walk:    chunks one behind the other, one workgroup per (sequence, head, columns); rows of k and q come from the inputs, transposed out of
//            LDS where the state takes them in; the next chunk lands while this one is multiplied.
#include "delta_chunk.h"

namespace {

// workspace of a (chunk, head) in fragments of 1 KiB: T [kTriangle][high, rest] | B [kTriangle][high, rest] | factors
constexpr int kB = 2 * kTriangle, kFactors = 4 * kTriangle, kScalarTotal = kFactors + 1;

// where 8 channels of a row lie in a fragment of 16 rows x 32 channels: four adjacent lanes of the transfer hold one row's 64 bytes, in an
// order that spreads the rows over the banks
__device__ __forceinline__ int row_chunk(int lane) { return (lane & 3) ^ ((lane >> 4) & 3); }
__device__ __forceinline__ int row_place(int row, int chunk) { return row * 4 + (chunk ^ ((row >> 2) & 3)); }

template <int NK>
__global__ void __launch_bounds__(256, NK < 5 ? 4 : 3) delta_scalar_prepare_kernel(DeltaPrep q) {
  typedef uint16_t T;
  constexpr int N = NK * 32, KS = N + 8;   // LDS row stride
  const MvDeltaArgs &p = q.a;
  constexpr int QB = L * KS * 2 > L * TS * 4 ? L * KS * 2 : L * TS * 4;
  __shared__ __attribute__((aligned(16))) char smem[L * KS * 2 + QB + 4 * L * 4];
  T *ks = (T *)smem, *qs = ks + L * KS;   // [L][KS]; later (from qs on) -A, then T
  float *ts = (float *)qs, *fk = (float *)(smem + L * KS * 2 + QB), *fq = fk + L, *bt = fq + L, *rs = bt + L;
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), r16 = lane & 15, g = lane >> 4;
  const int head = blockIdx.y, seq = chunk_sequence(p, blockIdx.x);
  const int q0 = p.cu_q[seq], len = p.cu_q[seq + 1] - q0, t0 = ((int)blockIdx.x - q0 / L - seq) * L;
  if (t0 >= len) return;
  const int nt = min(L, len - t0), grp = head / (p.heads / p.groups);
  char *ws = q.ws + ((int64_t)blockIdx.x * p.heads + head) * kScalarTotal * 1024;
  const T *x = (const T *)p.x + (int64_t)(q0 + t0) * p.x_stride;

  // ---- k, q (tokens behind the end: zeros) and their lengths: four threads a token
  {
    const int t = tid >> 2, part = tid & 3;
    const T *row = x + (int64_t)min(t, nt - 1) * p.x_stride + grp * N;
    float sk = 0.f, sq = 0.f;
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      const int c = part * 8 + 32 * s;
      u32x4 a = *(const u32x4 *)(row + p.k_off + c), b = *(const u32x4 *)(row + p.q_off + c);
      if (t >= nt) a = b = u32x4{0u, 0u, 0u, 0u};
      float fa[8], fb[8];
      unpack8<B16>(a, fa);
      unpack8<B16>(b, fb);
#pragma unroll
      for (int j = 0; j < 8; ++j) sk = fmaf(fa[j], fa[j], sk), sq = fmaf(fb[j], fb[j], sq);
      *(u32x4 *)(ks + t * KS + c) = a;
      *(u32x4 *)(qs + t * KS + c) = b;
    }
    sk += __shfl_xor(sk, 1, 64), sq += __shfl_xor(sq, 1, 64);
    sk += __shfl_xor(sk, 2, 64), sq += __shfl_xor(sq, 2, 64);
    if (part == 0) {
      fk[t] = 1.f / sqrtf(sk + p.unit_eps), fq[t] = p.q_scale / sqrtf(sq + p.unit_eps);
      bt[t] = t < nt ? sigmoid_f32(elem<B16>::ld(((const elem<B16>::T *)p.beta)[(int64_t)(q0 + t0 + t) * p.beta_stride + head])) : 0.f;
    }
  }
  if (wave == 0) {   // log2 decays, summed over the tokens
    typedef elem<B16>::T E;
    const float rate = -expf(elem<B16>::ld(((const E *)p.a_log)[head])) * 1.4426950408889634f;
    const float z = elem<B16>::ld(((const E *)p.a)[(int64_t)(q0 + t0 + min(lane, nt - 1)) * p.a_stride + head]) + elem<B16>::ld(((const E *)p.dt_bias)[head]);
    float sum = lane < nt ? rate * softplus_fast(z) : 0.f;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const float left = __shfl_up(sum, o, 64);
      if (lane >= o) sum += left;
    }
    rs[lane] = sum;
  }
  __syncthreads();
  if (tid < L) {
    float *f = (float *)(ws + kFactors * 1024);
    const float last = rs[L - 1];
    const bool is = tid < nt;
    f[tid] = is ? fk[tid] * __builtin_amdgcn_exp2f(rs[tid]) : 0.f;
    f[L + tid] = is ? fq[tid] * __builtin_amdgcn_exp2f(rs[tid]) : 0.f;
    f[2 * L + tid] = is ? fk[tid] * __builtin_amdgcn_exp2f(last - rs[tid]) : 0.f;
    f[3 * L + tid] = __builtin_amdgcn_exp2f(last);
  }

  // ---- A and B by blocks of 16 x 16 tokens; a lane gets row r16, columns 4 g ..
  f32x4 blk[3];
#pragma unroll
  for (int m = 0; m < 3; ++m) {
    const int idx = wave + 4 * m;
    if (idx >= 10) continue;
    int I, J;
    block_place(idx, I, J);
    const T *ki = ks + (16 * I + r16) * KS + 8 * g, *kj = ks + (16 * J + r16) * KS + 8 * g, *qi = qs + (16 * I + r16) * KS + 8 * g;
    f32x4 A = {0.f, 0.f, 0.f, 0.f}, B = A;
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      const u32x4 right = *(const u32x4 *)(kj + 32 * s);
      A = mfma16x16x32<B16>(right, *(const u32x4 *)(ki + 32 * s), A);
      B = mfma16x16x32<B16>(right, *(const u32x4 *)(qi + 32 * s), B);
    }
    const int i = 16 * I + r16, j0 = 16 * J + 4 * g;
    const float ri = rs[i], fi = -bt[i] * fk[i], gi = fq[i];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float f = fk[j0 + e] * __builtin_amdgcn_exp2f(j0 + e <= i ? ri - rs[j0 + e] : 0.f);
      A[e] = j0 + e < i ? A[e] * (fi * f) : 0.f;
      B[e] = j0 + e <= i ? B[e] * (gi * f) : 0.f;
    }
    blk[m] = A;   // (the negative)
    u32x2 hi, lo;
    split4(B, hi, lo);
    u32x2 *dst = (u32x2 *)(ws + (kB + triangle(I, J >> 1) * 2) * 1024 + lane * 16) + (J & 1);
    dst[0] = hi;
    dst[128] = lo;
    if (I == J && (I & 1) == 0) dst[1] = dst[129] = u32x2{0u, 0u};   // the columns behind, in the same step of 32
  }
  __syncthreads();   // q is done with
#pragma unroll
  for (int m = 0; m < 3; ++m) {
    const int idx = wave + 4 * m;
    if (idx >= 10) continue;
    int I, J;
    block_place(idx, I, J);
    *(f32x4 *)(ts + (16 * I + r16) * TS + 16 * J + 4 * g) = blk[m];
  }
  __syncthreads();
  solve_chunk(ts, bt, wave, lane);
  for (int m = wave; m < kTriangle; m += 4) {
    u32x4 hi, lo;
    solution_operand(ts, m, lane, hi, lo);
    u32x4 *dst = (u32x4 *)(ws + m * 2 * 1024) + lane;
    dst[0] = hi, dst[64] = lo;
  }
}

// Workgroup = 4 waves x CW tiles of 16 columns of one head of one sequence; a wave keeps S of its columns in accumulators, whose rows are
// dealt so that tiles 2 s and 2 s + 1 together hold n = 32 s + 8 g .. + 7 in lane group g: operands of the next product as they are.
template <int NK, int CW>
__global__ void __launch_bounds__(256, 1) delta_scalar_walk_kernel(DeltaPrep q) {
  typedef elem<B16>::T T;
  constexpr int N = NK * 32, ROWS = 4 * NK, STAGE = (2 * ROWS + kScalarTotal) * 1024, PER = (kScalarTotal + 3) / 4;
  const MvDeltaArgs &p = q.a;
  extern __shared__ __attribute__((aligned(16))) char smem[];   // 2 stages of k [4][NK] | q [4][NK] | T | B | factors, fragments of 1 KiB
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r16 = lane & 15, g = lane >> 4;
  const int head = blockIdx.y, seq = blockIdx.z, tiles = p.p / 16, tile0 = blockIdx.x * 4 * CW, grp = head / (p.heads / p.groups);
  const int q0 = p.cu_q[seq], len = p.cu_q[seq + 1] - q0;
  if (len <= 0) return;
  const int before = p.cu_k[seq + 1] - p.cu_k[seq] - len, slot = p.state_slots[seq];
  const bool keep = slot >= 0 && slot < p.slots;
  const int64_t size = (int64_t)p.heads * p.n * p.p;
  const int64_t stride = (int64_t)p.heads * kScalarTotal * 1024;
  const char *ws = q.ws + ((int64_t)(q0 / L + seq) * p.heads + head) * kScalarTotal * 1024 + lane * 16;
  const T *x = (const T *)p.x + (int64_t)q0 * p.x_stride;

  int col[CW];
  bool live[CW];
#pragma unroll
  for (int w = 0; w < CW; ++w) {
    const int t = tile0 + wave * CW + w;
    live[w] = t < tiles, col[w] = min(t, tiles - 1) * 16 + r16;
  }
  auto state_at = [&](int half, int w, int i, int e) {
    const int n = (i >> 1) * 32 + g * 8 + (i & 1) * 4 + e;
    return p.state + half * p.slots * size + (int64_t)(keep ? slot : 0) * size + ((int64_t)head * p.n + n) * p.p + col[w];
  };
  f32x4 st[CW][2 * NK];
#pragma unroll
  for (int w = 0; w < CW; ++w)
#pragma unroll
    for (int i = 0; i < 2 * NK; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) st[w][i][e] = keep && before > 0 ? *state_at(before & 1, w, i, e) : 0.f;

  auto transfer = [&](const void *from, char *to) {
    __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void *)from, (__attribute__((address_space(3))) void *)to, 16, 0, 0);
  };
  // a wave brings the rows of one token tile and its share of the rest (rows behind the end: the last row again, with factors 0)
  auto fetch = [&](int c) {
    char *to = smem + (c & 1) * STAGE;
    const T *row = x + (int64_t)min(c * L + 16 * wave + (lane >> 2), len - 1) * p.x_stride + grp * N + row_chunk(lane) * 8;
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      transfer(row + p.k_off + 32 * s, to + (wave * NK + s) * 1024);
      transfer(row + p.q_off + 32 * s, to + (ROWS + wave * NK + s) * 1024);
    }
    const char *from = ws + c * stride;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      const int f = min(i * 4 + wave, kScalarTotal - 1);
      transfer(from + f * 1024, to + (2 * ROWS + f) * 1024);
    }
  };
  T v[CW][16];
  auto fetch_v = [&](int c) {
#pragma unroll
    for (int w = 0; w < CW; ++w)
#pragma unroll
      for (int i = 0; i < 16; ++i)
        v[w][i] = x[(int64_t)min(c * L + 16 * (i >> 2) + 4 * g + (i & 3), len - 1) * p.x_stride + head * p.p + col[w]];
  };
  f32x4 o[CW][4];
  auto store = [&](int c) {
#pragma unroll
    for (int w = 0; w < CW; ++w)
#pragma unroll
      for (int it = 0; it < 4; ++it)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int t = c * L + 16 * it + 4 * g + e;
          if (live[w] && t < len) ((T *)p.out)[(int64_t)(q0 + t) * p.out_stride + head * p.p + col[w]] = elem<B16>::st(o[w][it][e]);
        }
  };
  const uint32_t lds = lds_address(smem);
  const int chunks = (len + L - 1) / L;
  fetch(0);
  fetch_v(0);
  for (int c = 0; c < chunks; ++c) {
    asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
    lds_barrier();   // this chunk has landed; every wave is done with the one before
    f32x4 rest[CW][4];   // v, then R
#pragma unroll
    for (int w = 0; w < CW; ++w)
#pragma unroll
      for (int i = 0; i < 16; ++i) rest[w][i >> 2][i & 3] = elem<B16>::ld(v[w][i]);
    if (c > 0) store(c - 1);
    if (c + 1 < chunks) {
      fetch(c + 1);
      fetch_v(c + 1);
    }
    const uint32_t at = lds + (c & 1) * STAGE, rows = at + row_place(r16, g) * 16, rest_at = at + 2 * ROWS * 1024;
    const uint32_t fl = rest_at + lane * 16, ff = rest_at + kFactors * 1024 + g * 16;
    const uint32_t tr = at + row_place(4 * g + (r16 >> 2), r16 & 3) * 16;
    // ---- k S and q S
    f32x4 ksum[CW][4];
#pragma unroll
    for (int w = 0; w < CW; ++w)
#pragma unroll
      for (int it = 0; it < 4; ++it) ksum[w][it] = o[w][it] = f32x4{0.f, 0.f, 0.f, 0.f};
    static_for<NK>([&](auto S) {
      constexpr int s = decltype(S)::value;
      u32x4 fk[4], fq[4], sh[CW], sl[CW];
      static_for<4>([&](auto I) {
        constexpr int it = decltype(I)::value;
        lds_read128<(it * NK + s) * 1024>(fk[it], rows);
        lds_read128<(ROWS + it * NK + s) * 1024>(fq[it], rows);
      });
#pragma unroll
      for (int w = 0; w < CW; ++w) split44(st[w][2 * s], st[w][2 * s + 1], sh[w], sl[w]);
      static_for<4>([&](auto I) {
        constexpr int it = decltype(I)::value;
        lds_wait<2 * (3 - it)>(fk[it], fq[it]);
      });
#pragma unroll
      for (int part = 0; part < 2; ++part)
#pragma unroll
        for (int it = 0; it < 4; ++it)
#pragma unroll
          for (int w = 0; w < CW; ++w) {
            ksum[w][it] = mfma16x16x32<B16>(fk[it], part ? sl[w] : sh[w], ksum[w][it]);
            o[w][it] = mfma16x16x32<B16>(fq[it], part ? sl[w] : sh[w], o[w][it]);
          }
    });
    // ---- R, U = T R
    u32x4 raw[3][4];
    static_for<4>([&](auto I) {
      constexpr int it = decltype(I)::value;
      lds_read128<it * 64>(raw[0][it], ff);
      lds_read128<it * 64 + 256>(raw[1][it], ff);
      lds_read128<it * 64 + 512>(raw[2][it], ff);
    });
    float last;
    lds_read32<kFactors * 1024 + 768>(last, rest_at);
    u32x4 ft[kTriangle][2];
    static_for<kTriangle>([&](auto M) {
      constexpr int m = decltype(M)::value;
      lds_read128<m * 2048>(ft[m][0], fl);
      lds_read128<m * 2048 + 1024>(ft[m][1], fl);
    });
    static_for<4>([&](auto I) {
      constexpr int it = decltype(I)::value;
      lds_wait<2 * kTriangle>(raw[0][it], raw[1][it]);
      lds_wait<2 * kTriangle>(raw[2][it]);
    });
    lds_wait<2 * kTriangle>(last);
    u32x4 uh[CW][2], ul[CW][2];
#pragma unroll
    for (int w = 0; w < CW; ++w) {
#pragma unroll
      for (int it = 0; it < 4; ++it) {
        rest[w][it] -= __builtin_bit_cast(f32x4, raw[0][it]) * ksum[w][it];
        o[w][it] *= __builtin_bit_cast(f32x4, raw[1][it]);
      }
#pragma unroll
      for (int s = 0; s < 2; ++s) split44(rest[w][2 * s], rest[w][2 * s + 1], uh[w][s], ul[w][s]);
    }
    f32x4 u[CW][4];
#pragma unroll
    for (int w = 0; w < CW; ++w)
#pragma unroll
      for (int it = 0; it < 4; ++it) u[w][it] = f32x4{0.f, 0.f, 0.f, 0.f};
    static_for<kTriangle>([&](auto M) { lds_wait<0>(ft[decltype(M)::value][0], ft[decltype(M)::value][1]); });
#pragma unroll
    for (int part = 0; part < 3; ++part)
      static_for<4>([&](auto I) {
        constexpr int it = decltype(I)::value;
        static_for<it / 2 + 1>([&](auto S) {
          constexpr int s = decltype(S)::value;
#pragma unroll
          for (int w = 0; w < CW; ++w) u[w][it] = mfma16x16x32<B16>(ft[triangle(it, s)][part == 2], part == 1 ? ul[w][s] : uh[w][s], u[w][it]);
        });
      });
    // ---- o += B U
    static_for<kTriangle>([&](auto M) {
      constexpr int m = decltype(M)::value;
      lds_read128<kB * 1024 + m * 2048>(ft[m][0], fl);
      lds_read128<kB * 1024 + m * 2048 + 1024>(ft[m][1], fl);
    });
#pragma unroll
    for (int w = 0; w < CW; ++w)
#pragma unroll
      for (int s = 0; s < 2; ++s) split44(u[w][2 * s], u[w][2 * s + 1], uh[w][s], ul[w][s]);
    static_for<kTriangle>([&](auto M) { lds_wait<0>(ft[decltype(M)::value][0], ft[decltype(M)::value][1]); });
#pragma unroll
    for (int part = 0; part < 3; ++part)
      static_for<4>([&](auto I) {
        constexpr int it = decltype(I)::value;
        static_for<it / 2 + 1>([&](auto S) {
          constexpr int s = decltype(S)::value;
#pragma unroll
          for (int w = 0; w < CW; ++w) o[w][it] = mfma16x16x32<B16>(ft[triangle(it, s)][part == 2], part == 1 ? ul[w][s] : uh[w][s], o[w][it]);
        });
      });
    // ---- S <- decay S + k^T (e^{r_last - r} f u); k transposed: row r16 of a state tile, tokens 16 (e >> 2) + 4 g + (e & 3) of a step of 32
#pragma unroll
    for (int w = 0; w < CW; ++w) {
#pragma unroll
      for (int it = 0; it < 4; ++it) u[w][it] *= __builtin_bit_cast(f32x4, raw[2][it]);
#pragma unroll
      for (int s = 0; s < 2; ++s) split44(u[w][2 * s], u[w][2 * s + 1], uh[w][s], ul[w][s]);
#pragma unroll
      for (int i = 0; i < 2 * NK; ++i) st[w][i] *= last;
    }
    static_for<NK>([&](auto P) {
      constexpr int pair = decltype(P)::value;
      u32x2 kt[2][2][2];   // [state tile][step of 32 tokens][its half]
      static_for<2>([&](auto D) {
        constexpr int d = decltype(D)::value;
        static_for<4>([&](auto I) {
          constexpr int it = decltype(I)::value;
          lds_read64_tr<(it * NK + pair) * 1024 + d * 8>(kt[d][it >> 1][it & 1], tr);
        });
      });
      static_for<2>([&](auto D) {
        constexpr int d = decltype(D)::value;
        lds_wait<0>(kt[d][0][0], kt[d][0][1]);
        lds_wait<0>(kt[d][1][0], kt[d][1][1]);
      });
#pragma unroll
      for (int s = 0; s < 2; ++s)
#pragma unroll
        for (int d = 0; d < 2; ++d) {
          const u32x4 k = {kt[d][s][0][0], kt[d][s][0][1], kt[d][s][1][0], kt[d][s][1][1]};
#pragma unroll
          for (int part = 0; part < 2; ++part)
#pragma unroll
            for (int w = 0; w < CW; ++w) st[w][2 * pair + d] = mfma16x16x32<B16>(k, part ? ul[w][s] : uh[w][s], st[w][2 * pair + d]);
        }
    });
  }
  store(chunks - 1);
  if (keep) {
#pragma unroll
    for (int w = 0; w < CW; ++w)
      if (live[w]) {
#pragma unroll
        for (int i = 0; i < 2 * NK; ++i)
#pragma unroll
          for (int e = 0; e < 4; ++e) *state_at((before + len) & 1, w, i, e) = st[w][i][e];
      }
  }
}

template <int NK>
int launch(const DeltaPrep &q, hipStream_t stream) {
  const MvDeltaArgs &a = q.a;
  hipLaunchKernelGGL((delta_scalar_prepare_kernel<NK>), dim3((unsigned)chunk_slots(a.n_seqs, a.total_q), a.heads), dim3(256), 0, stream, q);
  MV_LAUNCH_CHECK();
  // two column tiles a wave share every operand read, where that still leaves a workgroup per CU
  const int tiles = a.p / 16, wide = (tiles + 7) / 8, lds = 2 * (8 * NK + kScalarTotal) * 1024;
  if (tiles > 4 && (int64_t)wide * a.heads * a.n_seqs >= 256) {
    if (int rc = mv_allow_lds<delta_scalar_walk_kernel<NK, 2>>()) return rc;
    hipLaunchKernelGGL((delta_scalar_walk_kernel<NK, 2>), dim3(wide, a.heads, a.n_seqs), dim3(256), lds, stream, q);
  } else {
    if (int rc = mv_allow_lds<delta_scalar_walk_kernel<NK, 1>>()) return rc;
    hipLaunchKernelGGL((delta_scalar_walk_kernel<NK, 1>), dim3((tiles + 3) / 4, a.heads, a.n_seqs), dim3(256), lds, stream, q);
  }
  MV_LAUNCH_CHECK();
  return MV_OK;
}

}  // namespace

// (arguments checked by mv_delta_chunk_launch, whose workspace is larger)
int mv_delta_scalar_launch(const MvDeltaArgs &a, hipStream_t stream) {
  const DeltaPrep q{a, (char *)a.workspace};
  switch (a.n / 32) {
    case 1: return launch<1>(q, stream);
    case 2: return launch<2>(q, stream);
    case 3: return launch<3>(q, stream);
    case 4: return launch<4>(q, stream);
    case 5: return launch<5>(q, stream);
  }
  return MV_E_SHAPE;
}
