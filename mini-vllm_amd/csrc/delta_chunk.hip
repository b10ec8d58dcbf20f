// K16 — gated delta rule of prompts in chunks of 64 tokens on the matrix cores (16-bit operands, fp32 state).
//
// With r_i the running sum of the log decays in a chunk (per key channel), k and q scaled to their lengths, S the state ahead of the
// chunk and all vectors rows, the recurrence unrolls to
//     u_i = beta_i (v_i - (e^{r_i} k_i) S - sum_{j < i} A_ij u_j),    A_ij = sum_c k_ic k_jc e^{r_ic - r_jc}
//     o_i = (e^{r_i} q_i) S + sum_{j <= i} B_ij u_j,                  B_ij = sum_c q_ic k_jc e^{r_ic - r_jc}
//     S  <- e^{r_last} S + sum_j (e^{r_last - r_j} k_j)^T u_j
// The u of a chunk solve a unit lower triangular system: with T = (1 + A)^-1 diag(beta), U = U0 - W S, U0 = T v, W = T e^r k.
// Two launches:
//   prepare: everything that does not need S, one workgroup per (chunk, head): A, B, T, U0, W, the scaled operands;
//   walk:    chunks one behind the other, one workgroup per (sequence, head, columns): four products with S and U.
// What is fp32 by nature enters a product as the sum of two bf16 numbers (three MFMAs: high x high, high x rest, rest x high), about
// 16 bits of mantissa.  The operands lie in the workspace as MFMA fragments (64 lanes x 16 bytes), which the walk fetches by LDS-DMA.
//
// One decay per head needs less (delta_scalar.hip, bf16).
//
// Exponentials never overflow: A and B are computed by blocks of 16 x 16 tokens with the sums taken relative to r at the end of the
// block in front of the rows' (both factors at most 1), or in the middle of a diagonal block; where a block decays by more than
// 2^kRange a diagonal block is summed pair by pair instead.
#include "delta_chunk.h"

namespace {

constexpr float kRange = 60.f;     // log2
constexpr int kPrepareWaves = 8;

// sizes of a (chunk, head) in the workspace, in fragments of 1 KiB: [W | Q: 4 token tiles][NK][high, rest] | U0: 4 per 16 columns |
// K: [2 NK state tiles][2][high, rest] | B: [4 token tiles][2][high, rest] | decay of the whole chunk
struct Layout {
  int u0, k, b, tail, total;
  __host__ __device__ constexpr Layout(int nk, int p) : u0(16 * nk), k(16 * nk + p / 4), b(24 * nk + p / 4), tail(24 * nk + p / 4 + 16), total(24 * nk + p / 4 + 17) {}
};

template <typename Tag, int NK>
__global__ void __launch_bounds__(kPrepareWaves * 64, 4) delta_prepare_kernel(DeltaPrep q) {
  typedef typename elem<Tag>::T T;
  constexpr int N = NK * 32, W = kPrepareWaves, RS = N + 4, KS = N + 8;   // LDS row strides: fp32, 16-bit
  const MvDeltaArgs &p = q.a;
  extern __shared__ __attribute__((aligned(16))) char smem[];
  float *rs = (float *)smem;                              // [L][RS] running log2 decays
  T *ks = (T *)(smem + L * RS * 4), *qs = ks + L * KS;    // [L][KS]; later (from qs on) -A, then T
  float *ts = (float *)qs;                                // [L][TS]
  constexpr int QB = L * KS * 2 > L * TS * 4 ? L * KS * 2 : L * TS * 4;
  float *fk = (float *)((char *)qs + QB), *fq = fk + L, *bt = fq + L, *part_sums = bt + L;   // [W][64]
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), r16 = lane & 15, g = lane >> 4;
  const int head = blockIdx.y;
  const int seq = chunk_sequence(p, blockIdx.x);
  const int q0 = p.cu_q[seq], len = p.cu_q[seq + 1] - q0, t0 = ((int)blockIdx.x - q0 / L - seq) * L;
  if (t0 >= len) return;
  const int nt = min(L, len - t0), grp = head / (p.heads / p.groups);
  const Layout lay(NK, p.p);
  char *ws = q.ws + ((int64_t)blockIdx.x * p.heads + head) * lay.total * 1024;
  const T *x = (const T *)p.x + (int64_t)(q0 + t0) * p.x_stride;

  // ---- k, q (tokens behind the end: zeros) and their lengths: eight threads a token
  {
    const int t = tid >> 3, part = tid & 7;
    const T *row = x + (int64_t)min(t, nt - 1) * p.x_stride;
    float sk = 0.f, sq = 0.f;
    for (int c = part * 8; c < N; c += 64) {
      u32x4 a = *(const u32x4 *)(row + p.k_off + grp * N + c), b = *(const u32x4 *)(row + p.q_off + grp * N + c);
      if (t >= nt) a = b = u32x4{0u, 0u, 0u, 0u};
      float fa[8], fb[8];
      unpack8<Tag>(a, fa);
      unpack8<Tag>(b, fb);
#pragma unroll
      for (int j = 0; j < 8; ++j) sk = fmaf(fa[j], fa[j], sk), sq = fmaf(fb[j], fb[j], sq);
      *(u32x4 *)(ks + t * KS + c) = a;
      *(u32x4 *)(qs + t * KS + c) = b;
    }
#pragma unroll
    for (int o = 1; o <= 4; o <<= 1) sk += __shfl_xor(sk, o, 64), sq += __shfl_xor(sq, o, 64);
    if (part == 0) {
      fk[t] = 1.f / sqrtf(sk + p.unit_eps), fq[t] = p.q_scale / sqrtf(sq + p.unit_eps);
      bt[t] = t < nt ? sigmoid_f32(elem<Tag>::ld(((const T *)p.beta)[(int64_t)(q0 + t0 + t) * p.beta_stride + head])) : 0.f;
    }
  }
  // ---- log2 decays, summed over the tokens
  {
    const float rate = -expf(elem<Tag>::ld(((const T *)p.a_log)[head])) * 1.4426950408889634f;
    const T *a = (const T *)p.a + (int64_t)(q0 + t0) * p.a_stride, *bias = (const T *)p.dt_bias;
    if (p.channel_decay) {
      for (int i = tid; i < L * N / 8; i += W * 64) {
        const int t = i / (N / 8), c = (i - t * (N / 8)) * 8;
        float f[8], b[8];
        unpack8<Tag>(*(const u32x4 *)(a + (int64_t)min(t, nt - 1) * p.a_stride + head * N + c), f);
        unpack8<Tag>(*(const u32x4 *)(bias + head * N + c), b);
#pragma unroll
        for (int j = 0; j < 8; ++j) f[j] = t < nt ? rate * softplus_fast(f[j] + b[j]) : 0.f;
        f32x4 *dst = (f32x4 *)(rs + t * RS + c);
        dst[0] = f32x4{f[0], f[1], f[2], f[3]}, dst[1] = f32x4{f[4], f[5], f[6], f[7]};
      }
    } else {
      const float b = elem<Tag>::ld(bias[head]);
      const int t = tid >> 3;
      const float v = t < nt ? rate * softplus_fast(elem<Tag>::ld(a[(int64_t)t * p.a_stride + head]) + b) : 0.f;
      for (int c = tid & 7; c < N; c += 8) rs[t * RS + c] = v;
    }
    __syncthreads();
    // a thread TW of a channel's tokens (the threads of a wave: adjacent channels); then the sums ahead are added
    constexpr int TW = L / W;
    for (int c0 = 0; c0 < N; c0 += 64) {
      const int c = c0 + lane;
      float v[TW], sum = 0.f;
      if (c < N) {
#pragma unroll
        for (int t = 0; t < TW; ++t) v[t] = rs[(TW * wave + t) * RS + c];
#pragma unroll
        for (int t = 0; t < TW; ++t) sum += v[t], v[t] = sum;
        part_sums[wave * 64 + lane] = sum;
      }
      __syncthreads();
      if (c < N) {
        float ahead = 0.f;
#pragma unroll
        for (int w = 0; w < W - 1; ++w) ahead += w < wave ? part_sums[w * 64 + lane] : 0.f;
#pragma unroll
        for (int t = 0; t < TW; ++t) rs[(TW * wave + t) * RS + c] = ahead + v[t];
      }
      if (c0 + 64 < N) __syncthreads();
    }
  }
  __syncthreads();

  // ---- A and B by blocks of 16 x 16 tokens (rows I, columns J <= I), ten of them over the waves; a lane gets row r16, columns 4 g ..
  constexpr int BW = (10 + W - 1) / W;
  f32x4 blk[BW];
#pragma unroll
  for (int m = 0; m < BW; ++m) {
    const int idx = wave + W * m;
    if (idx >= 10) continue;
    int I, J;
    block_place(idx, I, J);
    const int ref = I == J ? 16 * I + 7 : 16 * I - 1;
    const float *ri = rs + (16 * I + r16) * RS + 8 * g, *rj = rs + (16 * J + r16) * RS + 8 * g, *rr = rs + ref * RS + 8 * g;
    const T *ki = ks + (16 * I + r16) * KS + 8 * g, *kj = ks + (16 * J + r16) * KS + 8 * g, *qi = qs + (16 * I + r16) * KS + 8 * g;
    f32x4 A = {0.f, 0.f, 0.f, 0.f}, B = A;
    bool fits = true;   // (the sums fall, so the ends of a diagonal block decide)
    if (I == J)
      for (int c = lane; c < N; c += 64)
        fits = fits && rs[16 * I * RS + c] - rs[ref * RS + c] <= kRange && rs[ref * RS + c] - rs[(16 * I + 15) * RS + c] <= kRange;
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      float fi[8], fj[8], fp[8];
      unpack8<Tag>(*(const u32x4 *)(ki + 32 * s), fi);
      unpack8<Tag>(*(const u32x4 *)(kj + 32 * s), fj);
      unpack8<Tag>(*(const u32x4 *)(qi + 32 * s), fp);
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        const f32x4 a = *(const f32x4 *)(ri + 32 * s + 4 * h), b = *(const f32x4 *)(rj + 32 * s + 4 * h), c = *(const f32x4 *)(rr + 32 * s + 4 * h);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float el = __builtin_amdgcn_exp2f(a[e] - c[e]);
          fi[4 * h + e] *= el, fp[4 * h + e] *= el;
          fj[4 * h + e] *= __builtin_amdgcn_exp2f(c[e] - b[e]);
        }
      }
      u32x4 ih, il, jh, jl, ph, pl;
      split8(fi, ih, il);
      split8(fj, jh, jl);
      split8(fp, ph, pl);
      A = mfma3(jh, jl, ih, il, A);
      B = mfma3(jh, jl, ph, pl, B);
    }
    const int i = 16 * I + r16, j0 = 16 * J + 4 * g;
    if (I == J && !__all(fits)) {
      for (int e = 0; e < 4; ++e) {
        float a = 0.f, b = 0.f;
        if (j0 + e <= i)
          for (int c = 0; c < N; ++c) {
            const float k = elem<Tag>::ld(ks[(j0 + e) * KS + c]) * __builtin_amdgcn_exp2f(rs[i * RS + c] - rs[(j0 + e) * RS + c]);
            a = fmaf(elem<Tag>::ld(ks[i * KS + c]), k, a);
            b = fmaf(elem<Tag>::ld(qs[i * KS + c]), k, b);
          }
        A[e] = a, B[e] = b;
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      A[e] = j0 + e < i ? -A[e] * (bt[i] * fk[i] * fk[j0 + e]) : 0.f;
      B[e] = j0 + e <= i ? B[e] * (fq[i] * fk[j0 + e]) : 0.f;
    }
    blk[m] = A;   // (the negative)
    // B as an operand whose k order is that of an accumulator pair: key 16 (e >> 2) + 4 g + (e & 3) of a step of 32
    u32x2 hi, lo;
    split4(B, hi, lo);
    u32x2 *dst = (u32x2 *)(ws + (lay.b + (I * 2 + (J >> 1)) * 2) * 1024 + lane * 16) + (J & 1);
    dst[0] = hi;
    dst[128] = lo;
    if (I == J && (I & 1) == 0) dst[1] = dst[129] = u32x2{0u, 0u};   // the columns behind, in the same step of 32
  }

  // ---- the operands that meet S and U: e^r q by rows; e^(r_last - r) k by state rows, in the order of the walk's accumulators
  for (int f = wave; f < 4 * NK; f += W) {
    const int it = f / NK, s = f - it * NK, t = 16 * it + r16, c = 32 * s + 8 * g;
    float v[8];
    u32x4 hi, lo;
    unpack8<Tag>(*(const u32x4 *)(qs + t * KS + c), v);
    const float w = fq[t];
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] *= w * __builtin_amdgcn_exp2f(rs[t * RS + c + e]);
    split8(v, hi, lo);
    u32x4 *dst = (u32x4 *)(ws + (8 * NK + f * 2) * 1024) + lane;
    dst[0] = hi, dst[64] = lo;
  }
  for (int c = tid; c < N; c += W * 64) ((float *)(ws + lay.tail * 1024))[c] = __builtin_amdgcn_exp2f(rs[(L - 1) * RS + c]);
  __syncthreads();   // q is done with
#pragma unroll
  for (int m = 0; m < BW; ++m) {
    const int idx = wave + W * m;
    if (idx >= 10) continue;
    int I, J;
    block_place(idx, I, J);
    *(f32x4 *)(ts + (16 * I + r16) * TS + 16 * J + 4 * g) = blk[m];
  }
  __syncthreads();

  solve_chunk(ts, bt, wave, lane);

  // ---- by 32 channels: K = e^(r_last - r) k by state rows, in the order of the walk's accumulators, and -W = -T e^r k by tokens;
  // by 16 columns of v: U0 = T v
  for (int item = wave; item < NK + p.p / 16; item += W) {
    if (item < NK) {
      f32x4 acc[2][4];
#pragma unroll
      for (int it = 0; it < 4; ++it) acc[0][it] = acc[1][it] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        u32x4 th[4], tl[4];
#pragma unroll
        for (int it = 2 * s; it < 4; ++it) solution_operand(ts, triangle(it, s), lane, th[it], tl[it]);
#pragma unroll
        for (int d = 0; d < 2; ++d) {
          const int i = 2 * item + d, c = item * 32 + (r16 >> 2) * 8 + d * 4 + (r16 & 3);
          const float last = rs[(L - 1) * RS + c];
          float v[8], w[8];
          u32x4 hi, lo;
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            const int t = 32 * s + 16 * (e >> 2) + 4 * g + (e & 3);
            const float k = elem<Tag>::ld(ks[t * KS + c]) * fk[t], r = rs[t * RS + c];
            v[e] = k * __builtin_amdgcn_exp2f(last - r);
            w[e] = k * __builtin_amdgcn_exp2f(r);
          }
          split8(v, hi, lo);
          u32x4 *dst = (u32x4 *)(ws + (lay.k + (i * 2 + s) * 2) * 1024) + lane;
          dst[0] = hi, dst[64] = lo;
          split8(w, hi, lo);
#pragma unroll
          for (int it = 2 * s; it < 4; ++it) acc[d][it] = mfma3(hi, lo, th[it], tl[it], acc[d][it]);
        }
      }
#pragma unroll
      for (int it = 0; it < 4; ++it) {
        u32x4 hi, lo;
        split44(-acc[0][it], -acc[1][it], hi, lo);
        u32x4 *dst = (u32x4 *)(ws + (it * NK + item) * 2 * 1024) + lane;
        dst[0] = hi, dst[64] = lo;
      }
    } else {
      const int ct = item - NK;
      const T *v = x + head * p.p + ct * 16 + r16;
      T raw[16];
#pragma unroll
      for (int e = 0; e < 16; ++e) raw[e] = v[(int64_t)min(16 * (e >> 2) + 4 * g + (e & 3), nt - 1) * p.x_stride];
      f32x4 acc[4];
#pragma unroll
      for (int it = 0; it < 4; ++it) acc[it] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        float f[8];
        u32x4 hi, lo;
#pragma unroll
        for (int e = 0; e < 8; ++e) f[e] = elem<Tag>::ld(raw[8 * s + e]);
        split8(f, hi, lo);
#pragma unroll
        for (int it = 2 * s; it < 4; ++it) {
          u32x4 th, tl;
          solution_operand(ts, triangle(it, s), lane, th, tl);
          acc[it] = mfma16x16x32<B16>(th, hi, acc[it]);
          acc[it] = mfma16x16x32<B16>(tl, hi, acc[it]);
          if constexpr (!__is_same(Tag, B16)) acc[it] = mfma16x16x32<B16>(th, lo, acc[it]);
        }
      }
      // in the layout of an accumulator: column lane & 15, tokens 4 (lane >> 4) ..
#pragma unroll
      for (int it = 0; it < 4; ++it) *((f32x4 *)(ws + (lay.u0 + ct * 4 + it) * 1024) + lane) = acc[it];
    }
  }
}

// Workgroup = 4 waves x CW tiles of 16 columns of one head of one sequence; a wave keeps S of its columns in accumulators.  The
// accumulators are the next product's operands as they are: the rows of S are dealt so that tiles 2 s and 2 s + 1 together hold
// n = 32 s + 8 g .. + 7 in lane group g.  LDS holds the operands of one phase while those of the other phase land.
template <typename Tag, int NK, int CW>
__global__ void __launch_bounds__(256, 1) delta_walk_kernel(DeltaPrep q) {
  typedef typename elem<Tag>::T T;
  constexpr int F1 = 16 * NK + 16 * CW, F2 = 8 * NK + 17, N1 = F1 / 4, N2 = (F2 + 3) / 4;   // fragments of a phase; a wave's
  const MvDeltaArgs &p = q.a;
  extern __shared__ __attribute__((aligned(16))) char smem[];   // [F1][1 KiB] | [F2][1 KiB]
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r16 = lane & 15, g = lane >> 4;
  const int head = blockIdx.y, seq = blockIdx.z, tiles = p.p / 16, tile0 = blockIdx.x * 4 * CW;
  const int q0 = p.cu_q[seq], len = p.cu_q[seq + 1] - q0;
  if (len <= 0) return;
  const int before = p.cu_k[seq + 1] - p.cu_k[seq] - len, slot = p.state_slots[seq];
  const bool keep = slot >= 0 && slot < p.slots;
  const int64_t size = (int64_t)p.heads * p.n * p.p;
  const Layout lay(NK, p.p);
  const int64_t stride = (int64_t)p.heads * lay.total * 1024;
  const char *ws = q.ws + ((int64_t)(q0 / L + seq) * p.heads + head) * lay.total * 1024 + lane * 16;

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

  auto fetch = [&](const char *from, int frag, char *to) {
    __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void *)(from + (int64_t)frag * 1024),
                                     (__attribute__((address_space(3))) void *)to, 16, 0, 0);
  };
  auto fetch1 = [&](const char *from) {
#pragma unroll
    for (int i = 0; i < N1; ++i) {
      const int f = i * 4 + wave, u = f - 16 * NK;   // u: (column tile, token tile)
      fetch(from, f < 16 * NK ? f : lay.u0 + min(tile0 + (u >> 2), tiles - 1) * 4 + (u & 3), smem + f * 1024);
    }
  };
  auto fetch2 = [&](const char *from) {
#pragma unroll
    for (int i = 0; i < N2; ++i) {
      const int f = min(i * 4 + wave, F2 - 1);
      fetch(from, lay.k + f, smem + (F1 + f) * 1024);
    }
  };
  const uint32_t base = lds_address(smem) + lane * 16;
  const uint32_t aw = base, aq = base + 8 * NK * 1024, au = base + (16 * NK + wave * CW * 4) * 1024;
  const uint32_t ak = base + F1 * 1024, ab = ak + 8 * NK * 1024, at = lds_address(smem) + (F1 + 8 * NK + 16) * 1024 + g * 32;
  const int chunks = (len + L - 1) / L;
  fetch1(ws);
  fetch2(ws);
  for (int c = 0; c < chunks; ++c) {
    const bool more = c + 1 < chunks;
    ws += stride;
    asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"n"(N2) : "memory");   // (the newest N2: the other phase's)
    lds_barrier();
    // ---- U = U0 - W S, O = Q S
    f32x4 u[CW][4], o[CW][4];
#pragma unroll
    for (int w = 0; w < CW; ++w)
#pragma unroll
      for (int it = 0; it < 4; ++it) o[w][it] = f32x4{0.f, 0.f, 0.f, 0.f};
    static_for<CW>([&](auto W) {
      constexpr int w = decltype(W)::value;
      u32x4 raw[4];
      static_for<4>([&](auto I) { lds_read128<(w * 4 + decltype(I)::value) * 1024>(raw[decltype(I)::value], au); });
      static_for<4>([&](auto I) {
        lds_wait<0>(raw[decltype(I)::value]);
        u[w][decltype(I)::value] = __builtin_bit_cast(f32x4, raw[decltype(I)::value]);
      });
    });
    static_for<NK>([&](auto S) {
      constexpr int s = decltype(S)::value;
      u32x4 fw[4][2], fo[4][2], sh[CW], sl[CW];
      static_for<4>([&](auto I) {
        constexpr int it = decltype(I)::value;
        lds_read128<((it * NK + s) * 2) * 1024>(fw[it][0], aw);
        lds_read128<((it * NK + s) * 2 + 1) * 1024>(fw[it][1], aw);
        lds_read128<((it * NK + s) * 2) * 1024>(fo[it][0], aq);
        lds_read128<((it * NK + s) * 2 + 1) * 1024>(fo[it][1], aq);
      });
#pragma unroll
      for (int w = 0; w < CW; ++w) split44(st[w][2 * s], st[w][2 * s + 1], sh[w], sl[w]);
      static_for<4>([&](auto I) {
        constexpr int it = decltype(I)::value, left = 4 * (3 - it);
        lds_wait<left>(fw[it][0], fw[it][1]);
        lds_wait<left>(fo[it][0], fo[it][1]);
      });
#pragma unroll
      for (int part = 0; part < 3; ++part)
#pragma unroll
        for (int it = 0; it < 4; ++it)
#pragma unroll
          for (int w = 0; w < CW; ++w) {
            u[w][it] = mfma16x16x32<B16>(fw[it][part == 2], part == 1 ? sl[w] : sh[w], u[w][it]);
            o[w][it] = mfma16x16x32<B16>(fo[it][part == 2], part == 1 ? sl[w] : sh[w], o[w][it]);
          }
    });
    lds_barrier();   // every wave has read phase 1
    if (more) {
      fetch1(ws);
      asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N1) : "memory");
    } else {
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    }
    lds_barrier();
    // ---- O += B U, S = decay S + K U
    u32x4 uh[CW][2], ul[CW][2];
#pragma unroll
    for (int w = 0; w < CW; ++w)
#pragma unroll
      for (int s = 0; s < 2; ++s) split44(u[w][2 * s], u[w][2 * s + 1], uh[w][s], ul[w][s]);
    static_for<4>([&](auto I) {
      constexpr int it = decltype(I)::value;
      u32x4 fb[2][2];
      static_for<it / 2 + 1>([&](auto S) {
        constexpr int s = decltype(S)::value;
        lds_read128<((it * 2 + s) * 2) * 1024>(fb[s][0], ab);
        lds_read128<((it * 2 + s) * 2 + 1) * 1024>(fb[s][1], ab);
      });
      static_for<it / 2 + 1>([&](auto S) { lds_wait<0>(fb[decltype(S)::value][0], fb[decltype(S)::value][1]); });
#pragma unroll
      for (int part = 0; part < 3; ++part)
        static_for<it / 2 + 1>([&](auto S) {
          constexpr int s = decltype(S)::value;
#pragma unroll
          for (int w = 0; w < CW; ++w) o[w][it] = mfma16x16x32<B16>(fb[s][part == 2], part == 1 ? ul[w][s] : uh[w][s], o[w][it]);
        });
    });
    static_for<NK>([&](auto P) {   // two state tiles at a time
      constexpr int i0 = 2 * decltype(P)::value;
      u32x4 fk[2][2][2], tail[2];
      static_for<2>([&](auto D) {
        constexpr int d = decltype(D)::value;
        lds_read128<((i0 + d) >> 1) * 128 + ((i0 + d) & 1) * 16>(tail[d], at);
        static_for<2>([&](auto S) {
          constexpr int s = decltype(S)::value;
          lds_read128<(((i0 + d) * 2 + s) * 2) * 1024>(fk[d][s][0], ak);
          lds_read128<(((i0 + d) * 2 + s) * 2 + 1) * 1024>(fk[d][s][1], ak);
        });
      });
      static_for<2>([&](auto D) {
        constexpr int d = decltype(D)::value;
        lds_wait<0>(tail[d]);
        lds_wait<0>(fk[d][0][0], fk[d][0][1]);
        lds_wait<0>(fk[d][1][0], fk[d][1][1]);
#pragma unroll
        for (int w = 0; w < CW; ++w) st[w][i0 + d] *= __builtin_bit_cast(f32x4, tail[d]);
      });
#pragma unroll
      for (int s = 0; s < 2; ++s)
#pragma unroll
        for (int part = 0; part < 3; ++part)
#pragma unroll
          for (int d = 0; d < 2; ++d)
#pragma unroll
            for (int w = 0; w < CW; ++w)
              st[w][i0 + d] = mfma16x16x32<B16>(fk[d][s][part == 2], part == 1 ? ul[w][s] : uh[w][s], st[w][i0 + d]);
    });
#pragma unroll
    for (int w = 0; w < CW; ++w)
#pragma unroll
      for (int it = 0; it < 4; ++it)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int t = c * L + 16 * it + 4 * g + e;
          if (live[w] && t < len) ((T *)p.out)[(int64_t)(q0 + t) * p.out_stride + head * p.p + col[w]] = elem<Tag>::st(o[w][it][e]);
        }
    lds_barrier();   // every wave has read phase 2
    if (more) fetch2(ws);
  }
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

template <typename Tag, int NK>
int launch(const DeltaPrep &q, hipStream_t stream) {
  const MvDeltaArgs &a = q.a;
  constexpr int RS = NK * 32 + 4, KS = NK * 32 + 8;
  constexpr int QB = L * KS * 2 > L * (L + 4) * 4 ? L * KS * 2 : L * (L + 4) * 4;
  if (int rc = mv_allow_lds<delta_prepare_kernel<Tag, NK>>()) return rc;
  hipLaunchKernelGGL((delta_prepare_kernel<Tag, NK>), dim3((unsigned)chunk_slots(a.n_seqs, a.total_q), a.heads),
                     dim3(kPrepareWaves * 64), L * RS * 4 + L * KS * 2 + QB + (3 + kPrepareWaves) * L * 4, stream, q);
  MV_LAUNCH_CHECK();
  // two column tiles a wave share every operand read, where that still leaves a workgroup per CU
  const int tiles = a.p / 16, wide = (tiles + 7) / 8;
  if (tiles > 4 && (int64_t)wide * a.heads * a.n_seqs >= 256 && 24 * NK + 32 + 17 <= 160) {
    if (int rc = mv_allow_lds<delta_walk_kernel<Tag, NK, 2>>()) return rc;
    hipLaunchKernelGGL((delta_walk_kernel<Tag, NK, 2>), dim3(wide, a.heads, a.n_seqs), dim3(256), (24 * NK + 32 + 17) * 1024, stream, q);
  } else {
    if (int rc = mv_allow_lds<delta_walk_kernel<Tag, NK, 1>>()) return rc;
    hipLaunchKernelGGL((delta_walk_kernel<Tag, NK, 1>), dim3((tiles + 3) / 4, a.heads, a.n_seqs), dim3(256), (24 * NK + 16 + 17) * 1024,
                       stream, q);
  }
  MV_LAUNCH_CHECK();
  return MV_OK;
}

}  // namespace

size_t mv_delta_chunk_workspace(int n_seqs, int total_q, int heads, int p, int n) {
  if (n_seqs <= 0 || total_q <= 0 || heads <= 0 || p <= 0 || n <= 0 || n > 160 || (n & 31)) return 0;
  return (size_t)chunk_slots(n_seqs, total_q) * heads * Layout(n / 32, p).total * 1024;
}

int mv_delta_chunk_launch(const MvDeltaArgs &a, int dtype, hipStream_t stream) {
  const size_t need = mv_delta_chunk_workspace(a.n_seqs, a.total_q, a.heads, a.p, a.n);
  if (!need || !a.workspace) return MV_E_SHAPE;   // larger states: token by token
  if ((size_t)a.ws_bytes < need || !mv_aligned16(a.workspace)) return MV_E_WORKSPACE;
  if (!mv_aligned16(a.x) || (a.x_stride & 7) || (a.k_off & 7) || (a.q_off & 7) || a.total_q > 64 * 1000000) return MV_E_ALIGN;
  if (a.channel_decay && (!mv_aligned16(a.a) || (a.a_stride & 7) || !mv_aligned16(a.dt_bias))) return MV_E_ALIGN;
  const DeltaPrep q{a, (char *)a.workspace};
  if (!a.channel_decay && dtype == MV_BF16) return mv_delta_scalar_launch(a, stream);
#define MV_DN(NK_) \
  if (a.n == 32 * NK_) return dtype == MV_BF16 ? launch<bf16_tag, NK_>(q, stream) : launch<f16_tag, NK_>(q, stream)
  MV_DN(1);
  MV_DN(2);
  MV_DN(3);
  MV_DN(4);
  MV_DN(5);
#undef MV_DN
  return MV_E_SHAPE;
}
