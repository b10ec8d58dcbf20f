// K14 — latent attention, prefill on the matrix cores (16-bit): packed varlen causal flash attention whose query / key rows
// [plain | rotated] and value rows differ in width, keys visible through a sliding window.
//
// One workgroup = NW waves of 32 query rows of one (sequence, head); keys in tiles of 64, K | V double-buffered in LDS by LDS-DMA.
//   * A key row comes from two places: its head's expanded plain part and the rotated part that all heads share.  The split falls
//     on a 16-byte chunk, so every DMA lane just holds its own source pointer and stride.
//   * The query's rotated part is rotated in registers when the Q fragments are loaded (pairs lie in one lane).
//   * S^T = K Q^T, online softmax, O^T += V^T P^T on v_mfma_f32_32x32x16, the S^T accumulators reused as P^T operand.
//   * Window: a workgroup starts at the tile of its first row's first key; a wave skips tiles that none of its rows see; tiles
//     on an edge are masked per key.
#include "latent.h"

#include <type_traits>

namespace {

typedef __attribute__((ext_vector_type(16))) float f32x16;
typedef __attribute__((ext_vector_type(4))) short s16x4;
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;
typedef __attribute__((address_space(3))) const u32x4 lds_u32x4;

constexpr int BN = 64;   // keys per tile

template <typename Tag>
__device__ __forceinline__ f32x16 mfma32(const u32x4 &a, const u32x4 &b, const f32x16 &c) {
  if constexpr (__is_same(Tag, bf16_tag))
    return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(mv_bf16x8, a), __builtin_bit_cast(mv_bf16x8, b), c, 0, 0, 0);
  else
    return __builtin_amdgcn_mfma_f32_32x32x16_f16(__builtin_bit_cast(mv_f16x8, a), __builtin_bit_cast(mv_f16x8, b), c, 0, 0, 0);
}
// chunk swizzles (XOR): rows of a multiple of 256 bytes all start in the same bank, other multiples of 128 in two
template <int CH> __device__ __forceinline__ int k_swz(int row) { return CH % 16 == 0 ? (row & 15) : ((row >> 1) & 7); }
template <int CH> __device__ __forceinline__ int v_swz(int row) {
  return CH % 16 == 0 ? (((row & 3) << 2) | ((row >> 2) & 3)) : (((row >> 1) & 1) << 2);
}

template <typename Tag, int DQ, int DV, int NW>
__global__ void __launch_bounds__(NW * 64, 2) latent_prefill_kernel(MvLatentPrefillArgs p) {
  typedef typename elem<Tag>::T T;
  constexpr int NS = DQ / 16, NDT = DV / 32, CQ = DQ / 8, CV = DV / 8;
  constexpr int KB = BN * DQ * 2, VB = BN * DV * 2, BUF = KB + VB, BM = NW * 32;
  constexpr int PK = CQ / NW, PV = CV / NW;   // 1-KiB DMA instructions of a K / V tile per wave
  static_assert(CQ % NW == 0 && CV % NW == 0 && NW * 32 * DV * 2 <= 2 * BUF);
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r = lane & 31, h = lane >> 5;
  // heads fastest (a head's blocks share an XCD's L2 when 8 divides the heads), query blocks slowest, the heaviest first
  const int head = blockIdx.x, seq = blockIdx.y, qb = (int)gridDim.z - 1 - (int)blockIdx.z;
  const int q0 = p.cu_q[seq], sq = p.cu_q[seq + 1] - q0, k0 = p.cu_k[seq], sk = p.cu_k[seq + 1] - k0;
  if (qb * BM >= sq) return;
  const int shift = sk - sq;
  const int qidx = qb * BM + wave * 32 + r;
  const bool q_ok = qidx < sq;

  // ---- Q^T fragments: lane (r, h) holds row r, columns 16 s + 8 h .. + 7, the rotated part turned here
  u32x4 qf[NS];
  {
    const int row = q0 + (q_ok ? qidx : 0), pairs = p.rot_dim >> 1;
    const T *qp = (const T *)p.q + (int64_t)row * p.q_stride + (int64_t)head * DQ + 8 * h;
    const int64_t pos = p.positions[row];
    const bool pos_ok = pos >= 0 && pos < p.max_pos;
    const float *ct = p.cos + (pos_ok ? pos * pairs : 0), *st = p.sin + (pos_ok ? pos * pairs : 0);
    float cs[NS][4], sn[NS][4];   // (every load of the row ahead of its arithmetic; only the rotated steps' are made)
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      qf[s] = *reinterpret_cast<const u32x4 *>(qp + 16 * s);
      if (16 * s >= p.plain_cols)   // (plain_cols is a multiple of 32: uniform over the step)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int i = min(((16 * s + 8 * h - p.plain_cols) >> 1) + j, pairs - 1);
          cs[s][j] = ct[i], sn[s][j] = st[i];
        }
    }
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      if (16 * s >= p.plain_cols) {
        float f[8];
        unpack8<Tag>(qf[s], f);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int i = ((16 * s + 8 * h - p.plain_cols) >> 1) + j;
          const float c = pos_ok ? cs[s][j] : 1.0f, n = pos_ok ? sn[s][j] : 0.0f, a = f[2 * j], b = f[2 * j + 1];
          f[2 * j] = i < pairs ? __fsub_rn(__fmul_rn(a, c), __fmul_rn(b, n)) : 0.f;
          f[2 * j + 1] = i < pairs ? __fadd_rn(__fmul_rn(b, c), __fmul_rn(a, n)) : 0.f;
        }
        qf[s] = pack8<Tag>(f);
      }
      if (!q_ok) qf[s] = u32x4{0u, 0u, 0u, 0u};
    }
    settle(qf);
  }

  f32x16 oacc[NDT];
#pragma unroll
  for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
    for (int i = 0; i < 16; ++i) oacc[dt][i] = 0.f;
  float m_run = -1e30f, l_run = 0.f;
  const float scale_log2 = p.scale * 1.4426950408889634f;

  const int q_last = min(sq, (qb + 1) * BM) - 1, kv_len = min(sk, q_last + shift + 1);
  const int win = p.window > 0 ? p.window : 0x3fffffff;
  const int kv_base = max(0, shift + qb * BM - win + 1) / BN * BN;
  const int n_tiles = (kv_len - kv_base + BN - 1) / BN;
  const int wave_min = shift + qb * BM + wave * 32, wave_max = wave_min + 31;        // positions of the wave's rows
  const int lo_min = wave_min - win + 1, lo_max = wave_max - win + 1;                // first visible keys

  // ---- DMA sources: instruction i of this wave fills chunks (NW i + wave) * 64 .. + 63 of a tile, row by row
  const T *ksrc[PK], *vsrc[PV];
  int krow[PK], vrow[PV], kstep[PK];   // tile row, elements between rows
#pragma unroll
  for (int i = 0; i < PK; ++i) {
    const int ci = (NW * i + wave) * 64 + lane, row = ci / CQ, c = ((ci % CQ) ^ k_swz<CQ>(row)) * 8;
    const bool rot = c >= p.plain_cols;
    const int rc = min(c - p.plain_cols, p.rot_cols - 8);   // (columns behind the rotated part meet zeros of q)
    krow[i] = row;
    kstep[i] = (int)(rot ? p.rot_stride : p.k_stride);
    ksrc[i] = (rot ? (const T *)p.rot + rc : (const T *)p.k + (int64_t)head * p.plain_cols + c) + (int64_t)(k0 + kv_base) * kstep[i];
  }
#pragma unroll
  for (int i = 0; i < PV; ++i) {
    const int ci = (NW * i + wave) * 64 + lane, row = ci / CV, c = ((ci % CV) ^ v_swz<CV>(row)) * 8;
    vrow[i] = row;
    vsrc[i] = (const T *)p.v + (int64_t)head * DV + c + (int64_t)(k0 + kv_base) * p.v_stride;
  }
  const int vstep = (int)p.v_stride;
  auto dma = [&](int t, int buf) {
    const int last = sk - 1 - (kv_base + t * BN);   // rows past the end re-read the last key (probability 0, finite data)
    char *dk = smem + buf * BUF, *dv = dk + KB;
    const int base = t * BN;
#pragma unroll
    for (int i = 0; i < PK; ++i)
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) void *)(ksrc[i] + (int64_t)(base + min(krow[i], last)) * kstep[i]),
          (__attribute__((address_space(3))) void *)(dk + (NW * i + wave) * 1024), 16, 0, 0);
#pragma unroll
    for (int i = 0; i < PV; ++i)
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) void *)(vsrc[i] + (int64_t)(base + min(vrow[i], last)) * vstep),
          (__attribute__((address_space(3))) void *)(dv + (NW * i + wave) * 1024), 16, 0, 0);
  };

  // ---- LDS read addresses (hand-counted reads, latent.h); the buffer is an instruction immediate where it fits in 16 bits
  constexpr bool IMM = BUF + (DQ * 2) * 32 < 65536 && BUF + 48 * (DV * 2) < 65536;
  // PIPE: hand-counted reads ahead of their use.  Not where the registers run out: a fragment that is still on its way must not be
  // moved to scratch
  constexpr bool PIPE = DQ <= 192 && DV <= 128;
  const uint32_t lds0 = lds_address(smem);
  uint32_t koff[NS];
#pragma unroll
  for (int s = 0; s < NS; ++s) koff[s] = lds0 + r * (DQ * 2) + (((2 * s + h) ^ k_swz<CQ>(r)) << 4);
  const int g = (lane >> 4) & 1, q4 = (lane & 15) >> 2, pp = lane & 3;
  uint32_t vlo[NDT], vhi[NDT];
#pragma unroll
  for (int dt = 0; dt < NDT; ++dt) {
    const int ch = 4 * dt + 2 * g + (pp >> 1);
    vlo[dt] = lds0 + KB + (4 * h + q4) * (DV * 2) + ((ch ^ v_swz<CV>(4 * h + q4)) << 4) + 8 * (pp & 1);
    vhi[dt] = lds0 + KB + (4 * h + q4 + 8) * (DV * 2) + ((ch ^ v_swz<CV>(4 * h + q4 + 8)) << 4) + 8 * (pp & 1);
  }

  auto tile = [&](const int t, auto Bc) __attribute__((always_inline)) {
    constexpr int BO = IMM ? decltype(Bc)::value * BUF : 0;
    constexpr uint32_t add = IMM ? 0 : decltype(Bc)::value * BUF;
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");   // (nothing else may be counted below)
    if (t + 1 < n_tiles) dma(t + 1, 1 - decltype(Bc)::value);
    const int kv0 = kv_base + t * BN;
    if (kv0 <= wave_max && kv0 + BN > lo_min) {
      f32x16 sacc[2];
      const f32x16 zero = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
      u32x4 kf[2][2];            // K fragments, one step ahead
      u32x2 va[NDT], vb[NDT];    // V^T fragments of 16 keys; the first ones go out before the softmax
      if constexpr (PIPE) {
        lds_read128<BO>(kf[0][0], koff[0] + add);
        lds_read128<BO + 32 * (DQ * 2)>(kf[0][1], koff[0] + add);
        static_for<NS>([&](auto S) {
          constexpr int s = decltype(S)::value;
          if constexpr (s + 1 < NS) {
            lds_read128<BO>(kf[(s + 1) & 1][0], koff[s + 1] + add);
            lds_read128<BO + 32 * (DQ * 2)>(kf[(s + 1) & 1][1], koff[s + 1] + add);
            lds_wait<2>(kf[s & 1][0], kf[s & 1][1]);
          } else {
            static_for<NDT>([&](auto D) {
              lds_read64_tr<BO>(va[decltype(D)::value], vlo[decltype(D)::value] + add);
              lds_read64_tr<BO>(vb[decltype(D)::value], vhi[decltype(D)::value] + add);
            });
            lds_wait<(2 * NDT < 15 ? 2 * NDT : 15)>(kf[s & 1][0], kf[s & 1][1]);
          }
          sacc[0] = mfma32<Tag>(kf[s & 1][0], qf[s], s ? sacc[0] : zero);
          sacc[1] = mfma32<Tag>(kf[s & 1][1], qf[s], s ? sacc[1] : zero);
        });
      } else {
#pragma unroll
        for (int s = 0; s < NS; ++s) {
          const u32x4 k_lo = *(lds_u32x4 *)(uintptr_t)(koff[s] + BO + add), k_hi = *(lds_u32x4 *)(uintptr_t)(koff[s] + BO + add + 32 * (DQ * 2));
          sacc[0] = mfma32<Tag>(k_lo, qf[s], s ? sacc[0] : zero);
          sacc[1] = mfma32<Tag>(k_hi, qf[s], s ? sacc[1] : zero);
        }
      }
      if (kv0 + BN - 1 > wave_min || kv0 + BN > sk || kv0 < lo_max) {
        const int hi = min(qidx + shift, sk - 1), lo = qidx + shift - win + 1;
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
          for (int i = 0; i < 16; ++i) {
            const int key = kv0 + kt * 32 + (i & 3) + 8 * (i >> 2) + 4 * h;
            sacc[kt][i] = key <= hi && key >= lo ? sacc[kt][i] : -INFINITY;
          }
      }
      float mx = -INFINITY;
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int i = 0; i < 16; ++i) mx = fmaxf(mx, sacc[kt][i]);
      {   // the other half of the row lies 32 lanes away (a vector instruction: an LDS one would wait for the reads in flight)
        float other = mx;
        asm volatile("s_nop 1\n\tv_permlane32_swap_b32 %0, %1" : "+v"(mx), "+v"(other));
        mx = fmaxf(mx, other);
      }
      const float m_new = fmaxf(m_run, mx * scale_log2);
      if (!__all(m_new - m_run <= 6.0f)) {   // rescale only when a maximum grew by more than 2^6
        const float alpha = __builtin_amdgcn_exp2f(m_run - m_new);
        m_run = m_new;
        l_run *= alpha;
#pragma unroll
        for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
          for (int i = 0; i < 16; ++i) oacc[dt][i] *= alpha;
      }
      const float nm = -m_run;
      float rs[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const float e = __builtin_amdgcn_exp2f(__builtin_fmaf(sacc[kt][i], scale_log2, nm));
          sacc[kt][i] = e;
          rs[i & 3] += e;
        }
      l_run += (rs[0] + rs[1]) + (rs[2] + rs[3]);
      u32x4 pf[4];
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j)
          pf[i][j] = pack_pair<Tag>(sacc[i >> 1][8 * (i & 1) + 2 * j], sacc[i >> 1][8 * (i & 1) + 2 * j + 1]);
      // 16 keys at a time; a fragment register is requested again right behind the product that used it
      static_for<4>([&](auto G) {
        constexpr int gr = decltype(G)::value;
        static_for<NDT>([&](auto D) {
          constexpr int dt = decltype(D)::value;
          if constexpr (!PIPE) {
            constexpr uint32_t o = BO + add + gr * 16 * (DV * 2);
            va[dt] = __builtin_bit_cast(u32x2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4 *)(uintptr_t)(vlo[dt] + o)));
            vb[dt] = __builtin_bit_cast(u32x2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4 *)(uintptr_t)(vhi[dt] + o)));
          } else if constexpr (gr < 3) lds_wait<2 * NDT - 2>(va[dt], vb[dt]);
          else lds_wait<2 * (NDT - 1 - dt)>(va[dt], vb[dt]);
          oacc[dt] = mfma32<Tag>(u32x4{va[dt].x, va[dt].y, vb[dt].x, vb[dt].y}, pf[gr], oacc[dt]);
          if constexpr (PIPE && gr < 3) {
            lds_read64_tr<BO + (gr + 1) * 16 * (DV * 2)>(va[dt], vlo[dt] + add);
            lds_read64_tr<BO + (gr + 1) * 16 * (DV * 2)>(vb[dt], vhi[dt] + add);
          }
        });
      });
    }
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");   // this wave's share of the next tile has landed
    __syncthreads();
  };
  if (n_tiles > 0) dma(0, 0);
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  for (int t = 0; t < n_tiles; t += 2) {
    tile(t, std::integral_constant<int, 0>{});
    if (t + 1 < n_tiles) tile(t + 1, std::integral_constant<int, 1>{});
  }

  // ---- O^T through the wave's own part of LDS, out as whole rows
  const float l_tot = l_run + __shfl_xor(l_run, 32, 64), inv = l_tot > 0.f ? 1.0f / l_tot : 0.f;
  constexpr int MASK = CV % 16 == 0 ? 15 : 7;
  char *stage = smem + wave * (32 * DV * 2);
#pragma unroll
  for (int dt = 0; dt < NDT; ++dt)
#pragma unroll
    for (int c = 0; c < 4; ++c)
      *reinterpret_cast<u32x2 *>(stage + r * (DV * 2) + (((4 * dt + c) ^ (r & MASK)) << 4) + 8 * h) =
          u32x2{pack_pair<Tag>(oacc[dt][4 * c] * inv, oacc[dt][4 * c + 1] * inv), pack_pair<Tag>(oacc[dt][4 * c + 2] * inv, oacc[dt][4 * c + 3] * inv)};
  const int row0 = qb * BM + wave * 32;
#pragma unroll
  for (int it = 0; it < CV / 2; ++it) {
    const int ci = it * 64 + lane, row = ci / CV, cc = ci % CV;
    const u32x4 v = *reinterpret_cast<const u32x4 *>(stage + row * (DV * 2) + ((cc ^ (row & MASK)) << 4));
    if (row0 + row < sq) *reinterpret_cast<u32x4 *>((T *)p.out + (int64_t)(q0 + row0 + row) * p.out_stride + (int64_t)head * DV + 8 * cc) = v;
  }
}

template <typename Tag, int DQ, int DV>
int launch(const MvLatentPrefillArgs &a, hipStream_t stream) {
  constexpr int lds = 2 * BN * (DQ + DV) * 2;
  constexpr bool wide_ok = 8 * 32 * DV * 2 <= lds;
  const bool wide = wide_ok && a.max_q >= 2048;   // 8 waves share a tile where the sequences are long enough
  const int bm = wide ? 256 : 128, blocks = (a.max_q + bm - 1) / bm;
  if (blocks > 65535 || a.n_seqs > 65535) return MV_E_SHAPE;
  const dim3 grid(a.heads, a.n_seqs, blocks);
  if (int e = mv_allow_lds<&latent_prefill_kernel<Tag, DQ, DV, 4>>()) return e;
  if constexpr (wide_ok) {
    if (int e = mv_allow_lds<&latent_prefill_kernel<Tag, DQ, DV, 8>>()) return e;
    if (wide) hipLaunchKernelGGL((latent_prefill_kernel<Tag, DQ, DV, 8>), grid, dim3(512), lds, stream, a);
  }
  if (!wide) hipLaunchKernelGGL((latent_prefill_kernel<Tag, DQ, DV, 4>), grid, dim3(256), lds, stream, a);
  MV_LAUNCH_CHECK();
  return MV_OK;
}

}  // namespace

int mv_latent_prefill_mfma_launch(const MvLatentPrefillArgs &a, int dtype, hipStream_t stream) {
  if (a.k_stride > 0x7fffffff || a.v_stride > 0x7fffffff || a.rot_stride > 0x7fffffff || a.rot_cols < 8) return MV_E_SHAPE;
#define MV_LP(DQ_, DV_) \
  if (a.dq == DQ_ && a.dv == DV_) return dtype == MV_BF16 ? launch<bf16_tag, DQ_, DV_>(a, stream) : launch<f16_tag, DQ_, DV_>(a, stream)
  MV_LP(64, 64);
  MV_LP(64, 128);
  MV_LP(128, 64);
  MV_LP(128, 128);
  MV_LP(192, 64);
  MV_LP(192, 128);
  MV_LP(192, 192);
  MV_LP(128, 192);
  MV_LP(256, 128);
  MV_LP(256, 192);
  MV_LP(256, 256);
#undef MV_LP
  return MV_E_SHAPE;
}
