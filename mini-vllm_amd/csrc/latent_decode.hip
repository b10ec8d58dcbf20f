// K14 — latent attention, decode on the matrix cores (16-bit): every head's query row against the cached rows themselves
// (scores over the whole row, values = its latent columns), so a row is read from HBM once for all heads.
//
// One workgroup = 4 waves = up to 16 HG heads of one sequence and one part of its visible keys; tiles of 32 keys (one page each) in
// a ring of four LDS buffers filled by LDS-DMA, three tiles in flight, one workgroup per CU.  LDS rows have an odd number of 16-byte chunks, so neither the row
// reads nor the transposed reads meet in a bank.  Per tile:
//   S^T[key][head] = rows . Q^T     wave w: keys 16 (w & 1) .., heads 16 (w >> 1) .. (HG = 1: two waves do the same work)
//   softmax                         running maxima per head, exchanged through LDS; probabilities to LDS as 16-bit rows
//   O^T[column][head] += V^T P^T    wave w: a quarter of the latent columns, all heads; V^T by transposed LDS reads
// A context in several parts leaves fp32 sums and (maximum, sum) pairs in the workspace; a second launch merges them.
#include "latent.h"

namespace {

typedef __attribute__((ext_vector_type(4))) short s16x4;
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;

constexpr int TK = 32;    // keys per tile
constexpr int NBUF = 4;   // tiles in LDS
constexpr int kMaxRot = 64, kMaxSplits = 64;

struct DecodeParams {
  const void *q, *plane;
  const int32_t *tables, *lens;
  void *out;
  float *part, *part_ml;   // [batch][heads][splits][kv_cols], [batch][heads][splits][2]
  int64_t table_stride, num_blocks;
  int heads, kv_cols, cols, block_size, max_blocks, window, splits;
  float scale;
};

__host__ __device__ constexpr int lds_chunks(int cols) { return cols / 8 + 1 - (cols / 8 & 1); }   // odd

// CT: latent column tiles of 16 per wave (kv_cols = 64 CT); RT: rotated columns / 32
template <typename Tag, int HG, int CT, int RT>
__global__ void __launch_bounds__(256, 2) latent_decode_kernel(DecodeParams p) {
  typedef typename elem<Tag>::T T;
  constexpr int KS = 2 * CT + RT, COLS = KS * 32, CH = lds_chunks(COLS), RB = CH * 16;   // 32-column steps of a row; its LDS form
  // 1-KiB transfers of a tile; every wave issues PERW of them (the surplus ones land in a spare KiB), so that a count of
  // outstanding transfers is a count of tiles
  constexpr int DMAS = (TK * CH + 63) / 64, BUF = DMAS * 1024, PERW = (DMAS + 3) / 4;
  static_assert((NBUF - 2) * PERW < 64);
  extern __shared__ __attribute__((aligned(16))) char smem[];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), r16 = lane & 15, g = lane >> 4;
  const int split = blockIdx.x, h0 = blockIdx.y * 16 * HG, b = blockIdx.z;
  char *spare = smem + NBUF * BUF;
  float *smax = (float *)(spare + 1024);                        // [2 key halves][16 HG heads]
  char *prob = (char *)(smax + 2 * 16 * HG);                    // [16 HG heads][TK] 16-bit, rows of 80 bytes
  constexpr int PR = 80;
  const int len = min(p.lens[b], p.max_blocks * p.block_size), lo = p.window > 0 && len > p.window ? len - p.window : 0;
  const int first = lo / TK, tiles = len > 0 ? (len + TK - 1) / TK - first : 0, per = (tiles + p.splits - 1) / p.splits;
  const int t0 = first + split * per, t1 = min(first + tiles, t0 + per);

  // Q^T fragments of this wave's heads
  const int kg = wave & 1, hg = HG == 2 ? wave >> 1 : 0, qh = h0 + hg * 16 + r16;
  u32x4 qf[KS];
  {
    const T *qp = (const T *)p.q + ((int64_t)b * p.heads + min(qh, p.heads - 1)) * COLS + g * 8;
#pragma unroll
    for (int s = 0; s < KS; ++s) qf[s] = *(const u32x4 *)(qp + s * 32);
  }
  settle(qf);
  f32x4 acc[HG][CT] = {};
  float m_run[HG], l_run[HG];
#pragma unroll
  for (int i = 0; i < HG; ++i) m_run[i] = -1e30f, l_run[i] = 0.f;
  const float scale_log2 = p.scale * 1.4426950408889634f;

  // pages: lane i of every wave holds table entry page_base + i (no load per tile: a scalar one would break the hand-counted
  // waits, a vector one would sit among the counted transfers)
  const int tpb = p.block_size / TK;
  int page_base = t0 / tpb, pages = 0;
  auto load_pages = [&]() {
    const int e = page_base + lane;
    const int blk = e < p.max_blocks ? p.tables[b * p.table_stride + e] : -1;
    pages = blk >= 0 && blk < p.num_blocks ? blk : -1;
  };
  if (t0 < t1) load_pages();
  auto page = [&](int t) {   // of a tile, or -1; t does not decrease
    const int e = t / tpb;
    if (e >= page_base + 64) {
      page_base = e;
      load_pages();
    }
    return __builtin_amdgcn_readlane(pages, e - page_base);
  };
  const int row_first = (wave * 64 + lane) / CH, col_first = (wave * 64 + lane) % CH;
  auto dma = [&](int t, int blk, int buf) {   // (a page that is not there: block 0, whose rows are then not used)
    const T *src = (const T *)p.plane + ((int64_t)max(blk, 0) * p.block_size + t * TK % p.block_size) * COLS;
    const int last = min(TK, len - t * TK) - 1;   // rows past the end re-read the last key (probability 0, finite data)
    int row = row_first, col = col_first;
#pragma unroll
    for (int i = 0; i < PERW; ++i) {
      __builtin_amdgcn_global_load_lds(
          (const __attribute__((address_space(1))) void *)(src + (min(row, last) * COLS + min(col, COLS / 8 - 1) * 8)),
          (__attribute__((address_space(3))) void *)(4 * i + wave < DMAS ? smem + buf * BUF + (4 * i + wave) * 1024 : spare), 16, 0, 0);
      row += 256 / CH, col += 256 % CH;
      if (col >= CH) col -= CH, ++row;
    }
  };

  int blk[NBUF];   // pages of the tiles in flight
#pragma unroll
  for (int i = 0; i < NBUF - 1; ++i)
    if (t0 + i < t1) dma(t0 + i, blk[i] = page(t0 + i), i);
  const uint32_t lds0 = lds_address(smem), smax_a = lds_address(smax) + r16 * 4, prob_a = lds_address(prob) + r16 * PR + g * 16;
  const uint32_t ka0 = lds0 + (kg * 16 + r16) * RB + g * 16, va0 = lds0 + (g * 8 + (r16 >> 2)) * RB + (r16 & 3) * 8 + wave * 32;
  int buf = 0;
  for (int t = t0; t < t1; ++t, buf = (buf + 1) & (NBUF - 1)) {
    // this wave's share of tile t has landed (newer tiles stay in flight); behind the barrier everybody's has, and the buffer
    // of tile t - 1 is free
    const int newer = t1 - 1 - t;
    if (newer >= NBUF - 2) asm volatile("s_waitcnt vmcnt(%0)" ::"n"((NBUF - 2) * PERW) : "memory");
    else if (newer == 1) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(PERW) : "memory");
    else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    lds_barrier();
    if (t + NBUF - 1 < t1) dma(t + NBUF - 1, blk[NBUF - 1] = page(t + NBUF - 1), (buf + NBUF - 1) & (NBUF - 1));
    if (blk[0] >= 0) {
      // ---- scores: 16 keys x 16 heads, row fragments some steps ahead
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");   // (nothing else may be counted below)
      f32x4 s = {0.f, 0.f, 0.f, 0.f}, s2 = {0.f, 0.f, 0.f, 0.f};   // (two chains: half the dependent latency)
      const uint32_t ka = ka0 + buf * BUF, va = va0 + buf * BUF;
      constexpr int AHEAD = KS < (HG == 2 ? 6 : 12) ? KS : (HG == 2 ? 6 : 12);
      u32x4 kf[KS];
      static_for<AHEAD>([&](auto I) { lds_read128<decltype(I)::value * 64>(kf[decltype(I)::value], ka); });
      static_for<KS>([&](auto I) {
        constexpr int i = decltype(I)::value, newer = KS - 1 - i < AHEAD - 1 ? KS - 1 - i : AHEAD - 1;
        lds_wait<newer>(kf[i]);
        if constexpr (i % 2 == 0) s = mfma16x16x32<Tag>(kf[i], qf[i], s);
        else s2 = mfma16x16x32<Tag>(kf[i], qf[i], s2);
        if constexpr (i + AHEAD < KS) lds_read128<(i + AHEAD) * 64>(kf[i + AHEAD], ka);
      });
      s += s2;
      float mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int key = t * TK + kg * 16 + g * 4 + i;
        s[i] = key < len && key >= lo ? s[i] * scale_log2 : -INFINITY;
        mx = fmaxf(mx, s[i]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      if (g == 0) smax[kg * 16 * HG + hg * 16 + r16] = mx;
      lds_barrier();
      // the value fragments' first reads go out under the softmax
      constexpr int VA = CT < 4 ? CT : 4;
      u32x2 v0[CT], v1[CT];
      float alpha[HG], top[2][HG];
      static_for<HG>([&](auto I) {
        lds_read32<decltype(I)::value * 64>(top[0][decltype(I)::value], smax_a);
        lds_read32<(HG + decltype(I)::value) * 64>(top[1][decltype(I)::value], smax_a);
      });
      static_for<VA>([&](auto C) {
        lds_read64_tr<decltype(C)::value * 128>(v0[decltype(C)::value], va);
        lds_read64_tr<4 * RB + decltype(C)::value * 128>(v1[decltype(C)::value], va);
      });
#pragma unroll
      for (int i = 0; i < HG; ++i) {
        lds_wait<2 * VA>(top[0][i], top[1][i]);   // (in order: all of them are older than the 2 VA value reads)
        const float m_new = fmaxf(m_run[i], fmaxf(top[0][i], top[1][i]));
        alpha[i] = __builtin_amdgcn_exp2f(m_run[i] - m_new);
        m_run[i] = m_new;
        l_run[i] *= alpha[i];
      }
      float e[4], sum = 0.f;
      const float m_own = HG == 2 && hg ? m_run[HG - 1] : m_run[0];
#pragma unroll
      for (int i = 0; i < 4; ++i) e[i] = __builtin_amdgcn_exp2f(s[i] - m_own), sum += e[i];
      if (HG == 2 && hg) l_run[HG - 1] += sum;
      else l_run[0] += sum;
      if (HG == 2 || wave < 2)
        *(u32x2 *)(prob + (hg * 16 + r16) * PR + (kg * 16 + g * 4) * 2) =
            u32x2{pack_pair<Tag>(e[0], e[1]), pack_pair<Tag>(e[2], e[3])};
      lds_barrier();
      // ---- values
      u32x4 pf[HG];
      static_for<HG>([&](auto I) { lds_read128<decltype(I)::value * 16 * PR>(pf[decltype(I)::value], prob_a); });
      static_for<HG>([&](auto I) { lds_wait<0>(pf[decltype(I)::value]); });
      static_for<VA>([&](auto C) { lds_wait<0>(v0[decltype(C)::value], v1[decltype(C)::value]); });
      static_for<CT>([&](auto C) {
        constexpr int c = decltype(C)::value;
        if constexpr (c >= VA) lds_wait<(CT - 1 - c < VA - 1 ? CT - 1 - c : VA - 1) * 2>(v0[c], v1[c]);
        if constexpr (c + VA < CT) {
          lds_read64_tr<(c + VA) * 128>(v0[c + VA], va);
          lds_read64_tr<4 * RB + (c + VA) * 128>(v1[c + VA], va);
        }
        const u32x4 a = {v0[c].x, v0[c].y, v1[c].x, v1[c].y};
#pragma unroll
        for (int i = 0; i < HG; ++i) acc[i][c] = mfma16x16x32<Tag>(a, pf[i], acc[i][c] * alpha[i]);
      });
    }
#pragma unroll
    for (int i = 0; i < NBUF - 1; ++i) blk[i] = blk[i + 1];
  }
  __syncthreads();
  // ---- sums of a head: over the waves that scored it (its two key halves) and their four lane groups
  float *sl = smax;   // [2][16 HG]
  {
    float l = HG == 2 && hg ? l_run[HG - 1] : l_run[0];
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
    if (g == 0 && (HG == 2 || wave < 2)) sl[kg * 16 * HG + hg * 16 + r16] = l;
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < HG; ++i) {
    const int head = h0 + i * 16 + r16;
    if (head >= p.heads) continue;
    const float l = sl[i * 16 + r16] + sl[16 * HG + i * 16 + r16];
    const int64_t row = (int64_t)b * p.heads + head;
    if (p.splits == 1) {
      const float inv = l > 0.f ? 1.0f / l : 0.f;
      T *o = (T *)p.out + row * p.kv_cols + wave * 16 + g * 4;
#pragma unroll
      for (int c = 0; c < CT; ++c) *(u32x2 *)(o + c * 64) = pack_quad<Tag>(acc[i][c] * inv);
    } else {
      float *o = p.part + (row * p.splits + split) * p.kv_cols + wave * 16 + g * 4;
#pragma unroll
      for (int c = 0; c < CT; ++c) *(f32x4 *)(o + c * 64) = acc[i][c];
      if (wave == 0 && g == 0) {
        float *ml = p.part_ml + (row * p.splits + split) * 2;
        ml[0] = m_run[i], ml[1] = l;
      }
    }
  }
}

// one (sequence, head) per workgroup: 4 columns per thread, the parts dealt to blockDim.x / (kv_cols / 4) groups of threads
template <typename Tag>
__global__ void __launch_bounds__(256) latent_merge_kernel(const float *part, const float *part_ml, void *out, int splits, int kv_cols) {
  typedef typename elem<Tag>::T T;
  __shared__ float w[kMaxSplits];
  __shared__ f32x4 sums[256];
  const int64_t row = blockIdx.x;
  const int tid = threadIdx.x, per = kv_cols / 4, groups = 256 / per, c = tid % per, first = tid / per;
  float total;
  {
    const float *ml = part_ml + row * splits * 2;
    const int lane = tid & 63;      // (kMaxSplits = one wave)
    const float m = lane < splits ? ml[2 * lane] : -1e30f, l = lane < splits ? ml[2 * lane + 1] : 0.f;
    const float top = wave_max(l > 0.f ? m : -1e30f);   // (all lanes take part)
    const float e = l > 0.f ? __builtin_amdgcn_exp2f(m - top) : 0.f;
    total = wave_sum(l * e);
    if (tid < splits) w[tid] = e;
  }
  __syncthreads();
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  if (first < groups) {
    const float *p = part + row * splits * kv_cols + 4 * c;
#pragma unroll 4
    for (int s = first; s < splits; s += groups) {
      const f32x4 v = *(const f32x4 *)(p + (int64_t)s * kv_cols);
      o += w[s] > 0.f ? v * w[s] : f32x4{0.f, 0.f, 0.f, 0.f};
    }
  }
  sums[tid] = o;
  __syncthreads();
  if (tid < per) {
    for (int i = 1; i < groups; ++i) o += sums[i * per + tid];
    *(u32x2 *)((T *)out + row * kv_cols + 4 * c) = pack_quad<Tag>(o * (total > 0.f ? 1.0f / total : 0.f));
  }
}

int head_groups(int heads) { return heads > 16 ? 2 : 1; }

// parts of a context: enough workgroups for every CU, at least two tiles each
int split_count(int batch, int heads, int block_size, int max_blocks, int window) {
  const int hg = head_groups(heads), wgs = batch * ((heads + 16 * hg - 1) / (16 * hg));
  int64_t keys = (int64_t)max_blocks * block_size;
  if (window > 0 && keys > window) keys = window;
  const int64_t tiles = (keys + 2 * TK - 2) / TK;
  int64_t s = (256 + wgs - 1) / wgs;
  if (s > tiles / 2) s = tiles / 2;
  if (s > kMaxSplits) s = kMaxSplits;
  return s < 1 ? 1 : (int)s;
}

template <typename Tag, int HG>
int launch(const DecodeParams &p, const dim3 &grid, size_t lds, hipStream_t stream) {
#define MV_LD(CT_, RT_)                                                                                     \
  if (p.kv_cols == 64 * CT_ && p.cols - p.kv_cols == 32 * RT_) {                                            \
    if (int e = mv_allow_lds<&latent_decode_kernel<Tag, HG, CT_, RT_>>()) return e;                         \
    hipLaunchKernelGGL((latent_decode_kernel<Tag, HG, CT_, RT_>), grid, dim3(256), lds, stream, p);          \
    MV_LAUNCH_CHECK();                                                                                      \
    return MV_OK;                                                                                           \
  }
#define MV_LDR(CT_) MV_LD(CT_, 1) MV_LD(CT_, 2)
  MV_LDR(1)
  MV_LDR(2)
  MV_LDR(3)
  MV_LDR(4)
  MV_LDR(5)
  MV_LDR(6)
  MV_LDR(7)
  MV_LDR(8)
#undef MV_LDR
#undef MV_LD
  return MV_E_SHAPE;
}

}  // namespace

size_t mv_latent_decode_mfma_workspace(int batch, int heads, int kv_cols, int rot_cols, int block_size, int max_blocks, int window) {
  const int s = split_count(batch, heads, block_size, max_blocks, window);
  return s == 1 ? 256 : ((size_t)batch * heads * s * (kv_cols + 2) * 4 + 255) / 256 * 256;
}

int mv_latent_decode_mfma_launch(const void *q, const void *plane, const int32_t *tables, int64_t table_stride,
                                 const int32_t *lens, void *out, int batch, int heads, int kv_cols, int rot_cols, int block_size,
                                 int max_blocks, int64_t num_blocks, int window, float scale, void *workspace,
                                 size_t workspace_bytes, int dtype, hipStream_t stream) {
  if ((kv_cols & 63) || kv_cols > 512 || rot_cols > kMaxRot || block_size % TK || batch > 65535) return MV_E_SHAPE;
  const int splits = split_count(batch, heads, block_size, max_blocks, window), hg = head_groups(heads);
  if (splits > 1 && (!workspace || workspace_bytes < mv_latent_decode_mfma_workspace(batch, heads, kv_cols, rot_cols, block_size,
                                                                                     max_blocks, window)))
    return MV_E_WORKSPACE;
  DecodeParams p;
  p.q = q, p.plane = plane, p.tables = tables, p.lens = lens, p.out = out;
  p.part = (float *)workspace, p.part_ml = p.part + (int64_t)batch * heads * splits * kv_cols;
  p.table_stride = table_stride, p.num_blocks = num_blocks, p.heads = heads, p.kv_cols = kv_cols, p.cols = kv_cols + rot_cols;
  p.block_size = block_size, p.max_blocks = max_blocks, p.window = window, p.splits = splits, p.scale = scale;
  const int CH = lds_chunks(p.cols);
  const size_t lds = (size_t)(NBUF * ((TK * CH + 63) / 64) + 1) * 1024 + 2 * 16 * hg * 4 + 16 * hg * 80;
  const dim3 grid(splits, (heads + 16 * hg - 1) / (16 * hg), batch);
  int rc;
  if (dtype == MV_BF16) rc = hg == 2 ? launch<bf16_tag, 2>(p, grid, lds, stream) : launch<bf16_tag, 1>(p, grid, lds, stream);
  else rc = hg == 2 ? launch<f16_tag, 2>(p, grid, lds, stream) : launch<f16_tag, 1>(p, grid, lds, stream);
  if (rc != MV_OK || splits == 1) return rc;
  const int rows = batch * heads;
  if (dtype == MV_BF16)
    hipLaunchKernelGGL((latent_merge_kernel<bf16_tag>), dim3(rows), dim3(256), 0, stream, p.part, p.part_ml, out, splits, kv_cols);
  else
    hipLaunchKernelGGL((latent_merge_kernel<f16_tag>), dim3(rows), dim3(256), 0, stream, p.part, p.part_ml, out, splits, kv_cols);
  MV_LAUNCH_CHECK();
  return MV_OK;
}
