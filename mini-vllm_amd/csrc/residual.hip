// K13 — steps of a 32-bit residual stream (models whose residual sum stays in fp32 whatever the activation dtype):
//   mv_residual_update: one launch per edge of the stream — [start the row from a scaled embedding] + the output of the
//     projections in front (plain, or RMS-normed by a weight of its own; or the fp32 partial sums of a K split; scaled by a
//     vector and a number)
//     [+ the scaled embedding] [+ a vector] -> the stream, and what the next projection reads: its RMSNorm or its cast;
//   mv_gated_lookup: gelu(s) * a slice of a per-token table (the per-token layer input);
//   mv_gated_lookup_linear: the same with the projection behind it, in one launch (decode-sized batches).
// One workgroup per row, the row in registers between the reductions and the store: the stream is read and written once.
#include "common.h"

namespace {

struct ResidualParams {
  float *x;                 // [rows][cols]
  const void *y;            // [rows] dtype rows (stride y_stride) or, y_splits > 0, fp32 [y_splits][rows][cols]
  const void *y_norm_w;     // RMS norm of y by a plain weight before it is added; NULL = y as it is
  const void *y_scale;      // dtype [cols], multiplies y behind its norm; NULL = ones
  const void *embed;        // dtype [vocab][cols]
  const int64_t *ids;
  const void *vec;          // dtype [cols], added to every row
  const void *norm_w;       // out = rms(x) * (norm_offset + norm_w); NULL: out = x rounded to dtype
  void *out;
  int64_t y_stride, out_stride, vocab;
  // see MvResidualArgs
  const void *y_norm_b, *norm_b, *pairs;
  const int64_t *positions;
  const int32_t *state_slots, *cu_q;
  int32_t *prev_tokens;
  const void *moe_out;
  const int32_t *moe_rows;
  const float *moe_w;
  int64_t buckets, mul_prev, mul_cur, slots;
  int n_seqs, moe_top;
  float embed_scale, norm_offset, eps, y_mult;
  int y_splits, embed_mode; // embed_mode: 0 none, 1 the row starts from the embedding, 2 the embedding is added
  int rows, cols, cols_true;
};

template <typename Tag>
__device__ __forceinline__ void load_row_vec(const typename elem<Tag>::T *p, float (&f)[elem<Tag>::VEC]) {
  const u32x4 raw = *reinterpret_cast<const u32x4 *>(p);
  if constexpr (elem<Tag>::VEC == 8) {
    unpack8<Tag>(raw, f);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) f[i] = u2f(raw[i]);
  }
}
template <typename Tag>
__device__ __forceinline__ void store_row_vec(typename elem<Tag>::T *p, const float (&f)[elem<Tag>::VEC]) {
  u32x4 raw;
  if constexpr (elem<Tag>::VEC == 8) {
    raw = pack8<Tag>(f);
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) raw[i] = f2u(f[i]);
  }
  *reinterpret_cast<u32x4 *>(p) = raw;
}
template <int VEC>
__device__ __forceinline__ void load_f32(const float *p, float (&f)[VEC]) {
#pragma unroll
  for (int q = 0; q < VEC / 4; ++q) {
    const f32x4 v = *reinterpret_cast<const f32x4 *>(p + 4 * q);
#pragma unroll
    for (int e = 0; e < 4; ++e) f[4 * q + e] = v[e];
  }
}

// sum over the workgroup, every thread gets it; red: one float per wave
__device__ __forceinline__ float group_sum(float x, float *red) {
  x = wave_sum(x);
  const int nw = blockDim.x >> 6;
  if (nw == 1) return x;
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = x;
  __syncthreads();
  float t = 0.f;
  for (int i = 0; i < nw; ++i) t += red[i];
  return t;
}

// Row of the pair table for this row's token (uniform in the workgroup); < 0: none.  The workgroup of a sequence's first row, the
// only one that reads the token kept from the step before, also keeps the step's last one.
__device__ __forceinline__ int64_t pair_row(const ResidualParams &p, int row, int64_t id) {
  int lo = row, first = row, last = row;
  if (p.cu_q) {
    lo = 0;
    for (int hi = p.n_seqs; hi - lo > 1;) {
      const int mid = (lo + hi) >> 1;
      if (p.cu_q[mid] <= row) lo = mid;
      else hi = mid;
    }
    first = p.cu_q[lo], last = p.cu_q[lo + 1] - 1;
  }
  const int64_t pos = p.positions[row];
  if (pos < 0) return -1;
  const int slot = p.state_slots[lo];
  const bool keep = slot >= 0 && slot < p.slots;
  int64_t prev = 0;
  if (row > first) {
    prev = p.ids[row - 1];
  } else {
    __shared__ int32_t kept;
    if (threadIdx.x == 0) {
      kept = pos > 0 && keep ? p.prev_tokens[(pos & 1) * p.slots + slot] : 0;
      if (keep) p.prev_tokens[((pos + last - first + 1) & 1) * p.slots + slot] = (int32_t)p.ids[last];
    }
    __syncthreads();
    prev = kept;
  }
  return pos == 0 ? p.buckets : (prev * p.mul_prev + id * p.mul_cur) % p.buckets;
}

// Per row z (held VEC at a time): the factors of its norm, (z - mean) * rs.  LN: mean over the true columns, else 0
template <bool LN, int MAXV, int VEC>
__device__ __forceinline__ float norm_factors(float (&z)[MAXV][VEC], int cols_true, float eps, float *red0, float *red1) {
  float ss = 0.f;
  if constexpr (LN) {
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < MAXV; ++i)
#pragma unroll
      for (int j = 0; j < VEC; ++j) sum += z[i][j];
    const float mean = group_sum(sum, red0) / (float)cols_true;
#pragma unroll
    for (int i = 0; i < MAXV; ++i)
#pragma unroll
      for (int j = 0; j < VEC; ++j) z[i][j] = (threadIdx.x + i * blockDim.x) * VEC + j < cols_true ? z[i][j] - mean : 0.f;
  }
#pragma unroll
  for (int i = 0; i < MAXV; ++i)
#pragma unroll
    for (int j = 0; j < VEC; ++j) ss = fmaf(z[i][j], z[i][j], ss);
  ss = group_sum(ss, red1);
  return 1.0f / sqrtf(ss / (float)cols_true + eps);
}

// MAXV = vectors per thread
template <typename Tag, int MAXV, bool LN>
__global__ void __launch_bounds__(1024) residual_update_kernel(ResidualParams p) {
  typedef typename elem<Tag>::T T;
  constexpr int VEC = elem<Tag>::VEC;
  __shared__ float red[4][16];
  const int row = blockIdx.x, nvec = p.cols / VEC;
  float x[MAXV][VEC], y[MAXV][VEC], e[MAXV][VEC], vv[MAXV][VEC], wy[MAXV][VEC], wn[MAXV][VEC], sy[MAXV][VEC];
  bool embed_ok = false;
  int64_t id = 0;
  if (p.embed_mode) {
    id = p.ids[row];
    embed_ok = id >= 0 && id < p.vocab;
  }
  const int64_t pair = embed_ok && p.pairs ? pair_row(p, row, id) : -1;
  // every load of the row before the first reduction
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * VEC;
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[i][j] = y[i][j] = e[i][j] = vv[i][j] = wy[i][j] = wn[i][j] = 0.f, sy[i][j] = 1.f;
    if (c < p.cols) {
      if (p.embed_mode != 1) load_f32<VEC>(p.x + (int64_t)row * p.cols + c, x[i]);
      if (p.y) {
        if (p.y_splits > 0) {
          const float *pp = (const float *)p.y + (int64_t)row * p.cols + c;
          load_f32<VEC>(pp, y[i]);
          for (int s = 1; s < p.y_splits; ++s) {
            float t[VEC];
            load_f32<VEC>(pp + (int64_t)s * p.rows * p.cols, t);
#pragma unroll
            for (int j = 0; j < VEC; ++j) y[i][j] += t[j];
          }
        } else {
          load_row_vec<Tag>((const T *)p.y + (int64_t)row * p.y_stride + c, y[i]);
        }
      }
      if (p.y_norm_w) load_row_vec<Tag>((const T *)p.y_norm_w + c, wy[i]);
      if (p.y_scale) load_row_vec<Tag>((const T *)p.y_scale + c, sy[i]);
      if (embed_ok) load_row_vec<Tag>((const T *)p.embed + id * p.cols + c, e[i]);
      if (pair >= 0) {
        float t[VEC];
        load_row_vec<Tag>((const T *)p.pairs + pair * p.cols + c, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) e[i][j] += t[j];
      }
      for (int k = 0; k < p.moe_top; ++k) {
        const int from = p.moe_rows[(int64_t)row * p.moe_top + k];
        const float mw = p.moe_w[(int64_t)row * p.moe_top + k];
        float t[VEC];
        if (from >= 0) load_row_vec<Tag>((const T *)p.moe_out + (int64_t)from * p.cols + c, t);
#pragma unroll
        for (int j = 0; j < VEC; ++j) y[i][j] = fmaf(mw, from >= 0 ? t[j] : x[i][j], y[i][j]);
      }
      if (p.vec) load_row_vec<Tag>((const T *)p.vec + c, vv[i]);
      if (p.norm_w) load_row_vec<Tag>((const T *)p.norm_w + c, wn[i]);
    }
  }
  if (p.y_norm_w) {
    const float rs = norm_factors<LN>(y, p.cols_true, p.eps, red[0], red[1]);
#pragma unroll
    for (int i = 0; i < MAXV; ++i) {
      const int c = (threadIdx.x + i * blockDim.x) * VEC;
      float b[VEC];
#pragma unroll
      for (int j = 0; j < VEC; ++j) b[j] = 0.f;
      if (LN && p.y_norm_b && c < p.cols) load_row_vec<Tag>((const T *)p.y_norm_b + c, b);
#pragma unroll
      for (int j = 0; j < VEC; ++j) y[i][j] = LN ? y[i][j] * rs * wy[i][j] + b[j] : y[i][j] * rs * wy[i][j];
    }
  }
  if (p.y_scale || p.y_mult != 1.0f) {
#pragma unroll
    for (int i = 0; i < MAXV; ++i)
#pragma unroll
      for (int j = 0; j < VEC; ++j) y[i][j] = y[i][j] * sy[i][j] * p.y_mult;
  }
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * VEC;
#pragma unroll
    for (int j = 0; j < VEC; ++j) x[i][j] = x[i][j] + y[i][j] + e[i][j] * p.embed_scale + vv[i][j];
    if (c < p.cols) {
      float *xr = p.x + (int64_t)row * p.cols + c;
#pragma unroll
      for (int q = 0; q < VEC / 4; ++q)
        *reinterpret_cast<f32x4 *>(xr + 4 * q) = f32x4{x[i][4 * q], x[i][4 * q + 1], x[i][4 * q + 2], x[i][4 * q + 3]};
    }
  }
  if (!p.out) return;
  float rs = 1.0f;
  if (p.norm_w) rs = norm_factors<LN>(x, p.cols_true, p.eps, red[2], red[3]);
#pragma unroll
  for (int i = 0; i < MAXV; ++i) {
    const int c = (threadIdx.x + i * blockDim.x) * VEC;
    if (c < p.cols) {
      float o[VEC], b[VEC];
#pragma unroll
      for (int j = 0; j < VEC; ++j) b[j] = 0.f;
      if (LN && p.norm_b) load_row_vec<Tag>((const T *)p.norm_b + c, b);
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        o[j] = p.norm_w ? x[i][j] * rs * (p.norm_offset + wn[i][j]) : x[i][j];
        if constexpr (LN) o[j] += b[j];
      }
      store_row_vec<Tag>((T *)p.out + (int64_t)row * p.out_stride + c, o);
    }
  }
}

// out[t][j] = gelu(s[t][j]) * table[ids[t]][offset + j] for j < dim, 0 for dim <= j < cols
template <typename Tag>
__global__ void __launch_bounds__(256) gated_lookup_kernel(const typename elem<Tag>::T *s, int64_t s_stride,
                                                           const typename elem<Tag>::T *table, int64_t table_stride,
                                                           int64_t vocab, int offset, const int64_t *ids,
                                                           typename elem<Tag>::T *out, int64_t out_stride, int rows,
                                                           int dim, int cols, bool table_vec) {
  constexpr int VEC = elem<Tag>::VEC;
  const int nvec = cols / VEC;
  const int64_t n = (int64_t)rows * nvec;
  for (int64_t v = (int64_t)blockIdx.x * 256 + threadIdx.x; v < n; v += (int64_t)gridDim.x * 256) {
    const int row = (int)(v / nvec), c = (int)(v - (int64_t)row * nvec) * VEC;
    const int64_t id = ids[row];
    const bool ok = id >= 0 && id < vocab;
    float a[VEC], e[VEC], o[VEC];
    load_row_vec<Tag>(s + (int64_t)row * s_stride + c, a);
    const typename elem<Tag>::T *tr = table + (ok ? id : 0) * table_stride + offset + c;
    if (table_vec && c + VEC <= dim) {
      load_row_vec<Tag>(tr, e);
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) e[j] = c + j < dim ? elem<Tag>::ld(tr[j]) : 0.f;
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = ok && c + j < dim ? gelu_tanh(a[j]) * e[j] : 0.f;
    store_row_vec<Tag>(out + (int64_t)row * out_stride + c, o);
  }
}

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef _Float16 f16x8 __attribute__((ext_vector_type(8)));

template <typename Tag>
__device__ __forceinline__ f32x4 side_mfma(u32x4 a, u32x4 b, f32x4 c) {
  if constexpr (__is_same(Tag, bf16_tag))
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), c, 0, 0, 0);
  else
    return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(f16x8, a), __builtin_bit_cast(f16x8, b), c, 0, 0, 0);
}

// out[t][n] = sum_j g[t][j] W[n][j], g = gated_lookup_kernel's row rounded to the dtype.  One workgroup: 16 tokens, whose rows
// of g it computes once, into LDS, in the MFMA B operand's order ([k-step][lane][8], lane l = token l & 15, k group l >> 4);
// then each wave walks blocks of 32 outputs.  W comes fragment-ordered (mv_pack_weight: [tile of 16][k-step][lane][8], lane =
// row + 16 * k group).  The two A fragments of a block take its rows as 8 (r >> 2) + (r & 3) and that + 4, so that a lane ends
// up with 8 consecutive outputs of its token: one 16-byte store.  The first kSideAhead k-steps of a wave's first block are in
// flight while the rows of g are computed.
constexpr int kSideAhead = 4, kSideMaxK = 512;
template <typename Tag>
__global__ void __launch_bounds__(256) gated_lookup_linear_kernel(const uint16_t *s, int64_t s_stride, const uint16_t *table,
                                                                  int64_t table_stride, int64_t vocab, int offset,
                                                                  const int64_t *ids, const uint16_t *wp, uint16_t *out,
                                                                  int64_t out_stride, int rows, int dim, int K, int N,
                                                                  bool table_vec) {
  extern __shared__ u32x4 g[];   // [K / 32][64]
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, steps = K / 32;
  const int64_t m0 = (int64_t)blockIdx.y * 16;
  const int r16 = lane & 15, kg = lane >> 4, n_pad = (N + 15) / 16 * 16, blocks = (N + 31) / 32, stride = gridDim.x * 4;
  const u32x4 *w = (const u32x4 *)wp;
  auto w_row = [&](int blk, int half) {   // this lane's row of W in half `half` of a block (clamped into the packed copy)
    int n = blk * 32 + (r16 >> 2) * 8 + (r16 & 3) + half * 4;
    n = n < n_pad ? n : n_pad - 1;
    return w + (int64_t)(n >> 4) * steps * 64 + kg * 16 + (n & 15);
  };
  u32x4 wf[kSideAhead][2];
  auto preload = [&](int blk) {
    const u32x4 *a = w_row(blk, 0), *b = w_row(blk, 1);
#pragma unroll
    for (int i = 0; i < kSideAhead; ++i) {
      const int k = i < steps ? i : steps - 1;
      wf[i][0] = a[k * 64], wf[i][1] = b[k * 64];
    }
  };
  int blk = blockIdx.x * 4 + wave;
  preload(blk < blocks ? blk : blocks - 1);
  for (int v = threadIdx.x; v < steps * 64; v += 256) {
    const int l = v & 63, c = (v >> 6) * 32 + (l >> 4) * 8;
    const int64_t m = m0 + (l & 15);
    float a[8], e[8], o[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) o[j] = 0.f;
    const int64_t id = m < rows ? ids[m] : -1;
    if (id >= 0 && id < vocab && c < dim) {
      load_row_vec<Tag>(s + m * s_stride + c, a);
      const uint16_t *tr = table + id * table_stride + offset + c;
      if (table_vec && c + 8 <= dim) {
        load_row_vec<Tag>(tr, e);
      } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) e[j] = c + j < dim ? elem<Tag>::ld(tr[j]) : 0.f;
      }
#pragma unroll
      for (int j = 0; j < 8; ++j) o[j] = c + j < dim ? gelu_tanh(a[j]) * e[j] : 0.f;
    }
    g[v] = pack8<Tag>(o);
  }
  __syncthreads();
  for (; blk < blocks; blk += stride) {
    f32x4 acc[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int i = 0; i < kSideAhead; ++i)
      if (i < steps) {
        const u32x4 x = g[i * 64 + lane];
        acc[0] = side_mfma<Tag>(wf[i][0], x, acc[0]);
        acc[1] = side_mfma<Tag>(wf[i][1], x, acc[1]);
      }
    if (steps > kSideAhead) {
      const u32x4 *a = w_row(blk, 0), *b = w_row(blk, 1);
      for (int i = kSideAhead; i < steps; ++i) {
        const u32x4 x = g[i * 64 + lane];
        acc[0] = side_mfma<Tag>(a[i * 64], x, acc[0]);
        acc[1] = side_mfma<Tag>(b[i * 64], x, acc[1]);
      }
    }
    if (blk + stride < blocks) preload(blk + stride);
    const int64_t m = m0 + r16;
    const int n = blk * 32 + kg * 8;
    if (m < rows && n < N) {
      const float o[8] = {acc[0][0], acc[0][1], acc[0][2], acc[0][3], acc[1][0], acc[1][1], acc[1][2], acc[1][3]};
      const u32x4 pk = pack8<Tag>(o);
      uint16_t *dst = out + m * out_stride + n;
      if (n + 8 <= N) *(u32x4 *)dst = pk;
      else *(u32x2 *)dst = u32x2{pk[0], pk[1]};   // N % 4 == 0: four outputs are left
    }
  }
}

}  // namespace

extern "C" int mv_residual_update(const MvResidualArgs *a, int rows, int cols, int cols_true, int dtype, void *stream) {
  if (rows == 0) return MV_OK;
  if (!a || !a->x) return MV_E_NULLPTR;
  if (rows < 0 || cols <= 0 || cols_true <= 0 || cols_true > cols || a->y_splits < 0) return MV_E_SHAPE;
  if (dtype != MV_BF16 && dtype != MV_F16 && dtype != MV_F32) return MV_E_DTYPE;
  if (a->embed_mode < 0 || a->embed_mode > 2) return MV_E_RANGE;
  if (a->embed_mode && (!a->embed || !a->ids || a->vocab <= 0)) return MV_E_NULLPTR;
  if ((a->y_norm_w || a->y_scale) && !a->y && a->moe_top == 0) return MV_E_NULLPTR;
  if (a->moe_top < 0 || (!a->layer_norm && (a->y_norm_b || a->norm_b))) return MV_E_SHAPE;
  if (a->moe_top && (!a->moe_out || !a->moe_rows || !a->moe_w || a->embed_mode == 1)) return MV_E_NULLPTR;
  if (a->pairs) {
    if (!a->embed_mode || !a->positions || !a->state_slots || (a->slots > 0 && !a->prev_tokens)) return MV_E_NULLPTR;
    if (a->buckets <= 0 || a->mul_prev < 0 || a->mul_cur < 0 || a->slots < 0 || (a->cu_q && a->n_seqs <= 0)) return MV_E_SHAPE;
  }
  const int vec = dtype == MV_F32 ? 4 : 8;
  if (cols % vec) return MV_E_SHAPE;
  if (!mv_aligned16(a->x) || (a->y && !mv_aligned16(a->y)) || (a->y_norm_w && !mv_aligned16(a->y_norm_w)) || (a->y_scale && !mv_aligned16(a->y_scale)) ||
      (a->embed_mode && !mv_aligned16(a->embed)) || (a->vec && !mv_aligned16(a->vec)) ||
      (a->norm_w && !mv_aligned16(a->norm_w)) || (a->y_norm_b && !mv_aligned16(a->y_norm_b)) ||
      (a->norm_b && !mv_aligned16(a->norm_b)) || (a->pairs && !mv_aligned16(a->pairs)) ||
      (a->moe_top && !mv_aligned16(a->moe_out)) || (a->out && (!mv_aligned16(a->out) || a->out_stride % vec)) ||
      (a->y && a->y_splits == 0 && a->y_stride % vec))
    return MV_E_ALIGN;
  ResidualParams p;
  p.x = a->x, p.y = a->y, p.y_norm_w = a->y_norm_w, p.embed = a->embed, p.ids = a->ids, p.vec = a->vec;
  p.norm_w = a->norm_w, p.out = a->out, p.y_stride = a->y_stride, p.out_stride = a->out_stride, p.vocab = a->vocab;
  p.y_scale = a->y_scale, p.y_mult = a->y_mult;
  p.embed_scale = a->embed_scale, p.norm_offset = a->norm_offset, p.eps = a->eps;
  p.y_norm_b = a->y_norm_b, p.norm_b = a->norm_b, p.pairs = a->pairs, p.positions = a->positions;
  p.state_slots = a->state_slots, p.cu_q = a->cu_q, p.prev_tokens = a->prev_tokens;
  p.moe_out = a->moe_out, p.moe_rows = a->moe_rows, p.moe_w = a->moe_w, p.moe_top = a->moe_top;
  p.buckets = a->buckets, p.mul_prev = a->mul_prev, p.mul_cur = a->mul_cur, p.slots = a->slots, p.n_seqs = a->n_seqs;
  p.y_splits = a->y_splits, p.embed_mode = a->embed_mode, p.rows = rows, p.cols = cols, p.cols_true = cols_true;
  const int nvec = cols / vec;
  int threads = (nvec + 63) / 64 * 64;
  if (threads > 1024) threads = 1024;
  const int per = (nvec + threads - 1) / threads;
  hipStream_t st = (hipStream_t)stream;
#define MV_RES(MV)                                                                                                              \
  MV_DISPATCH_DTYPE(dtype, {                                                                                                    \
    if (a->layer_norm) hipLaunchKernelGGL((residual_update_kernel<Tag, MV, true>), dim3(rows), dim3(threads), 0, st, p);       \
    else hipLaunchKernelGGL((residual_update_kernel<Tag, MV, false>), dim3(rows), dim3(threads), 0, st, p);                    \
  })
  if (per <= 1) MV_RES(1)
  else if (per <= 2) MV_RES(2)
  else return MV_E_SHAPE;   // > 16384 (16-bit) / 8192 (fp32) columns
#undef MV_RES
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_gated_lookup(const void *s, int64_t s_stride, const void *table, int64_t table_stride, int64_t vocab,
                               int offset, const int64_t *ids, void *out, int64_t out_stride, int rows, int dim, int cols,
                               int dtype, void *stream) {
  if (rows == 0) return MV_OK;
  if (!s || !table || !ids || !out) return MV_E_NULLPTR;
  if (rows < 0 || dim <= 0 || cols < dim || vocab <= 0 || offset < 0 || offset + dim > table_stride) return MV_E_SHAPE;
  if (dtype != MV_BF16 && dtype != MV_F16 && dtype != MV_F32) return MV_E_DTYPE;
  const int vec = dtype == MV_F32 ? 4 : 8;
  if (cols % vec) return MV_E_SHAPE;
  if (!mv_aligned16(s) || !mv_aligned16(out) || s_stride % vec || out_stride % vec) return MV_E_ALIGN;
  const bool table_vec = mv_aligned16(table) && table_stride % vec == 0 && offset % vec == 0;
  int64_t blocks = ((int64_t)rows * (cols / vec) + 255) / 256;
  if (blocks > 8192) blocks = 8192;
  MV_DISPATCH_DTYPE(dtype, {
    typedef typename elem<Tag>::T T;
    hipLaunchKernelGGL((gated_lookup_kernel<Tag>), dim3((unsigned)blocks), dim3(256), 0, (hipStream_t)stream, (const T *)s,
                       s_stride, (const T *)table, table_stride, vocab, offset, ids, (T *)out, out_stride, rows, dim, cols,
                       table_vec);
  });
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_gated_lookup_linear(const void *s, int64_t s_stride, const void *table, int64_t table_stride, int64_t vocab,
                                      int offset, const int64_t *ids, const void *w_packed, void *out, int64_t out_stride,
                                      int rows, int dim, int k, int n, int dtype, void *stream) {
  if (rows == 0 || n == 0) return MV_OK;
  if (!s || !table || !ids || !w_packed || !out) return MV_E_NULLPTR;
  if (dtype != MV_BF16 && dtype != MV_F16) return dtype == MV_F32 ? MV_E_SHAPE : MV_E_DTYPE;
  if (rows < 0 || dim <= 0 || k < dim || vocab <= 0 || offset < 0 || offset + dim > table_stride || n < 0 || (n & 3))
    return MV_E_SHAPE;
  if ((k & 31) || k > kSideMaxK) return MV_E_SHAPE;
  if (!mv_aligned16(s) || !mv_aligned16(w_packed) || !mv_aligned16(out) || (s_stride & 7) || (out_stride & 7)) return MV_E_ALIGN;
  const bool table_vec = mv_aligned16(table) && table_stride % 8 == 0 && offset % 8 == 0;
  const int row_blocks = (rows + 15) / 16, split_max = (n + 127) / 128;
  if (row_blocks > 65535) return MV_E_SHAPE;
  const int split = (2048 + row_blocks - 1) / row_blocks;
  const dim3 grid((unsigned)(split < split_max ? split : split_max), (unsigned)row_blocks);
#define MV_SIDE(TAG)                                                                                                          \
  hipLaunchKernelGGL((gated_lookup_linear_kernel<TAG>), grid, dim3(256), (size_t)k * 32, (hipStream_t)stream,                   \
                     (const uint16_t *)s, s_stride, (const uint16_t *)table, table_stride, vocab, offset, ids,                  \
                     (const uint16_t *)w_packed, (uint16_t *)out, out_stride, rows, dim, k, n, table_vec)
  if (dtype == MV_BF16) MV_SIDE(bf16_tag);
  else MV_SIDE(f16_tag);
#undef MV_SIDE
  MV_LAUNCH_CHECK();
  return MV_OK;
}
