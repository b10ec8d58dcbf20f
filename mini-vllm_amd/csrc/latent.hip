// K14 — latent attention: what surrounds the two attention kernels (latent_decode.hip, latent_prefill.hip).
//   mv_latent_prep:   the norms of the query latent and of the cached latent, rotation of the shared key part, cache store;
//   mv_head_linear:   per-head products (query into the latent's coordinates, with its rotation; latent output to values);
//   mv_latent_gather: cached rows of a batch of sequences, contiguous (prefill of portions).
#include "latent.h"

namespace {

// cos / sin of the VEC columns from `c` on of a rotated part of 2 * pairs columns, applied in place; 0 behind it
template <int VEC>
__device__ __forceinline__ void rotate_cols(float (&x)[VEC], const float *cos, const float *sin, int64_t pos, bool pos_ok,
                                            int c, int pairs) {
#pragma unroll
  for (int j = 0; j < VEC; j += 2) {
    const int i = (c + j) >> 1;
    if (i < pairs) {
      const float cs = pos_ok ? cos[pos * pairs + i] : 1.0f, sn = pos_ok ? sin[pos * pairs + i] : 0.0f;
      const float u = x[j], v = x[j + 1];
      x[j] = __fsub_rn(__fmul_rn(u, cs), __fmul_rn(v, sn));
      x[j + 1] = __fadd_rn(__fmul_rn(v, cs), __fmul_rn(u, sn));
    } else {
      x[j] = x[j + 1] = 0.f;
    }
  }
}

template <typename Tag>
__global__ void __launch_bounds__(256) latent_prep_kernel(MvLatentPrepArgs p) {
  typedef typename elem<Tag>::T T;
  constexpr int VEC = elem<Tag>::VEC;
  __shared__ float red[2][4];
  const int row = blockIdx.x, tid = threadIdx.x;
  const T *z = (const T *)p.z + (int64_t)row * p.z_stride;
  const int nq = p.q_cols / VEC, nk = p.kv_rank ? p.kv_cols / VEC : 0, nr = p.kv_rank ? p.rot_cols / VEC : 0;
  float sq = 0.f, sk = 0.f;
  for (int i = tid; i < nq + nk; i += 256) {
    float f[VEC];
    load_vec_row<Tag>(z + (i < nq ? p.q_off + i * VEC : p.kv_off + (i - nq) * VEC), f);
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < VEC; ++j) s = fmaf(f[j], f[j], s);
    if (i < nq) sq += s;
    else sk += s;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  if ((tid & 63) == 0) red[0][tid >> 6] = sq, red[1][tid >> 6] = sk;
  __syncthreads();
  sq = (red[0][0] + red[0][1]) + (red[0][2] + red[0][3]);
  sk = (red[1][0] + red[1][1]) + (red[1][2] + red[1][3]);
  const float rq = 1.0f / sqrtf(sq / (float)p.q_rank + p.eps);
  const float rk = p.kv_rank ? 1.0f / sqrtf(sk / (float)p.kv_rank + p.eps) : 0.f;
  const int cols = p.kv_cols + p.rot_cols;
  const int64_t slot = p.plane && p.slot_mapping ? p.slot_mapping[row] : -1;
  T *dst = slot >= 0 && slot < p.num_slots ? (T *)p.plane + slot * cols : nullptr;
  T *rows = p.rows_out ? (T *)p.rows_out + (int64_t)row * cols : nullptr;
  const int64_t pos = nr ? p.positions[row] : 0;
  const bool pos_ok = pos >= 0 && pos < p.max_pos;
  for (int i = tid; i < nq + nk + nr; i += 256) {
    float f[VEC], w[VEC];
    if (i < nq) {
      load_vec_row<Tag>(z + p.q_off + i * VEC, f);
      load_vec_row<Tag>((const T *)p.q_norm_w + i * VEC, w);
#pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] = f[j] * rq * w[j];
      store_vec_row<Tag>((T *)p.q_out + (int64_t)row * p.q_out_stride + i * VEC, f);
      continue;
    }
    int at = (i - nq) * VEC;
    if (i < nq + nk) {
      load_vec_row<Tag>(z + p.kv_off + at, f);
      load_vec_row<Tag>((const T *)p.kv_norm_w + at, w);
#pragma unroll
      for (int j = 0; j < VEC; ++j) f[j] = f[j] * rk * w[j];
    } else {
      const int c = (i - nq - nk) * VEC;
      load_vec_row<Tag>(z + p.rot_off + c, f);
      rotate_cols<VEC>(f, p.cos, p.sin, pos, pos_ok, c, p.rot_dim >> 1);
      at = p.kv_cols + c;
    }
    if (dst) store_vec_row<Tag>(dst + at, f);
    if (rows) store_vec_row<Tag>(rows + at, f);
  }
}

// rotated part of tokens t0 .. end - 1 of one head: out[t, h, n ..] = rotation of x[t, h, k ..]
template <typename Tag>
__device__ __forceinline__ void head_rotation(const MvHeadLinearArgs &p, int head, int t0, int end) {
  typedef typename elem<Tag>::T T;
  constexpr int VEC = elem<Tag>::VEC;
  const int per = p.rot_cols / VEC;
  for (int i = threadIdx.x; i < (end - t0) * per; i += 256) {
    const int t = t0 + i / per, c = i % per * VEC;
    float f[VEC];
    load_vec_row<Tag>((const T *)p.x + t * p.x_tok + head * p.x_head + p.k + c, f);
    const int64_t pos = p.positions[t];
    rotate_cols<VEC>(f, p.cos, p.sin, pos, pos >= 0 && pos < p.max_pos, c, p.rot_dim >> 1);
    store_vec_row<Tag>((T *)p.out + t * p.out_tok + head * p.out_head + p.n + c, f);
  }
}

// 16 TT tokens x 64 outputs of one head per workgroup: wave w computes outputs 16 w .. 16 w + 15.  Both operands come straight
// from memory in fragment order (a lane's 8 consecutive k), W rows as A, token rows as B; the loads of the next 128 k are in
// flight while the current ones are multiplied.
template <typename Tag, int TT>
__global__ void __launch_bounds__(256) head_linear_mfma_kernel(MvHeadLinearArgs p, int n_tiles, int n_tok) {
  typedef typename elem<Tag>::T T;
  const int head = blockIdx.y, t0 = blockIdx.z * (16 * TT);
  if ((int)blockIdx.x == n_tiles) return head_rotation<Tag>(p, head, t0, min(n_tok, t0 + 16 * TT));
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r16 = lane & 15, g = lane >> 4;
  const int n0 = (int)blockIdx.x * 64 + wave * 16;
  if (n0 >= p.n) return;
  const T *w = (const T *)p.w + ((int64_t)head * p.n + n0 + r16) * p.k + g * 8;
  const T *x[TT];
#pragma unroll
  for (int b = 0; b < TT; ++b)
    x[b] = (const T *)p.x + (int64_t)min(t0 + b * 16 + r16, n_tok - 1) * p.x_tok + head * p.x_head + g * 8;
  u32x4 wa[2][4], xa[2][TT][4];
  auto load = [&](int set, int k0) {   // (steps behind the end: weights of zero, x of the last step)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int k = min(k0 + 32 * i, p.k - 32);
      wa[set][i] = *(const u32x4 *)(w + k);
      if (k0 + 32 * i >= p.k) wa[set][i] = u32x4{0u, 0u, 0u, 0u};
#pragma unroll
      for (int b = 0; b < TT; ++b) xa[set][b][i] = *(const u32x4 *)(x[b] + k);
    }
  };
  f32x4 acc[TT] = {};
  auto multiply = [&](int set) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int b = 0; b < TT; ++b) acc[b] = mfma16x16x32<Tag>(wa[set][i], xa[set][b][i], acc[b]);
  };
  load(0, 0);
  for (int k = 0; k < p.k; k += 256) {
    if (k + 128 < p.k) load(1, k + 128);
    multiply(0);
    if (k + 256 < p.k) load(0, k + 256);
    if (k + 128 < p.k) multiply(1);
  }
#pragma unroll
  for (int b = 0; b < TT; ++b) {
    const int t = t0 + b * 16 + r16;
    if (t < n_tok) *(u32x2 *)((T *)p.out + (int64_t)t * p.out_tok + head * p.out_head + n0 + g * 4) = pack_quad<Tag>(acc[b]);
  }
}

// one output per thread, fp32
__global__ void __launch_bounds__(256) head_linear_f32_kernel(MvHeadLinearArgs p, int n_tiles, int n_tok) {
  const int head = blockIdx.y, t0 = blockIdx.z * 64;
  if ((int)blockIdx.x == n_tiles) return head_rotation<f32_tag>(p, head, t0, min(n_tok, t0 + 64));
  for (int i = threadIdx.x; i < 64 * 64; i += 256) {
    const int t = t0 + i / 64, n = (int)blockIdx.x * 64 + i % 64;
    if (t >= n_tok || n >= p.n) continue;
    const float *w = (const float *)p.w + ((int64_t)head * p.n + n) * p.k;
    const float *x = (const float *)p.x + (int64_t)t * p.x_tok + head * p.x_head;
    float s = 0.f;
    for (int k = 0; k < p.k; k += 4) {
      const f32x4 a = *(const f32x4 *)(w + k), b = *(const f32x4 *)(x + k);
#pragma unroll
      for (int j = 0; j < 4; ++j) s = fmaf(a[j], b[j], s);
    }
    ((float *)p.out)[(int64_t)t * p.out_tok + head * p.out_head + n] = s;
  }
}

// rows of cols16 16-byte pieces
__global__ void __launch_bounds__(256) latent_gather_kernel(const u32x4 *plane, int64_t num_blocks, int block_size, int cols16,
                                                            const int32_t *tables, int64_t table_stride, int table_width,
                                                            const int32_t *cu, const int32_t *start, u32x4 *out) {
  const int s = blockIdx.y, lo = cu[s], n = cu[s + 1] - lo, first = start[s];
  for (int i = blockIdx.x * 256 + threadIdx.x; i < n * cols16; i += gridDim.x * 256) {
    const int row = i / cols16, c = i - row * cols16, pos = first + row, b = pos / block_size;
    const int blk = b < table_width ? tables[s * table_stride + b] : -1;
    u32x4 v = {0u, 0u, 0u, 0u};
    if (blk >= 0 && blk < num_blocks) v = plane[((int64_t)blk * block_size + pos - b * block_size) * cols16 + c];
    out[(int64_t)(lo + row) * cols16 + c] = v;
  }
}

}  // namespace

extern "C" int mv_latent_prep(const MvLatentPrepArgs *a, int n_tok, int dtype, void *stream) {
  if (n_tok == 0) return MV_OK;
  if (!a || !a->z || !a->q_out || !a->q_norm_w) return MV_E_NULLPTR;
  if (n_tok < 0 || a->q_rank <= 0 || a->q_cols < a->q_rank || (a->q_cols & 31) || a->q_off < 0 ||
      a->q_off + a->q_cols > a->z_stride || a->q_out_stride < a->q_cols || (a->q_off & 7) || a->kv_rank < 0)
    return MV_E_SHAPE;
  if (a->kv_rank) {
    if (!a->kv_norm_w || !a->positions || !a->cos || !a->sin) return MV_E_NULLPTR;
    if (a->kv_cols < a->kv_rank || (a->kv_cols & 31) || a->rot_dim <= 0 || (a->rot_dim & 1) || a->rot_cols < a->rot_dim ||
        (a->rot_cols & 31) || a->kv_off < 0 || a->kv_off + a->kv_cols > a->z_stride || a->rot_off < 0 ||
        a->rot_off + a->rot_cols > a->z_stride || (a->kv_off & 7) || (a->rot_off & 7) || a->max_pos <= 0)
      return MV_E_SHAPE;
    if (a->plane && (!a->slot_mapping || a->num_slots <= 0)) return MV_E_NULLPTR;
  }
  const int vec = dtype == MV_F32 ? 4 : 8;
  if (!mv_aligned16(a->z) || a->z_stride % vec || !mv_aligned16(a->q_out) || a->q_out_stride % vec || !mv_aligned16(a->q_norm_w) ||
      (a->kv_rank && !mv_aligned16(a->kv_norm_w)) || (a->plane && !mv_aligned16(a->plane)) ||
      (a->rows_out && !mv_aligned16(a->rows_out)))
    return MV_E_ALIGN;
  MV_DISPATCH_DTYPE(dtype, hipLaunchKernelGGL((latent_prep_kernel<Tag>), dim3(n_tok), dim3(256), 0, (hipStream_t)stream, *a));
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_head_linear(const MvHeadLinearArgs *a, int n_tok, int dtype, void *stream) {
  if (n_tok == 0) return MV_OK;
  if (!a || !a->x || !a->w || !a->out) return MV_E_NULLPTR;
  if (n_tok < 0 || a->heads <= 0 || a->heads > 65535 || a->n <= 0 || (a->n & 15) || a->k <= 0 || (a->k & 31) || a->rot_dim < 0 ||
      (a->rot_dim & 1))
    return MV_E_SHAPE;
  if (a->rot_dim) {
    if (!a->positions || !a->cos || !a->sin) return MV_E_NULLPTR;
    if (a->rot_cols < a->rot_dim || (a->rot_cols & 7) || a->max_pos <= 0) return MV_E_SHAPE;
  }
  const int vec = dtype == MV_F32 ? 4 : 8;
  if (!mv_aligned16(a->x) || !mv_aligned16(a->w) || !mv_aligned16(a->out) || a->x_tok % vec || a->x_head % vec ||
      a->out_tok % vec || a->out_head % vec)
    return MV_E_ALIGN;
  const int n_tiles = (a->n + 63) / 64, x = n_tiles + (a->rot_dim ? 1 : 0);
  // token tiles per workgroup: a tile of weights is read once per workgroup, but the chip should be full
  int tt = 4;
  while (dtype != MV_F32 && tt > 1 && (n_tok <= 8 * tt || (int64_t)x * a->heads * ((n_tok + 16 * tt - 1) / (16 * tt)) < 512)) tt /= 2;
  const int z = (n_tok + 16 * tt - 1) / (16 * tt);
  if (z > 65535) return MV_E_SHAPE;
  const dim3 grid(x, a->heads, z), block(256);
  hipStream_t st = (hipStream_t)stream;
#define MV_HL(TAG)                                                                                                       \
  do {                                                                                                                   \
    if (tt == 4) hipLaunchKernelGGL((head_linear_mfma_kernel<TAG, 4>), grid, block, 0, st, *a, n_tiles, n_tok);          \
    else if (tt == 2) hipLaunchKernelGGL((head_linear_mfma_kernel<TAG, 2>), grid, block, 0, st, *a, n_tiles, n_tok);     \
    else hipLaunchKernelGGL((head_linear_mfma_kernel<TAG, 1>), grid, block, 0, st, *a, n_tiles, n_tok);                  \
  } while (0)
  if (dtype == MV_BF16) MV_HL(bf16_tag);
  else if (dtype == MV_F16) MV_HL(f16_tag);
  else if (dtype == MV_F32) hipLaunchKernelGGL(head_linear_f32_kernel, grid, block, 0, st, *a, n_tiles, n_tok);
  else return MV_E_DTYPE;
#undef MV_HL
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_latent_gather(const void *plane, int64_t num_blocks, int block_size, int cols, const int32_t *block_tables,
                                int64_t table_stride, int table_width, const int32_t *cu, const int32_t *start, int n_seqs,
                                int max_len, void *out, int dtype, void *stream) {
  if (n_seqs == 0 || max_len == 0) return MV_OK;
  if (!plane || !block_tables || !cu || !start || !out) return MV_E_NULLPTR;
  if (dtype != MV_BF16 && dtype != MV_F16 && dtype != MV_F32) return MV_E_DTYPE;
  if (n_seqs < 0 || n_seqs > 65535 || max_len < 0 || num_blocks <= 0 || block_size <= 0 || cols <= 0 || (cols & 31) ||
      table_width < 0)
    return MV_E_SHAPE;
  if (!mv_aligned16(plane) || !mv_aligned16(out)) return MV_E_ALIGN;
  const int cols16 = cols * (dtype == MV_F32 ? 4 : 2) / 16;
  const int64_t want = ((int64_t)max_len * cols16 + 255) / 256;
  if ((int64_t)max_len * cols16 > (1ll << 30)) return MV_E_SHAPE;
  hipLaunchKernelGGL(latent_gather_kernel, dim3((unsigned)(want < 2048 ? want : 2048), n_seqs), dim3(256), 0, (hipStream_t)stream,
                     (const u32x4 *)plane, num_blocks, block_size, cols16, block_tables, table_stride, table_width, cu, start,
                     (u32x4 *)out);
  MV_LAUNCH_CHECK();
  return MV_OK;
}
