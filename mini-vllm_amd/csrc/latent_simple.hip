// K14 — latent attention on the vector ALUs (every dtype and size; fp32 models run on it), and the C entry points of both
// attention forms, which pick the matrix-core kernels for 16-bit tensors.
// One workgroup = one (query row, head): 256 keys at a time, a score per thread, online softmax, then a column of the output
// per thread.
#include "latent.h"

namespace {

constexpr int kKeys = 256, kMaxCols = 2048;   // keys per round; columns of a query row (LDS)

__device__ __forceinline__ float block_reduce(float x, float *red, bool maximum) {
  x = maximum ? wave_max(x) : wave_sum(x);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = x;
  __syncthreads();
  return maximum ? fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])) : (red[0] + red[1]) + (red[2] + red[3]);
}

// row(key) -> index of the key's row, or -1; dot(row) -> raw score; value(row, col) -> fp32
template <typename Row, typename Dot, typename Value, typename Store>
__device__ __forceinline__ void attend(int lo, int hi, int cols, float scale, Row row, Dot dot, Value value, Store store) {
  __shared__ float prob[kKeys], red[4], o[kMaxCols];
  __shared__ int rows[kKeys];
  float m = -INFINITY, l = 0.f;
  for (int c = threadIdx.x; c < cols; c += 256) o[c] = 0.f;
  for (int k0 = lo; k0 < hi; k0 += kKeys) {
    const int key = k0 + threadIdx.x;
    const int r = key < hi ? row(key) : -1;
    const float s = r >= 0 ? dot(r) * scale : -INFINITY;
    const float m_new = fmaxf(m, block_reduce(s, red, true));
    const float p = s == -INFINITY ? 0.f : expf(s - m_new);
    const float alpha = m == -INFINITY ? 0.f : expf(m - m_new);
    l = l * alpha + block_reduce(p, red, false);
    m = m_new;
    prob[threadIdx.x] = p;
    rows[threadIdx.x] = r;
    __syncthreads();
    const int n = min(kKeys, hi - k0);
    for (int c = threadIdx.x; c < cols; c += 256) {
      float acc = o[c] * alpha;
      for (int j = 0; j < n; ++j)
        if (rows[j] >= 0) acc = fmaf(prob[j], value(rows[j], c), acc);
      o[c] = acc;
    }
    __syncthreads();
  }
  for (int c = threadIdx.x; c < cols; c += 256) store(c, l > 0.f ? o[c] / l : 0.f);
}

template <typename Tag>
__device__ __forceinline__ float dot_row(const float *q, const typename elem<Tag>::T *k, int n) {
  constexpr int VEC = elem<Tag>::VEC;
  float s = 0.f;
  for (int c = 0; c < n; c += VEC) {
    float f[VEC];
    load_vec_row<Tag>(k + c, f);
#pragma unroll
    for (int j = 0; j < VEC; ++j) s = fmaf(q[c + j], f[j], s);
  }
  return s;
}

template <typename Tag>
__global__ void __launch_bounds__(256) latent_decode_simple_kernel(const void *q_, const void *plane_, const int32_t *tables,
                                                                   int64_t table_stride, const int32_t *lens, void *out_,
                                                                   int heads, int kv_cols, int cols, int block_size,
                                                                   int max_blocks, int64_t num_blocks, int window, float scale) {
  typedef typename elem<Tag>::T T;
  __shared__ float q[kMaxCols];
  const int head = blockIdx.x, b = blockIdx.y;
  const T *qp = (const T *)q_ + ((int64_t)b * heads + head) * cols, *plane = (const T *)plane_;
  for (int c = threadIdx.x; c < cols; c += 256) q[c] = elem<Tag>::ld(qp[c]);
  __syncthreads();
  const int len = min(lens[b], max_blocks * block_size), lo = window > 0 && len > window ? len - window : 0;
  T *out = (T *)out_ + ((int64_t)b * heads + head) * kv_cols;
  attend(lo, len, kv_cols, scale,
         [&](int key) {
           const int blk = tables[b * table_stride + key / block_size];
           return blk >= 0 && blk < num_blocks ? blk * block_size + key % block_size : -1;
         },
         [&](int r) { return dot_row<Tag>(q, plane + (int64_t)r * cols, cols); },
         [&](int r, int c) { return elem<Tag>::ld(plane[(int64_t)r * cols + c]); },
         [&](int c, float v) { out[c] = elem<Tag>::st(v); });
}

template <typename Tag>
__global__ void __launch_bounds__(256) latent_prefill_simple_kernel(MvLatentPrefillArgs p) {
  typedef typename elem<Tag>::T T;
  __shared__ float q[kMaxCols];
  const int head = blockIdx.x, s = blockIdx.z;
  const int q0 = p.cu_q[s], sq = p.cu_q[s + 1] - q0, k0 = p.cu_k[s], sk = p.cu_k[s + 1] - k0;
  for (int i = blockIdx.y; i < sq; i += gridDim.y) {
    __syncthreads();
    const T *qp = (const T *)p.q + (int64_t)(q0 + i) * p.q_stride + head * p.dq;
    const int64_t pos = p.positions[q0 + i];
    const bool pos_ok = pos >= 0 && pos < p.max_pos;
    for (int c = threadIdx.x; c < p.plain_cols; c += 256) q[c] = elem<Tag>::ld(qp[c]);
    for (int c = threadIdx.x; c < p.rot_cols; c += 256) {
      const int pair = c >> 1, pairs = p.rot_dim >> 1;
      float r = 0.f;
      if (pair < pairs) {
        const float u = elem<Tag>::ld(qp[p.plain_cols + 2 * pair]), v = elem<Tag>::ld(qp[p.plain_cols + 2 * pair + 1]);
        const float cs = pos_ok ? p.cos[pos * pairs + pair] : 1.0f, sn = pos_ok ? p.sin[pos * pairs + pair] : 0.0f;
        r = (c & 1) ? __fadd_rn(__fmul_rn(v, cs), __fmul_rn(u, sn)) : __fsub_rn(__fmul_rn(u, cs), __fmul_rn(v, sn));
      }
      q[p.plain_cols + c] = elem<Tag>::ld(elem<Tag>::st(r));
    }
    __syncthreads();
    const int hi = min(sk, i + sk - sq + 1), lo = p.window > 0 && hi > p.window ? hi - p.window : 0;
    const T *kp = (const T *)p.k + (int64_t)k0 * p.k_stride + head * p.plain_cols;
    const T *vp = (const T *)p.v + (int64_t)k0 * p.v_stride + head * p.dv;
    const T *rp = (const T *)p.rot + (int64_t)k0 * p.rot_stride;
    T *out = (T *)p.out + (int64_t)(q0 + i) * p.out_stride + head * p.dv;
    attend(lo, hi, p.dv, p.scale, [&](int key) { return key; },
           [&](int r) {
             return dot_row<Tag>(q, kp + r * p.k_stride, p.plain_cols) + dot_row<Tag>(q + p.plain_cols, rp + r * p.rot_stride, p.rot_cols);
           },
           [&](int r, int c) { return elem<Tag>::ld(vp[r * p.v_stride + c]); },
           [&](int c, float v) { out[c] = elem<Tag>::st(v); });
  }
}

}  // namespace

int mv_latent_decode_simple_launch(const void *q, const void *plane, const int32_t *tables, int64_t table_stride,
                                   const int32_t *lens, void *out, int batch, int heads, int kv_cols, int rot_cols,
                                   int block_size, int max_blocks, int64_t num_blocks, int window, float scale, int dtype,
                                   hipStream_t stream) {
  if (kv_cols + rot_cols > kMaxCols || batch > 65535) return MV_E_SHAPE;
  MV_DISPATCH_DTYPE(dtype, hipLaunchKernelGGL((latent_decode_simple_kernel<Tag>), dim3(heads, batch), dim3(256), 0, stream, q,
                                              plane, tables, table_stride, lens, out, heads, kv_cols, kv_cols + rot_cols,
                                              block_size, max_blocks, num_blocks, window, scale));
  MV_LAUNCH_CHECK();
  return MV_OK;
}

int mv_latent_prefill_simple_launch(const MvLatentPrefillArgs &a, int dtype, hipStream_t stream) {
  if (a.plain_cols + a.rot_cols > kMaxCols || a.dv > kMaxCols || a.n_seqs > 65535) return MV_E_SHAPE;
  const int rows = a.max_q < 65535 ? a.max_q : 65535;
  MV_DISPATCH_DTYPE(dtype, hipLaunchKernelGGL((latent_prefill_simple_kernel<Tag>), dim3(a.heads, rows, a.n_seqs), dim3(256), 0,
                                              stream, a));
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" size_t mv_latent_decode_workspace_bytes(int batch, int heads, int kv_cols, int rot_cols, int block_size,
                                                   int max_blocks, int window, int dtype) {
  if (batch <= 0 || heads <= 0 || kv_cols <= 0 || block_size <= 0 || dtype == MV_F32) return 256;
  return mv_latent_decode_mfma_workspace(batch, heads, kv_cols, rot_cols, block_size, max_blocks, window);
}

extern "C" int mv_latent_decode(const void *q, const void *plane, const int32_t *block_tables, int64_t table_stride,
                                const int32_t *context_lens, void *out, int batch, int heads, int kv_cols, int rot_cols,
                                int block_size, int max_blocks, int64_t num_blocks, int window, float scale, void *workspace,
                                size_t workspace_bytes, int dtype, int flags, void *stream) {
  if (batch == 0) return MV_OK;
  if (!q || !plane || !context_lens || !out || (max_blocks > 0 && !block_tables)) return MV_E_NULLPTR;
  if (dtype != MV_BF16 && dtype != MV_F16 && dtype != MV_F32) return MV_E_DTYPE;
  if (batch < 0 || heads <= 0 || kv_cols <= 0 || (kv_cols & 31) || rot_cols < 0 || (rot_cols & 31) || block_size <= 0 ||
      max_blocks < 0 || num_blocks <= 0 || window < 0)
    return MV_E_SHAPE;
  if (num_blocks * block_size > 0x7fffffffll) return MV_E_SHAPE;
  if (!mv_aligned16(q) || !mv_aligned16(plane) || !mv_aligned16(out)) return MV_E_ALIGN;
  if (dtype != MV_F32 && !(flags & MV_LATENT_SIMPLE)) {
    const int rc = mv_latent_decode_mfma_launch(q, plane, block_tables, table_stride, context_lens, out, batch, heads, kv_cols,
                                                rot_cols, block_size, max_blocks, num_blocks, window, scale, workspace,
                                                workspace_bytes, dtype, (hipStream_t)stream);
    if (rc != MV_E_SHAPE) return rc;
  }
  return mv_latent_decode_simple_launch(q, plane, block_tables, table_stride, context_lens, out, batch, heads, kv_cols, rot_cols,
                                        block_size, max_blocks, num_blocks, window, scale, dtype, (hipStream_t)stream);
}

extern "C" int mv_latent_prefill(const MvLatentPrefillArgs *a, int dtype, int flags, void *stream) {
  if (!a) return MV_E_NULLPTR;
  if (a->n_seqs == 0 || a->max_q == 0) return MV_OK;
  if (!a->q || !a->k || !a->v || !a->rot || !a->out || !a->cu_q || !a->cu_k || !a->positions || !a->cos || !a->sin)
    return MV_E_NULLPTR;
  if (dtype != MV_BF16 && dtype != MV_F16 && dtype != MV_F32) return MV_E_DTYPE;
  if (a->n_seqs < 0 || a->max_q < 0 || a->max_k < 0 || a->heads <= 0 || a->plain_cols <= 0 || (a->plain_cols & 31) ||
      a->rot_dim <= 0 || (a->rot_dim & 1) || a->rot_cols < a->rot_dim || (a->rot_cols & 31) ||
      a->dq < a->plain_cols + a->rot_cols || (a->dq & 31) || a->dv <= 0 || (a->dv & 31) || a->window < 0 || a->max_pos <= 0 ||
      a->q_stride < (int64_t)a->heads * a->dq || a->out_stride < (int64_t)a->heads * a->dv)
    return MV_E_SHAPE;
  const int vec = dtype == MV_F32 ? 4 : 8;
  if (!mv_aligned16(a->q) || !mv_aligned16(a->k) || !mv_aligned16(a->v) || !mv_aligned16(a->rot) || !mv_aligned16(a->out) ||
      a->q_stride % vec || a->k_stride % vec || a->v_stride % vec || a->rot_stride % vec || a->out_stride % vec)
    return MV_E_ALIGN;
  if (dtype != MV_F32 && !(flags & MV_LATENT_SIMPLE)) {
    const int rc = mv_latent_prefill_mfma_launch(*a, dtype, (hipStream_t)stream);
    if (rc != MV_E_SHAPE) return rc;
  }
  return mv_latent_prefill_simple_launch(*a, dtype, (hipStream_t)stream);
}
