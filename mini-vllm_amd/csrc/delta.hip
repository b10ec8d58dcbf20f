// K16 — gated delta rule (include/mvhip.h): recurrence over [n][p] states with a decay per head or per key channel.
//   prefill: mv_causal_conv (ssm.hip) over the projected channels, then mv_delta_prefill (token by token here; in chunks on the
//            matrix cores in delta_chunk.hip), then mv_head_norm_gate;
//   decode:  mv_delta_step, all of it for one token per sequence in one launch: the state streams through once.
// Everything but the projections and the convolution is fp32.
#include "delta.h"

namespace {

template <typename Tag>
__device__ __forceinline__ float param(const void *p, int64_t i) { return elem<Tag>::ld(((const typename elem<Tag>::T *)p)[i]); }

constexpr int kMaxTaps = 8, kMaxN16 = 32;   // n <= 512

// ---- recurrence, token by token.  One workgroup: 16 columns of one head; thread = (state rows l, l + 16, ..., column col): the
// 16 lanes of a DPP row share a column.  kScanRows tokens' operands are staged in LDS at a time.
constexpr int kScanRows = 8;

template <typename Tag>
__global__ void __launch_bounds__(256) delta_scan_kernel(MvDeltaArgs p) {
  typedef typename elem<Tag>::T T;
  extern __shared__ float lds[];   // unit k [rows][n] | unit q [rows][n] | decay [rows][n] | v [rows][16] | beta [rows]
  const int slice = blockIdx.x, head = blockIdx.y, s = blockIdx.z, tid = threadIdx.x, l = tid & 15, col = tid >> 4;
  const int q0 = p.cu_q[s], len = p.cu_q[s + 1] - q0;
  if (len <= 0) return;
  const int before = p.cu_k[s + 1] - p.cu_k[s] - len, slot = p.state_slots[s], n16 = p.n / 16;
  const bool keep = slot >= 0 && slot < p.slots;
  const int64_t size = (int64_t)p.heads * p.n * p.p, at = (int64_t)(keep ? slot : 0) * size + (int64_t)head * p.n * p.p + slice * 16 + col;
  float st[kMaxN16];
#pragma unroll
  for (int k = 0; k < kMaxN16; ++k) {
    st[k] = 0.f;
    if (k < n16 && keep && before > 0) st[k] = p.state[(before & 1) * p.slots * size + at + (int64_t)(l + 16 * k) * p.p];
  }
  const int g = head / (p.heads / p.groups);
  float *ks = lds, *qs = ks + kScanRows * p.n, *dec = qs + kScanRows * p.n, *vs = dec + kScanRows * p.n, *bs = vs + kScanRows * 16;
  const float rate = expf(param<Tag>(p.a_log, head));
  const T *x = (const T *)p.x + (int64_t)q0 * p.x_stride, *a = (const T *)p.a + (int64_t)q0 * p.a_stride;
  for (int t0 = 0; t0 < len; t0 += kScanRows) {
    const int nt = min(kScanRows, len - t0);
    __syncthreads();
    if ((col & 7) < nt) {   // a DPP row per (token, k or q): unit vectors
      const int t = col & 7;
      const bool isq = col >= 8;
      const T *row = x + (int64_t)(t0 + t) * p.x_stride + (isq ? p.q_off : p.k_off) + g * p.n;
      float ss = 0.f;
      for (int k = 0; k < n16; ++k) {
        const float f = elem<Tag>::ld(row[l + 16 * k]);
        ss = fmaf(f, f, ss);
      }
      const float f = (isq ? p.q_scale : 1.f) / sqrtf(row16_sum(ss) + p.unit_eps);
      for (int k = 0; k < n16; ++k) (isq ? qs : ks)[t * p.n + l + 16 * k] = elem<Tag>::ld(row[l + 16 * k]) * f;
    }
    for (int i = tid; i < nt * p.n; i += 256) {
      const int t = i / p.n, j = p.channel_decay ? head * p.n + i - t * p.n : head;
      dec[i] = expf(decay_log(rate, elem<Tag>::ld(a[(int64_t)(t0 + t) * p.a_stride + j]), param<Tag>(p.dt_bias, j)));
    }
    if (tid < nt * 16) vs[tid] = elem<Tag>::ld(x[(int64_t)(t0 + (tid >> 4)) * p.x_stride + head * p.p + slice * 16 + (tid & 15)]);
    if (tid < nt) bs[tid] = sigmoid_f32(elem<Tag>::ld(((const T *)p.beta)[(int64_t)(q0 + t0 + tid) * p.beta_stride + head]));
    __syncthreads();
    for (int t = 0; t < nt; ++t) {
      const float *kt = ks + t * p.n + l, *qt = qs + t * p.n + l, *dt = dec + t * p.n + l;
      float seen = 0.f, y = 0.f;
#pragma unroll
      for (int k = 0; k < kMaxN16; ++k)
        if (k < n16) {
          st[k] *= dt[16 * k];
          seen = fmaf(st[k], kt[16 * k], seen);
        }
      const float u = bs[t] * (vs[t * 16 + col] - row16_sum(seen));
#pragma unroll
      for (int k = 0; k < kMaxN16; ++k)
        if (k < n16) {
          st[k] = fmaf(kt[16 * k], u, st[k]);
          y = fmaf(st[k], qt[16 * k], y);
        }
      y = row16_sum(y);
      if (l == 0) ((T *)p.out)[(int64_t)(q0 + t0 + t) * p.out_stride + head * p.p + slice * 16 + col] = elem<Tag>::st(y);
    }
  }
  if (keep) {
    float *ns = p.state + ((before + len) & 1) * p.slots * size + at;
#pragma unroll
    for (int k = 0; k < kMaxN16; ++k)
      if (k < n16) ns[(int64_t)(l + 16 * k) * p.p] = st[k];
  }
}

// ---- one token: workgroup = (head, sequence).  The state [n][p] is requested first (up to kStepAhead 16-byte pieces per thread)
// and stays in registers; under that, the convolution of the head's v and of its group's k and q.  With S the decayed state,
//     u = beta (v - k S),   o = q S + (k . q) u,   S += k outer u            (vectors are rows)
// so both reductions over the rows of S happen in one pass.  k and q enter as they are, their lengths as factors of the sums.
constexpr int kStepAhead = 16;

template <typename Tag, int THREADS>
__global__ void __launch_bounds__(THREADS) delta_step_kernel(MvDeltaArgs p) {
  typedef typename elem<Tag>::T T;
  extern __shared__ float lds[];   // v [p] | k [n] | q [n] | decay [n] | u [p] | o [p] | partial k S, q S [rows][p] each
  __shared__ float sums[3];        // |k|^2, |q|^2, k . q
  const int head = blockIdx.x, s = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int before = p.context_lens[s] - 1, slot = p.state_slots[s], back = p.taps - 1;
  const int per = p.heads / p.groups, g = head / per;
  T *out = (T *)p.out + (int64_t)s * p.out_stride + head * p.p;
  if (before < 0) {
    for (int c = tid; c < p.p; c += THREADS) out[c] = elem<Tag>::st(0.f);
    return;
  }
  const bool keep = slot >= 0 && slot < p.slots, have = keep && before > 0;
  const int64_t size = (int64_t)p.heads * p.n * p.p, at = (int64_t)(keep ? slot : 0) * size + (int64_t)head * p.n * p.p;
  const f32x4 *os = (const f32x4 *)(p.state + (before & 1) * p.slots * size + at);
  f32x4 *ns = (f32x4 *)(p.state + ((before + 1) & 1) * p.slots * size + at);
  const int p4 = p.p / 4, rows = THREADS / p4;   // threads across a state row; state rows per trip
  const int c4 = tid % p4, r0 = tid / p4;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  f32x4 v[kStepAhead];
#pragma unroll
  for (int i = 0; i < kStepAhead; ++i) {
    const int r = r0 + i * rows;
    v[i] = have && r0 < rows && r < p.n ? __builtin_nontemporal_load(os + r * p4 + c4) : zero;
  }
  const int64_t chalf = p.slots * back * p.channels, cbase = (int64_t)(keep ? slot : 0) * back * p.channels;
  const T *x = (const T *)p.x + (int64_t)s * p.x_stride, *w = (const T *)p.conv_w;
  const T *oc = (const T *)p.conv_state + (before & 1) * chalf + cbase;
  T *nc = (T *)p.conv_state + ((before + 1) & 1) * chalf + cbase;
  float *vs = lds, *ks = vs + p.p, *qs = ks + p.n, *dec = qs + p.n, *us = dec + p.n, *ys = us + p.p, *pk = ys + p.p, *pq = pk + rows * p.p;
  for (int i = tid; i < p.p + 2 * p.n; i += THREADS) {
    const int ch = i < p.p ? head * p.p + i : (i < p.p + p.n ? p.k_off + g * p.n + i - p.p : p.q_off + g * p.n + i - p.p - p.n);
    const bool owner = keep && (i < p.p || head == g * per);   // k and q of a group: kept once
    const T cur = x[ch];
    T raw[kMaxTaps - 1];
    float wt[kMaxTaps - 1];
#pragma unroll
    for (int j = 0; j < kMaxTaps - 1; ++j) {
      raw[j] = j < back && have ? oc[(int64_t)j * p.channels + ch] : elem<Tag>::st(0.f);
      wt[j] = j < back ? elem<Tag>::ld(w[(int64_t)j * p.channels + ch]) : 0.f;
    }
    float o = 0.f;
    const float wc = elem<Tag>::ld(w[(int64_t)back * p.channels + ch]);
#pragma unroll
    for (int j = 0; j < kMaxTaps - 1; ++j) {
      o = fmaf(elem<Tag>::ld(raw[j]), wt[j], o);
      if (owner && j > 0 && j < back) nc[(int64_t)(j - 1) * p.channels + ch] = raw[j];
    }
    if (owner && back > 0) nc[(int64_t)(back - 1) * p.channels + ch] = cur;
    o = fmaf(elem<Tag>::ld(cur), wc, o);
    lds[i] = elem<Tag>::ld(elem<Tag>::st(silu_of<Tag>(o)));   // (the rounding of the prefill's convolved rows)
  }
  {
    const float rate = expf(param<Tag>(p.a_log, head));
    const T *a = (const T *)p.a + (int64_t)s * p.a_stride;
    for (int i = tid; i < p.n; i += THREADS) {
      const int j = p.channel_decay ? head * p.n + i : head;
      dec[i] = expf(decay_log(rate, elem<Tag>::ld(a[j]), param<Tag>(p.dt_bias, j)));
    }
  }
  const float beta = sigmoid_f32(elem<Tag>::ld(((const T *)p.beta)[(int64_t)s * p.beta_stride + head]));
  __syncthreads();
  if (wave < 3) {
    const float *fa = wave == 1 ? qs : ks, *fb = wave == 0 ? ks : qs;
    float t = 0.f;
    for (int i = lane; i < p.n; i += 64) t = fmaf(fa[i], fb[i], t);
    t = wave_sum(t);
    if (lane == 0) sums[wave] = t;
  }
  if (r0 < rows) {
    f32x4 a = zero, b = zero;
    auto reduce = [&](f32x4 st, int r) {
      const float d = dec[r], k = ks[r], q = qs[r];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        st[j] *= d;
        a[j] = fmaf(st[j], k, a[j]);
        b[j] = fmaf(st[j], q, b[j]);
      }
      return st;
    };
#pragma unroll
    for (int i = 0; i < kStepAhead; ++i)
      if (r0 + i * rows < p.n) v[i] = reduce(v[i], r0 + i * rows);
    for (int r = r0 + kStepAhead * rows; r < p.n; r += rows) reduce(have ? os[r * p4 + c4] : zero, r);
    *(f32x4 *)(pk + r0 * p.p + 4 * c4) = a;
    *(f32x4 *)(pq + r0 * p.p + 4 * c4) = b;
  }
  __syncthreads();
  const float fk = 1.f / sqrtf(sums[0] + p.unit_eps), fq = p.q_scale / sqrtf(sums[1] + p.unit_eps), kq = sums[2] * fk * fq;
  for (int c = tid; c < p.p; c += THREADS) {
    float a = 0.f, b = 0.f;
    for (int r = 0; r < rows; ++r) a += pk[r * p.p + c], b += pq[r * p.p + c];
    const float u = beta * (vs[c] - a * fk);
    ys[c] = c < p.p_true ? fmaf(kq, u, b * fq) : 0.f;
    us[c] = u * fk;
  }
  __syncthreads();
  if (keep && r0 < rows) {
    const f32x4 u = *(const f32x4 *)(us + 4 * c4);
#pragma unroll
    for (int i = 0; i < kStepAhead; ++i) {
      const int r = r0 + i * rows;
      if (r < p.n) {
        const float k = ks[r];
#pragma unroll
        for (int j = 0; j < 4; ++j) v[i][j] = fmaf(k, u[j], v[i][j]);
        __builtin_nontemporal_store(v[i], ns + r * p4 + c4);
      }
    }
    for (int r = r0 + kStepAhead * rows; r < p.n; r += rows) {   // (states beyond the registers are read once more)
      f32x4 st = have ? os[r * p4 + c4] : zero;
      const float k = ks[r], d = dec[r];
#pragma unroll
      for (int j = 0; j < 4; ++j) st[j] = fmaf(k, u[j], st[j] * d);
      __builtin_nontemporal_store(st, ns + r * p4 + c4);
    }
  }
  if (wave == 0) {
    float ss = 0.f;
    for (int c = lane; c < p.p; c += 64) ss = fmaf(ys[c], ys[c], ss);
    const float rs = p.out_scale / sqrtf(wave_sum(ss) / (float)p.p_true + p.eps);
    const T *gate = (const T *)p.gate + (int64_t)s * p.gate_stride + head * p.p;
    for (int c = lane; c < p.p; c += 64) {
      const float z = elem<Tag>::ld(gate[c]);
      out[c] = elem<Tag>::st(ys[c] * rs * param<Tag>(p.norm_w, c) * (p.gate_kind == MV_GATE_SIGMOID ? sigmoid_f32(z) : silu_f32(z)));
    }
  }
}

// ---- rms over each head of y, a weight shared by the heads, act(gate): LPT lanes per (token, head), PER vectors per lane
template <typename Tag, int LPT, int PER>
__global__ void __launch_bounds__(256) head_norm_gate_kernel(const typename elem<Tag>::T *y, int64_t y_stride,
                                                             const typename elem<Tag>::T *z, int64_t z_stride,
                                                             const typename elem<Tag>::T *w, typename elem<Tag>::T *out,
                                                             int64_t out_stride, int64_t items, int heads, int p, int p_true,
                                                             float eps, int gate_kind, float out_scale) {
  constexpr int VEC = elem<Tag>::VEC;
  const int sub = threadIdx.x % LPT;
  const int64_t item = (int64_t)blockIdx.x * (256 / LPT) + threadIdx.x / LPT;
  const bool live = item < items;
  const int64_t row = live ? item / heads : 0;
  const int head = live ? (int)(item - row * heads) : 0;
  float f[PER][VEC], g[PER][VEC], ss = 0.f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (sub + i * LPT) * VEC;
#pragma unroll
    for (int j = 0; j < VEC; ++j) f[i][j] = g[i][j] = 0.f;
    if (live && c < p) {
      load_vec_row<Tag>(y + row * y_stride + head * p + c, f[i]);
      load_vec_row<Tag>(z + row * z_stride + head * p + c, g[i]);
    }
#pragma unroll
    for (int j = 0; j < VEC; ++j) {
      if (c + j >= p_true) f[i][j] = 0.f;
      ss = fmaf(f[i][j], f[i][j], ss);
    }
  }
#pragma unroll
  for (int off = 1; off < LPT; off <<= 1) ss += __shfl_xor(ss, off, 64);
  const float rs = out_scale / sqrtf(ss / (float)p_true + eps);
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = (sub + i * LPT) * VEC;
    if (live && c < p) {
      float wv[VEC], o[VEC];
      load_vec_row<Tag>(w + c, wv);
#pragma unroll
      for (int j = 0; j < VEC; ++j) {
        float act;
        if constexpr (__is_same(Tag, f32_tag)) act = gate_kind == MV_GATE_SIGMOID ? sigmoid_f32(g[i][j]) : silu_f32(g[i][j]);
        else act = (gate_kind == MV_GATE_SIGMOID ? 1.f : g[i][j]) * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * g[i][j]));
        o[j] = f[i][j] * rs * wv[j] * act;
      }
      store_vec_row<Tag>(out + row * out_stride + head * p + c, o);
    }
  }
}

int check_delta(const MvDeltaArgs *a, int dtype) {
  if (!a || !a->x || !a->out || !a->state_slots || !a->beta || !a->a || !a->dt_bias || !a->a_log || (a->slots > 0 && !a->state))
    return MV_E_NULLPTR;
  if (dtype != MV_BF16 && dtype != MV_F16 && dtype != MV_F32) return MV_E_DTYPE;
  if (a->n_seqs < 0 || a->n_seqs > 65535 || a->heads <= 0 || a->heads > 65535 || a->groups <= 0 || a->heads % a->groups || a->p <= 0 ||
      (a->p & 15) || a->p > 512 || a->n <= 0 || (a->n & 31) || a->n > 16 * kMaxN16 || a->slots < 0 || a->k_off < a->heads * a->p ||
      a->k_off + a->groups * a->n > a->channels || a->q_off < a->heads * a->p || a->q_off + a->groups * a->n > a->channels ||
      a->x_stride < a->channels || a->beta_stride < a->heads || a->a_stride < (int64_t)a->heads * (a->channel_decay ? a->n : 1) ||
      a->out_stride < (int64_t)a->heads * a->p)
    return MV_E_SHAPE;
  return (a->state && !mv_aligned16(a->state)) ? MV_E_ALIGN : MV_OK;
}

}  // namespace

extern "C" size_t mv_delta_prefill_workspace_bytes(int n_seqs, int total_q, int heads, int p, int n, int dtype) {
  return dtype == MV_F32 ? 0 : mv_delta_chunk_workspace(n_seqs, total_q, heads, p, n);
}

extern "C" int mv_delta_prefill(const MvDeltaArgs *a, int dtype, int flags, void *stream) {
  if (a && (a->n_seqs == 0 || a->max_q == 0)) return MV_OK;
  if (int e = check_delta(a, dtype)) return e;
  if (!a->cu_q || !a->cu_k) return MV_E_NULLPTR;
  if (a->max_q < 0) return MV_E_SHAPE;
  if (dtype != MV_F32 && !(flags & MV_DELTA_SCAN)) {
    const int rc = mv_delta_chunk_launch(*a, dtype, (hipStream_t)stream);
    if (rc != MV_E_SHAPE) return rc;
  }
  const size_t lds = (size_t)(3 * kScanRows * a->n + kScanRows * 17) * 4;
  const dim3 grid(a->p / 16, a->heads, a->n_seqs);
  MV_DISPATCH_DTYPE(dtype, hipLaunchKernelGGL((delta_scan_kernel<Tag>), grid, dim3(256), lds, (hipStream_t)stream, *a));
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_delta_step(const MvDeltaArgs *a, int dtype, void *stream) {
  if (a && a->n_seqs == 0) return MV_OK;
  if (int e = check_delta(a, dtype)) return e;
  if (!a->conv_w || !a->context_lens || !a->gate || !a->norm_w || (a->slots > 0 && a->taps > 1 && !a->conv_state)) return MV_E_NULLPTR;
  if (a->taps < 1 || a->taps > kMaxTaps || a->p_true <= 0 || a->p_true > a->p || a->gate_stride < (int64_t)a->heads * a->p) return MV_E_SHAPE;
  if (a->gate_kind != MV_GATE_SILU && a->gate_kind != MV_GATE_SIGMOID) return MV_E_RANGE;
  const int pieces = a->n * a->p / 4;
  // (few workgroups: latency decides, and eight waves a head are quicker through its dependent phases)
  const int threads = pieces > 512 * kStepAhead ? 1024 : pieces > 256 * kStepAhead || (int64_t)a->heads * a->n_seqs <= 512 ? 512 : 256;
  const size_t lds = (size_t)(3 * a->p + 3 * a->n + 2 * (threads / (a->p / 4)) * a->p) * 4;
  const dim3 grid(a->heads, a->n_seqs);
  MV_DISPATCH_DTYPE(dtype, {
    if (threads == 256) hipLaunchKernelGGL((delta_step_kernel<Tag, 256>), grid, dim3(256), lds, (hipStream_t)stream, *a);
    else if (threads == 512) hipLaunchKernelGGL((delta_step_kernel<Tag, 512>), grid, dim3(512), lds, (hipStream_t)stream, *a);
    else hipLaunchKernelGGL((delta_step_kernel<Tag, 1024>), grid, dim3(1024), lds, (hipStream_t)stream, *a);
  });
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_head_norm_gate(const void *y, int64_t y_stride, const void *gate, int64_t gate_stride, const void *w, void *out,
                                 int64_t out_stride, int rows, int heads, int p, int p_true, float eps, int gate_kind, float out_scale,
                                 int dtype, void *stream) {
  if (rows == 0) return MV_OK;
  if (!y || !gate || !w || !out) return MV_E_NULLPTR;
  if (rows < 0 || heads <= 0 || p_true <= 0 || p < p_true || (p & 7) || p > 1024 || y_stride < (int64_t)heads * p ||
      gate_stride < (int64_t)heads * p || out_stride < (int64_t)heads * p)
    return MV_E_SHAPE;
  if (gate_kind != MV_GATE_SILU && gate_kind != MV_GATE_SIGMOID) return MV_E_RANGE;
  const int vec = dtype == MV_F32 ? 4 : 8;
  if (!mv_aligned16(y) || !mv_aligned16(gate) || !mv_aligned16(w) || !mv_aligned16(out) || y_stride % vec || gate_stride % vec ||
      out_stride % vec)
    return MV_E_ALIGN;
  const int64_t items = (int64_t)rows * heads;
  const int vecs = p / vec;
#define MV_HN(LPT, PER)                                                                                                          \
  hipLaunchKernelGGL((head_norm_gate_kernel<Tag, LPT, PER>), dim3((unsigned)((items + 256 / LPT - 1) / (256 / LPT))), dim3(256), 0, \
                     (hipStream_t)stream, (const T *)y, y_stride, (const T *)gate, gate_stride, (const T *)w, (T *)out, out_stride,  \
                     items, heads, p, p_true, eps, gate_kind, out_scale)
  MV_DISPATCH_DTYPE(dtype, {
    typedef typename elem<Tag>::T T;
    if (vecs <= 4) MV_HN(4, 1);
    else if (vecs <= 8) MV_HN(8, 1);
    else if (vecs <= 16) MV_HN(16, 1);
    else if (vecs <= 32) MV_HN(32, 1);
    else if (vecs <= 64) MV_HN(64, 1);
    else MV_HN(64, 4);
  });
#undef MV_HN
  MV_LAUNCH_CHECK();
  return MV_OK;
}
