// K15 — selective state space layer (include/mvhip.h): causal convolution, recurrence, gated group norm.
//   prefill: mv_causal_conv over the projected rows, then the recurrence (mv_ssm_prefill: token by token here; in chunks on
//            the matrix cores in ssm_chunk.hip), one workgroup per (sequence, head, slice of columns);
//   decode:  mv_ssm_step, convolution + recurrence of one token per sequence in one launch: the state streams through once.
// Everything from the step size on is fp32.
#include "ssm.h"

namespace {

template <typename Tag>
__device__ __forceinline__ float param(const void *p, int i) { return elem<Tag>::ld(((const typename elem<Tag>::T *)p)[i]); }

// ---- convolution: 8 (fp32: 4) channels per thread, kConvRows tokens per workgroup, a sliding window of inputs in registers
constexpr int kConvRows = 32, kConvAhead = 8, kMaxTaps = 8;

template <typename Tag, int TAPS>
__global__ void __launch_bounds__(64) causal_conv_kernel(MvSsmArgs p) {
  typedef typename elem<Tag>::T T;
  constexpr int VEC = elem<Tag>::VEC;
  const int c = ((int)blockIdx.x * 64 + threadIdx.x) * VEC, s = blockIdx.z;
  const int q0 = p.cu_q[s], len = p.cu_q[s + 1] - q0, t0 = blockIdx.y * kConvRows;
  if (t0 >= len || c >= p.channels) return;
  const int before = p.cu_k[s + 1] - p.cu_k[s] - len, slot = p.state_slots[s], back = p.taps - 1;
  const bool keep = slot >= 0 && slot < p.slots;
  const int64_t half = p.slots * back * p.channels;
  T *state = (T *)p.conv_state;
  const T *old_state = state + (before & 1) * half + (int64_t)(keep ? slot : 0) * back * p.channels + c;
  const T *x = (const T *)p.x + (int64_t)q0 * p.x_stride + c;
  // input `t` of the step (t < 0: of the steps before it)
  auto input = [&](int t, float (&f)[VEC]) {
    if (t >= 0) return load_vec_row<Tag>(x + (int64_t)t * p.x_stride, f);
    if (before > 0 && keep) return load_vec_row<Tag>(old_state + (int64_t)(back + t) * p.channels, f);
#pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] = 0.f;
  };
  // weights aligned at the current token: tap TAPS - 1 is its own
  float w[TAPS][VEC], bias[VEC], win[TAPS][VEC];
#pragma unroll
  for (int i = 0; i < TAPS; ++i)
#pragma unroll
    for (int j = 0; j < VEC; ++j) w[i][j] = win[i][j] = 0.f;
#pragma unroll
  for (int i = 0; i < TAPS; ++i) {
    const int tap = i - (TAPS - p.taps);
    if (tap >= 0) {
      load_vec_row<Tag>((const T *)p.conv_w + (int64_t)tap * p.channels + c, w[i]);
      if (i < TAPS - 1) input(t0 + i - (TAPS - 1), win[i + 1]);   // shifted down below
    }
  }
#pragma unroll
  for (int j = 0; j < VEC; ++j) bias[j] = 0.f;
  if (p.conv_b) load_vec_row<Tag>((const T *)p.conv_b + c, bias);
  if (t0 == 0 && keep && back > 0) {   // the only workgroup that reads the old state writes the new one, behind its reads
    float last[kMaxTaps - 1][VEC];
    for (int j = 0; j < kMaxTaps - 1; ++j)
      if (j < back) input(len - back + j, last[j]);
    T *ns = state + ((before + len) & 1) * half + (int64_t)slot * back * p.channels + c;
    for (int j = 0; j < kMaxTaps - 1; ++j)
      if (j < back) store_vec_row<Tag>(ns + (int64_t)j * p.channels, last[j]);
  }
  const int t1 = min(len, t0 + kConvRows);
  for (int tb = t0; tb < t1; tb += kConvAhead) {
    u32x4 raw[kConvAhead];
#pragma unroll
    for (int u = 0; u < kConvAhead; ++u) raw[u] = *(const u32x4 *)(x + (int64_t)min(tb + u, len - 1) * p.x_stride);
#pragma unroll
    for (int u = 0; u < kConvAhead; ++u) {
      float o[VEC];
#pragma unroll
      for (int i = 0; i < TAPS - 1; ++i)
#pragma unroll
        for (int j = 0; j < VEC; ++j) win[i][j] = win[i + 1][j];
      if constexpr (VEC == 8) {
        unpack8<Tag>(raw[u], win[TAPS - 1]);
      } else {
#pragma unroll
        for (int j = 0; j < VEC; ++j) win[TAPS - 1][j] = u2f(raw[u][j]);
      }
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = bias[j];
#pragma unroll
      for (int i = 0; i < TAPS; ++i)
#pragma unroll
        for (int j = 0; j < VEC; ++j) o[j] = fmaf(win[i][j], w[i][j], o[j]);
#pragma unroll
      for (int j = 0; j < VEC; ++j) o[j] = silu_of<Tag>(o[j]);
      if (tb + u < t1) store_vec_row<Tag>((T *)p.out + (int64_t)(q0 + tb + u) * p.out_stride + c, o);
    }
  }
}

// ---- recurrence, token by token.  One workgroup: 16 columns of one head; thread = (state rows l, l + 16, ..., column i):
// the 16 lanes of a DPP row share a column, so y is a row sum.  kScanRows tokens' operands are staged in LDS at a time.
constexpr int kScanRows = 16, kMaxN16 = 32;   // N <= 512

template <typename Tag>
__global__ void __launch_bounds__(256) ssm_scan_kernel(MvSsmArgs p) {
  typedef typename elem<Tag>::T T;
  extern __shared__ float lds[];   // b [rows][n] | c [rows][n] | x [rows][16] | decay [rows] | dt [rows]
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
    if (k < n16 && keep && before > 0) st[k] = p.ssm_state[(before & 1) * p.slots * size + at + (int64_t)(l + 16 * k) * p.p];
  }
  const int g = head / (p.heads / p.groups);
  float *bs = lds, *cs = bs + kScanRows * p.n, *xs = cs + kScanRows * p.n, *dec = xs + kScanRows * 16, *dts = dec + kScanRows;
  const float na = -expf(param<Tag>(p.a_log, head)), bias = param<Tag>(p.dt_bias, head), d = param<Tag>(p.d, head);
  const T *x = (const T *)p.x, *dt = (const T *)p.dt;
  for (int t0 = 0; t0 < len; t0 += kScanRows) {
    const int nt = min(kScanRows, len - t0);
    __syncthreads();
    for (int i = tid; i < nt * p.n; i += 256) {
      const int t = i / p.n, k = i - t * p.n;
      const T *row = x + (int64_t)(q0 + t0 + t) * p.x_stride;
      bs[i] = elem<Tag>::ld(row[p.b_off + g * p.n + k]);
      cs[i] = elem<Tag>::ld(row[p.c_off + g * p.n + k]);
    }
    if (tid < nt * 16) xs[tid] = elem<Tag>::ld(x[(int64_t)(q0 + t0 + (tid >> 4)) * p.x_stride + head * p.p + slice * 16 + (tid & 15)]);
    if (tid < nt) {
      const float step = softplus_f32(elem<Tag>::ld(dt[(int64_t)(q0 + t0 + tid) * p.dt_stride + head]) + bias);
      dts[tid] = step;
      dec[tid] = expf(na * step);
    }
    __syncthreads();
    for (int t = 0; t < nt; ++t) {
      const float a = dec[t], xv = xs[t * 16 + col], u = dts[t] * xv;
      float y = 0.f;
#pragma unroll
      for (int k = 0; k < kMaxN16; ++k)
        if (k < n16) {
          st[k] = fmaf(a, st[k], bs[t * p.n + l + 16 * k] * u);
          y = fmaf(st[k], cs[t * p.n + l + 16 * k], y);
        }
      y = row16_sum(y);
      if (l == 0) ((T *)p.out)[(int64_t)(q0 + t0 + t) * p.out_stride + head * p.p + slice * 16 + col] = elem<Tag>::st(fmaf(d, xv, y));
    }
  }
  if (keep) {
    float *ns = p.ssm_state + ((before + len) & 1) * p.slots * size + at;
#pragma unroll
    for (int k = 0; k < kMaxN16; ++k)
      if (k < n16) ns[(int64_t)(l + 16 * k) * p.p] = st[k];
  }
}

// ---- one token: workgroup = (head, sequence).  The state [n][p] is requested first (up to kStepAhead 16-byte pieces per
// thread); under that, the convolution of the head's columns and of its group's b and c (a few hundred channels); then each piece
// of state is updated, multiplied into y and written once.
constexpr int kStepAhead = 8;

template <typename Tag>
__global__ void __launch_bounds__(256) ssm_step_kernel(MvSsmArgs p) {
  typedef typename elem<Tag>::T T;
  extern __shared__ float lds[];   // x [p] | b [n] | c [n] | partial y [256 / (p / 4)][p]
  const int head = blockIdx.x, s = blockIdx.y, tid = threadIdx.x;
  const int before = p.context_lens[s] - 1, slot = p.state_slots[s], back = p.taps - 1;
  const int per = p.heads / p.groups, g = head / per;
  if (before < 0) {
    for (int c = tid; c < p.p; c += 256) ((T *)p.out)[(int64_t)s * p.out_stride + head * p.p + c] = elem<Tag>::st(0.f);
    return;
  }
  const bool keep = slot >= 0 && slot < p.slots, have = keep && before > 0;
  const int64_t size = (int64_t)p.heads * p.n * p.p, at = (int64_t)(keep ? slot : 0) * size + (int64_t)head * p.n * p.p;
  const f32x4 *os = (const f32x4 *)(p.ssm_state + (before & 1) * p.slots * size + at);
  f32x4 *ns = (f32x4 *)(p.ssm_state + ((before + 1) & 1) * p.slots * size + at);
  const int p4 = p.p / 4, rows = 256 / p4;   // threads across a state row; state rows per trip
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
  float *xs = lds, *bs = xs + p.p, *cs = bs + p.n, *ys = cs + p.n;
  for (int i = tid; i < p.p + 2 * p.n; i += 256) {
    const int ch = i < p.p ? head * p.p + i : (i < p.p + p.n ? p.b_off + g * p.n + i - p.p : p.c_off + g * p.n + i - p.p - p.n);
    const bool owner = keep && (i < p.p || head == g * per);   // b and c of a group: kept once
    const T cur = x[ch];
    T raw[kMaxTaps - 1];
    float wt[kMaxTaps - 1];
#pragma unroll
    for (int j = 0; j < kMaxTaps - 1; ++j) {
      raw[j] = j < back && have ? oc[(int64_t)j * p.channels + ch] : elem<Tag>::st(0.f);
      wt[j] = j < back ? elem<Tag>::ld(w[(int64_t)j * p.channels + ch]) : 0.f;
    }
    float o = param<Tag>(p.conv_b, ch);
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
  const float step = softplus_f32(elem<Tag>::ld(((const T *)p.dt)[(int64_t)s * p.dt_stride + head]) + param<Tag>(p.dt_bias, head));
  const float a = expf(-expf(param<Tag>(p.a_log, head)) * step), d = param<Tag>(p.d, head);
  __syncthreads();
  f32x4 y = zero;
  if (r0 < rows) {
    const f32x4 u = *(const f32x4 *)(xs + 4 * c4) * step;
    auto advance = [&](f32x4 st, int r) {
      const float b = bs[r], c = cs[r];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        st[j] = fmaf(a, st[j], b * u[j]);
        y[j] = fmaf(st[j], c, y[j]);
      }
      if (keep) __builtin_nontemporal_store(st, ns + r * p4 + c4);
    };
#pragma unroll
    for (int i = 0; i < kStepAhead; ++i)
      if (r0 + i * rows < p.n) advance(v[i], r0 + i * rows);
    for (int r = r0 + kStepAhead * rows; r < p.n; r += rows) advance(have ? os[r * p4 + c4] : zero, r);
    *(f32x4 *)(ys + r0 * p.p + 4 * c4) = y;
  }
  __syncthreads();
  for (int c = tid; c < p.p; c += 256) {
    float o = 0.f;
    for (int r = 0; r < rows; ++r) o += ys[r * p.p + c];
    ((T *)p.out)[(int64_t)s * p.out_stride + head * p.p + c] = elem<Tag>::st(fmaf(d, xs[c], o));
  }
}

// ---- rms over parts of y * silu(z): workgroup = (token, part)
template <typename Tag>
__global__ void __launch_bounds__(256) gated_group_norm_kernel(const typename elem<Tag>::T *y, int64_t y_stride,
                                                               const typename elem<Tag>::T *z, int64_t z_stride,
                                                               const typename elem<Tag>::T *w, typename elem<Tag>::T *out,
                                                               int64_t out_stride, int heads, int p, int p_true, int size,
                                                               float eps) {
  constexpr int VEC = elem<Tag>::VEC;
  __shared__ float red[4];
  const int64_t row = blockIdx.x;
  const int g = blockIdx.y, tid = threadIdx.x;
  y += row * y_stride, z += row * z_stride, out += row * out_stride;
  auto place = [&](int i) { return p == p_true ? i : i / p_true * p + i % p_true; };   // true column -> stored column
  const bool vec = size % VEC == 0 && p_true % VEC == 0;
  constexpr int KEEP = 4;   // vectors of the gated row that a thread keeps between the sum and the product
  float v[KEEP][VEC];
  float ss = 0.f;
  auto gated = [&](int c, float (&f)[VEC]) {
    float b[VEC];
    load_vec_row<Tag>(y + c, f);
    load_vec_row<Tag>(z + c, b);
#pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] = f[j] * silu_of<Tag>(b[j]);
  };
  if (vec) {
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int i = (tid + 256 * k) * VEC;
      if (i < size) {
        gated(place(g * size + i), v[k]);
#pragma unroll
        for (int j = 0; j < VEC; ++j) ss = fmaf(v[k][j], v[k][j], ss);
      }
    }
    for (int i = (tid + 256 * KEEP) * VEC; i < size; i += 256 * VEC) {
      float f[VEC];
      gated(place(g * size + i), f);
#pragma unroll
      for (int j = 0; j < VEC; ++j) ss = fmaf(f[j], f[j], ss);
    }
  } else {
    for (int i = tid; i < size; i += 256) {
      const int c = place(g * size + i);
      const float f = elem<Tag>::ld(y[c]) * silu_of<Tag>(elem<Tag>::ld(z[c]));
      ss = fmaf(f, f, ss);
    }
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float rs = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)size + eps);
  auto finish = [&](int c, const float (&f)[VEC]) {
    float o[VEC];
    load_vec_row<Tag>(w + c, o);
#pragma unroll
    for (int j = 0; j < VEC; ++j) o[j] = f[j] * rs * o[j];
    store_vec_row<Tag>(out + c, o);
  };
  if (vec) {
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int i = (tid + 256 * k) * VEC;
      if (i < size) finish(place(g * size + i), v[k]);
    }
    for (int i = (tid + 256 * KEEP) * VEC; i < size; i += 256 * VEC) {
      float f[VEC];
      const int c = place(g * size + i);
      gated(c, f);
      finish(c, f);
    }
  } else {
    for (int i = tid; i < size; i += 256) {
      const int c = place(g * size + i);
      out[c] = elem<Tag>::st(elem<Tag>::ld(y[c]) * silu_of<Tag>(elem<Tag>::ld(z[c])) * rs * elem<Tag>::ld(w[c]));
    }
  }
  if (p != p_true) {   // padding columns: this part's share of the heads
    const int pad = p - p_true, lo = (int64_t)heads * g / gridDim.y, hi = (int64_t)heads * (g + 1) / gridDim.y;
    for (int i = tid; i < (hi - lo) * pad; i += 256) out[(lo + i / pad) * p + p_true + i % pad] = elem<Tag>::st(0.f);
  }
}

}  // namespace

static int check_ssm(const MvSsmArgs *a, int dtype) {
  if (!a || !a->x || !a->out || !a->state_slots) return MV_E_NULLPTR;
  if (dtype != MV_BF16 && dtype != MV_F16 && dtype != MV_F32) return MV_E_DTYPE;
  if (a->n_seqs < 0 || a->n_seqs > 65535 || a->heads <= 0 || a->heads > 65535 || a->groups <= 0 || a->heads % a->groups ||
      a->p <= 0 || (a->p & 15) || a->p > 1024 || a->n <= 0 || (a->n & 31) || a->n > 512 || a->slots < 0 || a->taps < 1 ||
      a->taps > kMaxTaps || (a->channels & 31) || a->b_off < a->heads * a->p || a->b_off + a->groups * a->n > a->channels ||
      a->c_off < a->heads * a->p || a->c_off + a->groups * a->n > a->channels || a->x_stride < a->channels)
    return MV_E_SHAPE;
  const int vec = dtype == MV_F32 ? 4 : 8;
  if (!mv_aligned16(a->x) || a->x_stride % vec || (a->b_off & 7) || (a->c_off & 7) || !mv_aligned16(a->out) ||
      a->out_stride % vec)
    return MV_E_ALIGN;
  return MV_OK;
}

extern "C" int mv_causal_conv(const MvSsmArgs *a, int dtype, void *stream) {
  if (a && (a->n_seqs == 0 || a->max_q == 0)) return MV_OK;
  if (int e = check_ssm(a, dtype)) return e;
  if (!a->conv_w || !a->cu_q || !a->cu_k || (a->slots > 0 && a->taps > 1 && !a->conv_state)) return MV_E_NULLPTR;
  if (a->max_q < 0 || a->out_stride < a->channels) return MV_E_SHAPE;
  if (!mv_aligned16(a->conv_w) || (a->conv_b && !mv_aligned16(a->conv_b)) || (a->conv_state && !mv_aligned16(a->conv_state))) return MV_E_ALIGN;
  const int vec = dtype == MV_F32 ? 4 : 8, y = (a->max_q + kConvRows - 1) / kConvRows;
  if (y > 65535) return MV_E_SHAPE;
  const dim3 grid((a->channels / vec + 63) / 64, y, a->n_seqs);
  MV_DISPATCH_DTYPE(dtype, {
    if (a->taps <= 2) hipLaunchKernelGGL((causal_conv_kernel<Tag, 2>), grid, dim3(64), 0, (hipStream_t)stream, *a);
    else if (a->taps <= 4) hipLaunchKernelGGL((causal_conv_kernel<Tag, 4>), grid, dim3(64), 0, (hipStream_t)stream, *a);
    else hipLaunchKernelGGL((causal_conv_kernel<Tag, kMaxTaps>), grid, dim3(64), 0, (hipStream_t)stream, *a);
  });
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_ssm_prefill(const MvSsmArgs *a, int dtype, int flags, void *stream) {
  if (a && (a->n_seqs == 0 || a->max_q == 0)) return MV_OK;
  if (int e = check_ssm(a, dtype)) return e;
  if (!a->dt || !a->dt_bias || !a->a_log || !a->d || !a->cu_q || !a->cu_k || (a->slots > 0 && !a->ssm_state)) return MV_E_NULLPTR;
  if (a->max_q < 0 || a->dt_stride < a->heads || a->out_stride < a->heads * a->p) return MV_E_SHAPE;
  if (a->ssm_state && !mv_aligned16(a->ssm_state)) return MV_E_ALIGN;
  if (dtype != MV_F32 && !(flags & MV_SSM_SCAN)) {
    const int rc = mv_ssm_chunk_launch(*a, dtype, (hipStream_t)stream);
    if (rc != MV_E_SHAPE) return rc;
  }
  const size_t lds = (size_t)(2 * kScanRows * a->n + kScanRows * 16 + 2 * kScanRows) * 4;
  const dim3 grid(a->p / 16, a->heads, a->n_seqs);
  MV_DISPATCH_DTYPE(dtype, hipLaunchKernelGGL((ssm_scan_kernel<Tag>), grid, dim3(256), lds, (hipStream_t)stream, *a));
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_ssm_step(const MvSsmArgs *a, int dtype, void *stream) {
  if (a && a->n_seqs == 0) return MV_OK;
  if (int e = check_ssm(a, dtype)) return e;
  if (!a->dt || !a->dt_bias || !a->a_log || !a->d || !a->conv_w || !a->conv_b || !a->context_lens ||
      (a->slots > 0 && (!a->ssm_state || (a->taps > 1 && !a->conv_state))))
    return MV_E_NULLPTR;
  if (a->dt_stride < a->heads || a->out_stride < a->heads * a->p) return MV_E_SHAPE;
  if (a->ssm_state && !mv_aligned16(a->ssm_state)) return MV_E_ALIGN;
  const size_t lds = (size_t)(a->p + 2 * a->n + 256 / (a->p / 4) * a->p) * 4;
  MV_DISPATCH_DTYPE(dtype, hipLaunchKernelGGL((ssm_step_kernel<Tag>), dim3(a->heads, a->n_seqs), dim3(256), lds,
                                              (hipStream_t)stream, *a));
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_gated_group_norm(const void *y, int64_t y_stride, const void *z, int64_t z_stride, const void *w, void *out,
                                   int64_t out_stride, int rows, int heads, int p, int p_true, int norm_groups, float eps,
                                   int dtype, void *stream) {
  if (rows == 0) return MV_OK;
  if (!y || !z || !w || !out) return MV_E_NULLPTR;
  if (rows < 0 || heads <= 0 || p_true <= 0 || p < p_true || (p & 7) || norm_groups <= 0 || norm_groups > 65535 ||
      (int64_t)heads * p_true % norm_groups || y_stride < (int64_t)heads * p || z_stride < (int64_t)heads * p ||
      out_stride < (int64_t)heads * p)
    return MV_E_SHAPE;
  const int vec = dtype == MV_F32 ? 4 : 8;
  if (!mv_aligned16(y) || !mv_aligned16(z) || !mv_aligned16(w) || !mv_aligned16(out) || y_stride % vec || z_stride % vec ||
      out_stride % vec)
    return MV_E_ALIGN;
  MV_DISPATCH_DTYPE(dtype, {
    typedef typename elem<Tag>::T T;
    hipLaunchKernelGGL((gated_group_norm_kernel<Tag>), dim3(rows, norm_groups), dim3(256), 0, (hipStream_t)stream, (const T *)y,
                       y_stride, (const T *)z, z_stride, (const T *)w, (T *)out, out_stride, heads, p, p_true,
                       heads * p_true / norm_groups, eps);
  });
  MV_LAUNCH_CHECK();
  return MV_OK;
}
