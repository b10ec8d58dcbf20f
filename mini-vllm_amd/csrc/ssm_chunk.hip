// K15 — selective state space recurrence of prompts in chunks of 64 tokens on the matrix cores (16-bit operands, fp32 state).
//
// Within a chunk, with r_i = the sum of the log decays of tokens 0 .. i, the recurrence unrolls to
//     y_i  = exp(r_i) S^T c_i + sum_{j <= i} exp(r_i - r_j) dt_j (c_i . b_j) x_j + d x_i
//     S   <- exp(r_last) S + sum_j exp(r_last - r_j) dt_j b_j x_j^T
// b, c and x are 16-bit values, so c_i . b_j is exact products in fp32.  What is fp32 by nature (S, the weighted scores, the
// weighted x) enters its product as the sum of two 16-bit numbers, high part and remainder: two MFMAs instead of one, about
// 16 bits of mantissa.
//
// One workgroup = PT waves = PT tiles of 16 columns of one head of one sequence, chunks one behind the other; wave w keeps S of
// its columns in accumulators for the whole sequence (v_mfma_f32_16x16x32, S[n][p]: a lane holds rows of one column).
// Accumulators are operands of the next product as they are: the transposed reads of b deal the rows of S so that tiles 2 s and
// 2 s + 1 together hold n = 32 s + 8 g .. + 7 in lane group g, the k order of an operand; the weighted scores' two key tiles are
// one operand with k permuted (k = 8 g + e means key 16 (e >> 2) + 4 g + (e & 3)), and x is read in that order.  So S stays in
// registers, and the scores go through LDS once (each wave computes some of the 4 token tiles, all waves read all).  The next
// chunk's rows are requested before the current chunk's products.
#include "ssm.h"

namespace {

typedef __attribute__((ext_vector_type(4))) short s16x4;
typedef __attribute__((address_space(3))) s16x4 lds_s16x4;

constexpr int L = 64;   // tokens per chunk

// v = hi + lo in 16-bit parts
template <typename Tag>
__device__ __forceinline__ void split4(const f32x4 &v, u32x2 &hi, u32x2 &lo) {
  hi = pack_quad<Tag>(v);
  f32x4 r;
#pragma unroll
  for (int i = 0; i < 2; ++i) {
    if constexpr (__is_same(Tag, bf16_tag)) {
      r[2 * i] = v[2 * i] - u2f(hi[i] << 16);
      r[2 * i + 1] = v[2 * i + 1] - u2f(hi[i] & 0xffff0000u);
    } else {
      r[2 * i] = v[2 * i] - f16_bits_to_f32((uint16_t)(hi[i] & 0xffffu));
      r[2 * i + 1] = v[2 * i + 1] - f16_bits_to_f32((uint16_t)(hi[i] >> 16));
    }
  }
  lo = pack_quad<Tag>(r);
}
__device__ __forceinline__ u32x4 join(const u32x2 &a, const u32x2 &b) { return u32x4{a.x, a.y, b.x, b.y}; }
__device__ __forceinline__ u32x2 read_tr(const char *p) {
  return __builtin_bit_cast(u32x2, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4 *)p));
}

// NK: state rows / 32
template <typename Tag, int NK, int PT>
__global__ void __launch_bounds__(PT * 64, PT == 4 ? 2 : 1) ssm_chunk_kernel(MvSsmArgs p) {
  typedef typename elem<Tag>::T T;
  constexpr int N = NK * 32, THREADS = PT * 64;
  // LDS rows: x an odd number of 16-byte pieces; b and c 2 (mod 4), so that the row reads stay apart over 8 rows and the
  // transposed reads, whose pieces lie 16 bytes apart, meet at most in pairs
  constexpr int RB = (N / 8 + 2) * 16, RX = (2 * PT + 1) * 16;
  constexpr int CB = L * N / 8, CX = L * 2 * PT, PIECES = 2 * CB + CX;   // 16-byte pieces of b, c and x
  constexpr int PER = (PIECES + THREADS - 1) / THREADS, AHEAD = PER <= 20 ? PER : 20;
  __shared__ __attribute__((aligned(16))) char bs[L * RB], cs[L * RB], xs[L * RX];
  __shared__ u32x4 wf[2][4][2][64];            // weighted scores, high / remainder: [token tile][32 keys][lane]
  __shared__ float steps[2][3][L];             // of this and the next chunk: r_i (log2), dt_i, exp(r_last - r_i) dt_i
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), r16 = lane & 15, g = lane >> 4;
  const int slice = blockIdx.x, head = blockIdx.y, seq = blockIdx.z;
  const int q0 = p.cu_q[seq], len = p.cu_q[seq + 1] - q0;
  if (len <= 0) return;
  const int before = p.cu_k[seq + 1] - p.cu_k[seq] - len, slot = p.state_slots[seq], grp = head / (p.heads / p.groups);
  const bool keep = slot >= 0 && slot < p.slots;
  const int64_t size = (int64_t)p.heads * p.n * p.p;
  const int64_t at = (int64_t)(keep ? slot : 0) * size + (int64_t)head * p.n * p.p + slice * 16 * PT + wave * 16 + r16;
  const T *x = (const T *)p.x + (int64_t)q0 * p.x_stride, *dt = (const T *)p.dt + (int64_t)q0 * p.dt_stride + head;
  const int bcol = p.b_off + grp * p.n, ccol = p.c_off + grp * p.n, xcol = head * p.p + slice * 16 * PT;
  const float na2 = -expf(elem<Tag>::ld(((const T *)p.a_log)[head])) * 1.4426950408889634f;
  const float bias = elem<Tag>::ld(((const T *)p.dt_bias)[head]), d = elem<Tag>::ld(((const T *)p.d)[head]);

  auto state_row = [&](int i, int e) { return (i >> 1) * 32 + g * 8 + (i & 1) * 4 + e; };
  f32x4 st[2 * NK];
#pragma unroll
  for (int i = 0; i < 2 * NK; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e)
      st[i][e] = keep && before > 0 ? p.ssm_state[(before & 1) * p.slots * size + at + (int64_t)state_row(i, e) * p.p] : 0.f;

  // piece i of a chunk: its row, where it comes from (of row 0), where it goes
  auto piece = [&](int i, int &row, int &col) {
    const bool isx = i >= 2 * CB;
    const int j = isx ? i - 2 * CB : (i >= CB ? i - CB : i), c = isx ? j % (2 * PT) : j % (N / 8);
    row = isx ? j / (2 * PT) : j / (N / 8);
    col = (isx ? xcol : (i >= CB ? ccol : bcol)) + c * 8;
    return (isx ? xs + row * RX : (i >= CB ? cs : bs) + row * RB) + c * 16;
  };
  char *dst[AHEAD];
  const T *src[AHEAD];
  int rows[AHEAD];
#pragma unroll
  for (int k = 0; k < AHEAD; ++k) {
    int col;
    dst[k] = piece(min(k * THREADS + tid, PIECES - 1), rows[k], col);
    src[k] = x + (int64_t)rows[k] * p.x_stride + col;
  }
  u32x4 ahead[AHEAD];
  float dt_ahead = 0.f;
  auto request = [&](int t0) {
    if (wave == 0) dt_ahead = elem<Tag>::ld(dt[(int64_t)min(t0 + lane, len - 1) * p.dt_stride]);
    if (t0 + L <= len) {
      const int64_t off = (int64_t)t0 * p.x_stride;
#pragma unroll
      for (int k = 0; k < AHEAD; ++k) ahead[k] = *(const u32x4 *)(src[k] + off);
    } else {   // the last, short chunk: rows behind the end repeat the last token (weight 0)
#pragma unroll
      for (int k = 0; k < AHEAD; ++k)
        ahead[k] = *(const u32x4 *)(src[k] + (int64_t)(min(t0 + rows[k], len - 1) - rows[k]) * p.x_stride);
    }
  };
  // step sizes and decays of the requested chunk (wave 0); tokens behind the end: dt = 0, no decay
  auto scan = [&](int nt, float (*to)[L]) {
    const float step = lane < nt ? softplus_f32(dt_ahead + bias) : 0.f;
    float r = na2 * step;
#pragma unroll
    for (int o = 1; o < 64; o *= 2) {
      const float v = __shfl_up(r, o, 64);
      if (lane >= o) r += v;
    }
    to[0][lane] = r, to[1][lane] = step;
    to[2][lane] = __builtin_amdgcn_exp2f(__shfl(r, 63, 64) - r) * step;
  };
  request(0);
  if (wave == 0) scan(min(L, len), steps[0]);

  for (int t0 = 0; t0 < len; t0 += L) {
    const int nt = min(L, len - t0), cur = (t0 / L) & 1;
    const float *rs = steps[cur][0], *dts = steps[cur][1], *ws = steps[cur][2];
#pragma unroll
    for (int k = 0; k < AHEAD; ++k) *(u32x4 *)dst[k] = ahead[k];   // (threads without a piece repeat the last one)
    if constexpr (PER > AHEAD) {
      for (int i = AHEAD * THREADS + tid; i < PIECES; i += THREADS) {
        int row, col;
        char *to = piece(i, row, col);
        *(u32x4 *)to = *(const u32x4 *)(x + (int64_t)min(t0 + row, len - 1) * p.x_stride + col);
      }
    }
    __syncthreads();
    if (t0 + L < len) request(t0 + L);

    // ---- S^T c of all tokens (this wave's columns), scaled by exp(r_i)
    f32x4 y[4] = {};
#pragma unroll
    for (int s = 0; s < NK; ++s) {
      u32x2 h0, l0, h1, l1;
      split4<Tag>(st[2 * s], h0, l0);
      split4<Tag>(st[2 * s + 1], h1, l1);
      const u32x4 hi = join(h0, h1), lo = join(l0, l1);
      u32x4 c[4];
#pragma unroll
      for (int it = 0; it < 4; ++it) c[it] = *(const u32x4 *)(cs + (it * 16 + r16) * RB + s * 64 + g * 16);
      // (products of one accumulator never back to back: the second would wait for the first's whole latency)
#pragma unroll
      for (int it = 0; it < 4; ++it) y[it] = mfma16x16x32<Tag>(hi, c[it], y[it]);
#pragma unroll
      for (int it = 0; it < 4; ++it) y[it] = mfma16x16x32<Tag>(lo, c[it], y[it]);
    }
    float ri[4];
#pragma unroll
    for (int it = 0; it < 4; ++it) {
      ri[it] = rs[it * 16 + r16];
      y[it] *= __builtin_amdgcn_exp2f(ri[it]);
    }
    // ---- weighted scores of this wave's token tiles, [key][token]
    for (int it = wave; it < 4; it += PT) {
      u32x4 cf[NK];
#pragma unroll
      for (int s = 0; s < NK; ++s) cf[s] = *(const u32x4 *)(cs + (it * 16 + r16) * RB + s * 64 + g * 16);
      const float r_tok = rs[it * 16 + r16];
      f32x4 sc[4] = {};
#pragma unroll
      for (int s = 0; s < NK; ++s)
#pragma unroll
        for (int jt = 0; jt < 4; ++jt)
          if (jt <= it) sc[jt] = mfma16x16x32<Tag>(*(const u32x4 *)(bs + (jt * 16 + r16) * RB + s * 64 + g * 16), cf[s], sc[jt]);
#pragma unroll
      for (int jt = 0; jt < 4; ++jt) {
        u32x2 hi = {0u, 0u}, lo = {0u, 0u};
        if (jt <= it) {
          f32x4 a = sc[jt];
          const f32x4 rk = *(const f32x4 *)(rs + jt * 16 + g * 4), dk = *(const f32x4 *)(dts + jt * 16 + g * 4);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const bool seen = jt * 16 + g * 4 + e <= it * 16 + r16;
            a[e] = seen ? a[e] * (__builtin_amdgcn_exp2f(seen ? r_tok - rk[e] : 0.f) * dk[e]) : 0.f;
          }
          split4<Tag>(a, hi, lo);
        }
        *((u32x2 *)&wf[0][it][jt >> 1][lane] + (jt & 1)) = hi;
        *((u32x2 *)&wf[1][it][jt >> 1][lane] + (jt & 1)) = lo;
      }
    }
    if (wave == 0 && t0 + L < len) scan(min(L, len - t0 - L), steps[cur ^ 1]);   // (wave 0 scored the fewest keys)
    __syncthreads();
    // ---- sum over the chunk's keys; then the state moves on
    const float tail = __builtin_amdgcn_exp2f(rs[L - 1]);
#pragma unroll
    for (int i = 0; i < 2 * NK; ++i) st[i] *= tail;
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      const char *xa = xs + (32 * s + 4 * g + (r16 >> 2)) * RX + wave * 32 + (r16 & 3) * 8;
      const u32x2 x0 = read_tr(xa), x1 = read_tr(xa + 16 * RX);
      const u32x4 xf = join(x0, x1);
#pragma unroll
      for (int part = 0; part < 2; ++part)
#pragma unroll
        for (int it = 2 * s; it < 4; ++it) y[it] = mfma16x16x32<Tag>(xf, wf[part][it][s][lane], y[it]);   // keys 32 s ..
      float f[8];
      unpack8<Tag>(xf, f);
      const f32x4 w0 = *(const f32x4 *)(ws + 32 * s + 4 * g), w1 = *(const f32x4 *)(ws + 32 * s + 16 + 4 * g);
      u32x2 h0, l0, h1, l1;
      split4<Tag>(f32x4{f[0], f[1], f[2], f[3]} * w0, h0, l0);
      split4<Tag>(f32x4{f[4], f[5], f[6], f[7]} * w1, h1, l1);
      const u32x4 hi = join(h0, h1), lo = join(l0, l1);
      const char *ba = bs + (32 * s + 4 * g + (r16 >> 2)) * RB + (r16 & 3) * 16;
      constexpr int IB = NK % 2 == 0 ? 4 : 2;   // state tiles at a time
#pragma unroll
      for (int i = 0; i < 2 * NK; i += IB) {
        u32x4 b[IB];
#pragma unroll
        for (int j = 0; j < IB; ++j) {
          const int o = ((i + j) >> 1) * 64 + ((i + j) & 1) * 8;
          b[j] = join(read_tr(ba + o), read_tr(ba + 16 * RB + o));
        }
#pragma unroll
        for (int j = 0; j < IB; ++j) st[i + j] = mfma16x16x32<Tag>(b[j], hi, st[i + j]);
#pragma unroll
        for (int j = 0; j < IB; ++j) st[i + j] = mfma16x16x32<Tag>(b[j], lo, st[i + j]);
      }
    }
    // ---- out: lane (token r16, columns 4 g ..)
#pragma unroll
    for (int it = 0; it < 4; ++it) {
      const int t = it * 16 + r16;
      const u32x2 raw = *(const u32x2 *)(xs + t * RX + wave * 32 + g * 8);
      float o[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const uint32_t bits = raw[e >> 1];
        o[e] = fmaf(d, elem<Tag>::ld((uint16_t)((e & 1) ? bits >> 16 : bits & 0xffffu)), y[it][e]);
      }
      if (t < nt)
        *(u32x2 *)((T *)p.out + (int64_t)(q0 + t0 + t) * p.out_stride + xcol + wave * 16 + g * 4) =
            u32x2{pack_pair<Tag>(o[0], o[1]), pack_pair<Tag>(o[2], o[3])};
    }
    __syncthreads();
  }
  if (keep) {
    float *ns = p.ssm_state + ((before + len) & 1) * p.slots * size + at;
#pragma unroll
    for (int i = 0; i < 2 * NK; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) ns[(int64_t)state_row(i, e) * p.p] = st[i][e];
  }
}

template <typename Tag, int NK>
int launch(const MvSsmArgs &a, hipStream_t stream) {
  // column tiles per workgroup: as many as divide the head's.  They share the b / c rows and the scores; fewer per workgroup
  // measured slower even where they fill an otherwise idle chip (a lone wave loads and scores everything by itself)
  const int tiles = a.p / 16, pt = tiles % 4 == 0 ? 4 : tiles % 3 == 0 ? 3 : tiles % 2 == 0 ? 2 : 1;
  const dim3 grid(tiles / pt, a.heads, a.n_seqs);
#define MV_SC(PT_) hipLaunchKernelGGL((ssm_chunk_kernel<Tag, NK, PT_>), grid, dim3(PT_ * 64), 0, stream, a)
  if (pt == 4) MV_SC(4);
  else if (pt == 3) MV_SC(3);
  else if (pt == 2) MV_SC(2);
  else MV_SC(1);
#undef MV_SC
  MV_LAUNCH_CHECK();
  return MV_OK;
}

}  // namespace

int mv_ssm_chunk_launch(const MvSsmArgs &a, int dtype, hipStream_t stream) {
#define MV_SN(N_) \
  if (a.n == N_) return dtype == MV_BF16 ? launch<bf16_tag, N_ / 32>(a, stream) : launch<f16_tag, N_ / 32>(a, stream)
  MV_SN(32);
  MV_SN(64);
  MV_SN(96);
  MV_SN(128);
  MV_SN(160);
  MV_SN(192);
  MV_SN(256);
#undef MV_SN
  return MV_E_SHAPE;   // larger states: token by token
}
