// K18 — several residual streams (hyper-connections), include/mvhip.h: mv_stream_update.  One launch per edge: what the sublayer behind
// it gave is written to all streams, they are mixed, and what the next one reads comes out: a weighted sum of the new streams, its RMS
// norm, and (token shift) a blend with the norm of the token before.
//
// A workgroup takes a run of rows; a thread four columns of every stream.  With a token shift it needs the norm of the row ahead of
// its run, which it computes from that row's old streams once more (nothing is written), so old and new streams are different buffers.
// The workgroup of a sequence's first row, the only one that reads the kept norm of the step before, also writes the step's last one.
#include "vec4.h"

namespace {

constexpr int kMaxRun = 8;

// sum over the workgroup, every thread gets it; calls take turns with the two halves of red, so that one barrier a call is enough
__device__ __forceinline__ float turn_sum(float x, float (&red)[2][16], int &turn) {
  x = wave_sum(x);
  const int nw = blockDim.x >> 6;
  if (nw == 1) return x;
  float *r = red[turn ^= 1];
  if ((threadIdx.x & 63) == 0) r[threadIdx.x >> 6] = x;
  __syncthreads();
  float t = 0.f;
  for (int i = 0; i < nw; ++i) t += r[i];
  return t;
}

// S: streams (8: up to that many); MAXV: columns of a thread / 4
template <typename Tag, int S, int MAXV, bool SHIFT>
__global__ void __launch_bounds__(1024) stream_update_kernel(MvStreamArgs p, int rows, int cols, int cols_true, int run) {
  typedef typename elem<Tag>::T T;
  typedef vec4<Tag> V;
  __shared__ float red[2][16];
  const int tid = threadIdx.x, nt = blockDim.x, r0 = blockIdx.x * run, r1 = min(rows, r0 + run), n = S == 8 ? p.streams : S;
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  int turn = 0;
  auto weight = [](const void *w, int i) { return elem<Tag>::ld(((const T *)w)[i]); };
  auto column = [&](int v) { return (tid + v * nt) * 4; };
  f32x4 wn[MAXV], sh[MAXV];
#pragma unroll
  for (int v = 0; v < MAXV; ++v) {
    const int c = column(v);
    wn[v] = sh[v] = zero;
    if (c < cols) {
      wn[v] = V::load((const T *)p.norm_w + c);
      if (SHIFT) sh[v] = V::load((const T *)p.shift + c);
    }
  }
  // the norm that row `row` gives the next sublayer; `write`: its new streams are kept
  auto normed = [&](int row, bool write, f32x4 (&h)[MAXV]) {
    int64_t id = -1;
    if (p.embed) {
      id = p.ids[row];
      if (id >= p.vocab) id = -1;
    }
    float ss = 0.f;
#pragma unroll
    for (int v = 0; v < MAXV; ++v) {
      const int c = column(v);
      h[v] = zero;
      if (c >= cols) continue;
      f32x4 x[S], y = zero;
      if (p.embed) {
        const f32x4 e = id >= 0 ? V::load((const T *)p.embed + id * cols + c) : zero;
#pragma unroll
        for (int j = 0; j < S; ++j) x[j] = e;
      } else {
        const float *xr = p.x + (int64_t)row * n * cols + c;
#pragma unroll
        for (int j = 0; j < S; ++j) x[j] = S < 8 || j < n ? *reinterpret_cast<const f32x4 *>(xr + (int64_t)j * cols) : zero;
        if (p.y_splits > 0) {
          const float *yr = (const float *)p.y + (int64_t)row * cols + c;
          y = *reinterpret_cast<const f32x4 *>(yr);
          for (int s = 1; s < p.y_splits; ++s) y += *reinterpret_cast<const f32x4 *>(yr + (int64_t)s * rows * cols);
        } else if (p.y) {
          y = V::load((const T *)p.y + (int64_t)row * p.y_stride + c);
        }
        for (int k = 0; k < p.moe_top; ++k) {
          const int from = p.moe_rows[(int64_t)row * p.moe_top + k];
          const float w = p.moe_w ? p.moe_w[(int64_t)row * p.moe_top + k] : 1.0f;
          if (from >= 0) y += w * V::load((const T *)p.moe_out + (int64_t)from * cols + c);
        }
      }
#pragma unroll
      for (int j = 0; j < S; ++j) {
        if (S == 8 && j >= n) continue;
        f32x4 to = x[j];
        if (!p.embed) {
          to = weight(p.out_w, j) * y;
#pragma unroll
          for (int i = 0; i < S; ++i) {
            if (S == 8 && i >= n) continue;
            const float m = weight(p.mix, i * n + j);
#pragma unroll
            for (int e = 0; e < 4; ++e) to[e] = fmaf(m, x[i][e], to[e]);
          }
        }
        if (write && p.x_out) *reinterpret_cast<f32x4 *>(p.x_out + ((int64_t)row * n + j) * cols + c) = to;
        const float a = p.in_w ? weight(p.in_w, j) : 1.0f;
#pragma unroll
        for (int e = 0; e < 4; ++e) h[v][e] = fmaf(a, to[e], h[v][e]);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(h[v][e], h[v][e], ss);
    }
    const float rs = 1.0f / sqrtf(turn_sum(ss, red, turn) / (float)cols_true + p.eps);
#pragma unroll
    for (int v = 0; v < MAXV; ++v) h[v] = h[v] * rs * wn[v];
  };
  f32x4 h[MAXV], before[MAXV];
  int seq = 0, first = 0, last = 0;
  float *kept = nullptr;   // where this sequence's last norm goes (columns of this thread apart)
  if (SHIFT && p.cu_q) {
    for (int hi = p.n_seqs; hi - seq > 1;) {
      const int mid = (seq + hi) >> 1;
      if (p.cu_q[mid] <= r0) seq = mid;
      else hi = mid;
    }
  }
  auto keep = [&](const f32x4 (&hl)[MAXV]) {
#pragma unroll
    for (int v = 0; v < MAXV; ++v)
      if (column(v) < cols) *reinterpret_cast<f32x4 *>(kept + column(v)) = hl[v];
  };
  for (int row = r0; row < r1; ++row) {
    if constexpr (SHIFT) {
      if (p.cu_q) {
        while (seq + 1 < p.n_seqs && row >= p.cu_q[seq + 1]) ++seq;
        first = p.cu_q[seq], last = p.cu_q[seq + 1] - 1;
      } else {
        seq = first = last = row;
      }
      if (row == first) {
        const int64_t pos = p.positions[row];
        const int slot = p.state_slots[seq];
        const bool held = pos >= 0 && slot >= 0 && slot < p.slots;
        const float *old = held && pos > 0 ? p.prev + ((pos & 1) * p.slots + slot) * cols : nullptr;
        kept = held ? p.prev + (((pos + last - first + 1) & 1) * p.slots + slot) * cols : nullptr;
#pragma unroll
        for (int v = 0; v < MAXV; ++v)
          before[v] = old && column(v) < cols ? *reinterpret_cast<const f32x4 *>(old + column(v)) : zero;
        if (kept && last >= r1) {
          normed(last, false, h);
          keep(h);
        }
      } else if (row == r0) {
        kept = nullptr;
        normed(row - 1, false, before);
      }
    }
    normed(row, true, h);
    if (p.out) {
#pragma unroll
      for (int v = 0; v < MAXV; ++v) {
        const int c = column(v);
        if (c >= cols) continue;
        f32x4 o = h[v];
        if constexpr (SHIFT) {
#pragma unroll
          for (int e = 0; e < 4; ++e) o[e] = fmaf(before[v][e] - o[e], sh[v][e], o[e]);
        }
        V::store((T *)p.out + (int64_t)row * p.out_stride + c, o);
      }
    }
    if constexpr (SHIFT) {
      if (row == last && kept) keep(h);
#pragma unroll
      for (int v = 0; v < MAXV; ++v) before[v] = h[v];
    }
  }
}

template <typename Tag, int S, int MAXV>
void launch(const MvStreamArgs &a, int rows, int cols, int cols_true, int run, int threads, hipStream_t st) {
  const dim3 grid((rows + run - 1) / run);
  if (a.shift) hipLaunchKernelGGL((stream_update_kernel<Tag, S, MAXV, true>), grid, dim3(threads), 0, st, a, rows, cols, cols_true, run);
  else hipLaunchKernelGGL((stream_update_kernel<Tag, S, MAXV, false>), grid, dim3(threads), 0, st, a, rows, cols, cols_true, run);
}
template <typename Tag, int S>
int launch_width(const MvStreamArgs &a, int rows, int cols, int cols_true, int run, hipStream_t st) {
  const int threads = min((cols / 4 + 63) / 64 * 64, 1024), per = (cols / 4 + threads - 1) / threads;
  if (per <= 1) launch<Tag, S, 1>(a, rows, cols, cols_true, run, threads, st);
  else if (per <= 2) launch<Tag, S, 2>(a, rows, cols, cols_true, run, threads, st);
  else if (per <= 4) launch<Tag, S, 4>(a, rows, cols, cols_true, run, threads, st);
  else return MV_E_SHAPE;   // > 16384 columns
  MV_LAUNCH_CHECK();
  return MV_OK;
}

}  // namespace

extern "C" int mv_stream_update(const MvStreamArgs *a, int rows, int cols, int cols_true, int dtype, void *stream) {
  if (rows == 0) return MV_OK;
  if (!a || !a->norm_w || (!a->out && !a->x_out)) return MV_E_NULLPTR;
  if (rows < 0 || cols <= 0 || (cols & 7) || cols_true <= 0 || cols_true > cols || a->streams < 1 || a->streams > 8 || a->y_splits < 0 ||
      a->moe_top < 0 || (a->out && a->out_stride < cols) || (a->y && a->y_splits == 0 && a->y_stride < cols))
    return MV_E_SHAPE;
  if (dtype != MV_BF16 && dtype != MV_F16 && dtype != MV_F32) return MV_E_DTYPE;
  if (a->embed ? (!a->ids || a->vocab <= 0) : (!a->x || !a->mix || !a->out_w)) return MV_E_NULLPTR;
  if ((a->y_splits > 0 && !a->y) || (a->moe_top && (!a->moe_out || !a->moe_rows))) return MV_E_NULLPTR;
  if (a->shift) {
    if (!a->positions || !a->state_slots || (a->slots > 0 && !a->prev)) return MV_E_NULLPTR;
    if (a->slots < 0 || (a->cu_q && a->n_seqs <= 0)) return MV_E_SHAPE;
    if (a->cu_q && !a->embed && a->x_out == a->x) return MV_E_ALIAS;
  }
  const void *at[] = {a->x, a->x_out, a->y, a->embed, a->norm_w, a->shift, a->out, a->moe_out, a->prev};
  for (const void *q : at)
    if (q && !mv_aligned16(q)) return MV_E_ALIGN;
  if ((a->out && (a->out_stride & 7)) || (a->y && a->y_splits == 0 && (a->y_stride & 7))) return MV_E_ALIGN;
  // runs of rows: the row ahead of a run is computed twice, but the chip has to be full
  int run = 1;
  while (a->shift && a->cu_q && run < kMaxRun && rows / run > 2048) run *= 2;
  hipStream_t st = (hipStream_t)stream;
  MV_DISPATCH_DTYPE(dtype, {
    switch (a->streams) {
      case 1: return launch_width<Tag, 1>(*a, rows, cols, cols_true, run, st);
      case 2: return launch_width<Tag, 2>(*a, rows, cols, cols_true, run, st);
      case 3: return launch_width<Tag, 3>(*a, rows, cols, cols_true, run, st);
      case 4: return launch_width<Tag, 4>(*a, rows, cols, cols_true, run, st);
      default: return launch_width<Tag, 8>(*a, rows, cols, cols_true, run, st);
    }
  });
  return MV_OK;
}
