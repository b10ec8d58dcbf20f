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

// S: streams (8: up to that many); MAXV: columns of a thread / 4; MOE: expert rows are part of y
template <typename Tag, int S, int MAXV, bool SHIFT, bool MOE>
__global__ void __launch_bounds__(MAXV > 1 ? 512 : 1024) stream_update_kernel(MvStreamArgs p, int rows, int cols, int cols_true, int run) {
  typedef typename elem<Tag>::T T;
  typedef vec4<Tag> V;
  __shared__ float red[2][16];
  const int tid = threadIdx.x, nt = blockDim.x, r0 = blockIdx.x * run, r1 = min(rows, r0 + run), n = S == 8 ? p.streams : S;
  constexpr int CHOICES = !MOE ? 1 : MAXV == 1 ? 8 : 2;   // of a token's expert rows, requested ahead
  const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
  int turn = 0;
  // the streams' weights: mix by target, then what is written, then what is read
  __shared__ __attribute__((aligned(16))) float weights[S * S + 2 * S];
  for (int i = tid; i < S * S + 2 * S; i += nt) {
    const int j = i < S * S ? i / S : i - S * S - (i >= S * S + S ? S : 0), from = i % S;
    const void *w = i < S * S ? p.mix : i < S * S + S ? p.out_w : p.in_w;
    const bool live = j < n && (i >= S * S || from < n);
    float f = i >= S * S + S ? 1.0f : 0.f;
    if (w && live) f = elem<Tag>::ld(((const T *)w)[i < S * S ? from * n + j : j]);
    weights[i] = live ? f : 0.f;
  }
  __syncthreads();
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
  // what a row's arithmetic starts from, on its way from memory
  struct Raw {
    f32x4 x[MAXV][S];
    typename V::R y[MAXV], m[MAXV][CHOICES];
    int from[CHOICES], from_next[CHOICES], next;   // places of the expert rows, and of those of row `next`
  };
  auto request = [&](int row, Raw &r) __attribute__((always_inline)) {
    if (p.embed) return;
#pragma unroll
    for (int v = 0; v < MAXV; ++v) {
      const int c = column(v);
      if (c >= cols) continue;
      const float *xr = p.x + (int64_t)row * n * cols + c;
#pragma unroll
      for (int j = 0; j < S; ++j)
        if (S < 8 || j < n) r.x[v][j] = *reinterpret_cast<const f32x4 *>(xr + (int64_t)j * cols);
      if (p.y && p.y_splits == 0) r.y[v] = V::raw((const T *)p.y + (int64_t)row * p.y_stride + c);
    }
    if constexpr (!MOE) return;
    if (row == r.next) {
#pragma unroll
      for (int k = 0; k < CHOICES; ++k) r.from[k] = r.from_next[k];
    } else {
#pragma unroll
      for (int k = 0; k < CHOICES; ++k) r.from[k] = k < p.moe_top ? p.moe_rows[(int64_t)row * p.moe_top + k] : -1;
    }
    r.next = row + 1;
    if (row + 1 < r1) {
#pragma unroll
      for (int k = 0; k < CHOICES; ++k) r.from_next[k] = k < p.moe_top ? p.moe_rows[(int64_t)(row + 1) * p.moe_top + k] : -1;
    }
#pragma unroll
    for (int v = 0; v < MAXV; ++v)
#pragma unroll
      for (int k = 0; k < CHOICES; ++k)
        if (column(v) < cols && r.from[k] >= 0) r.m[v][k] = V::raw((const T *)p.moe_out + (int64_t)r.from[k] * cols + column(v));
  };
  // the norm that row `row` gives the next sublayer; `write`: its new streams are kept; next >= 0: the row to request in the place of
  // this one, ahead of the stores and the reduction
  auto normed = [&](int row, Raw &r, bool write, int next, f32x4 (&h)[MAXV]) __attribute__((always_inline)) {
    const bool start = p.embed != nullptr;
    int64_t id = -1;
    if (start) {
      id = p.ids[row];
      if (id >= p.vocab) id = -1;
    }
    float ss = 0.f;
    f32x4 to[MAXV][S];
#pragma unroll
    for (int v = 0; v < MAXV; ++v) {
      const int c = column(v);
      h[v] = zero;
      if (c >= cols) continue;
      f32x4 y = zero;
      if (start) {
        if (id >= 0) y = V::load((const T *)p.embed + id * cols + c);
      } else {
        if (p.y_splits > 0) {
          const float *yr = (const float *)p.y + (int64_t)row * cols + c;
          y = *reinterpret_cast<const f32x4 *>(yr);
          for (int s = 1; s < p.y_splits; ++s) y += *reinterpret_cast<const f32x4 *>(yr + (int64_t)s * rows * cols);
        } else if (p.y) {
          y = V::unpack(r.y[v]);
        }
        if constexpr (MOE) {
#pragma unroll
          for (int k = 0; k < CHOICES; ++k)
            if (r.from[k] >= 0) y += (p.moe_w ? p.moe_w[(int64_t)row * p.moe_top + k] : 1.0f) * V::unpack(r.m[v][k]);
          for (int k = CHOICES; k < p.moe_top; ++k) {
            const int from = p.moe_rows[(int64_t)row * p.moe_top + k];
            const float w = p.moe_w ? p.moe_w[(int64_t)row * p.moe_top + k] : 1.0f;
            if (from >= 0) y += w * V::load((const T *)p.moe_out + (int64_t)from * cols + c);
          }
        }
      }
#pragma unroll
      for (int j = 0; j < S; ++j) {
        if (S == 8 && j >= n) continue;
        to[v][j] = start ? y : weights[S * S + j] * y;
        if (!start) {
#pragma unroll
          for (int i = 0; i < S; ++i) {
            if (S == 8 && i >= n) continue;
            const float m = weights[j * S + i];
#pragma unroll
            for (int e = 0; e < 4; ++e) to[v][j][e] = fmaf(m, r.x[v][i][e], to[v][j][e]);
          }
        }
        const float a = weights[S * S + S + j];
#pragma unroll
        for (int e = 0; e < 4; ++e) h[v][e] = fmaf(a, to[v][j][e], h[v][e]);
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) ss = fmaf(h[v][e], h[v][e], ss);
    }
    if (next >= 0) request(next, r);
    if (write && p.x_out) {
#pragma unroll
      for (int v = 0; v < MAXV; ++v)
        if (column(v) < cols) {
#pragma unroll
          for (int j = 0; j < S; ++j)
            if (S < 8 || j < n) *reinterpret_cast<f32x4 *>(p.x_out + ((int64_t)row * n + j) * cols + column(v)) = to[v][j];
        }
    }
    const float rs = 1.0f / sqrtf(turn_sum(ss, red, turn) / (float)cols_true + p.eps);
#pragma unroll
    for (int v = 0; v < MAXV; ++v) h[v] = h[v] * rs * wn[v];
  };
  f32x4 h[MAXV], before[MAXV];
  int seq = 0, first = 0, last = 0;
  float *kept = nullptr;   // where this sequence's last norm goes
  if (SHIFT && p.cu_q) {
    for (int hi = p.n_seqs; hi - seq > 1;) {
      const int mid = (seq + hi) >> 1;
      if (p.cu_q[mid] <= r0) seq = mid;
      else hi = mid;
    }
  }
  // the sequence of `row`; at its first row also the norm of the token before
  auto enter = [&](int row) __attribute__((always_inline)) {
    if (p.cu_q) {
      while (seq + 1 < p.n_seqs && row >= p.cu_q[seq + 1]) ++seq;
      first = p.cu_q[seq], last = p.cu_q[seq + 1] - 1;
    } else {
      seq = first = last = row;
    }
    kept = nullptr;
    if (row != first) return;
    const int64_t pos = p.positions[row];
    const int slot = p.state_slots[seq];
    const bool held = pos >= 0 && slot >= 0 && slot < p.slots;
    const float *old = held && pos > 0 ? p.prev + ((pos & 1) * p.slots + slot) * cols : nullptr;
    if (held) kept = p.prev + (((pos + last - first + 1) & 1) * p.slots + slot) * cols;
#pragma unroll
    for (int v = 0; v < MAXV; ++v) before[v] = old && column(v) < cols ? *reinterpret_cast<const f32x4 *>(old + column(v)) : zero;
  };
  // what is computed at a time: a row of the run; ahead of it, at the run's start, the row before it; at a sequence's start, its last row
  enum { kRow, kAhead, kLast };
  int row = r0, kind = kRow, at = r0;
  if constexpr (SHIFT) {
    enter(r0);
    if (r0 != first) kind = kAhead, at = r0 - 1;
    else if (kept && last >= r1) kind = kLast, at = last;
  }
  Raw raw;
  raw.next = -1;
  request(at, raw);
  for (;;) {
    const int then = kind == kRow ? row + 1 : row;
    const bool more = then < r1, border = SHIFT && then > last;
    normed(at, raw, kind == kRow, more && !border ? then : -1, h);
    if (kind == kRow && p.out) {
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
      if (kept && at == last) {
#pragma unroll
        for (int v = 0; v < MAXV; ++v)
          if (column(v) < cols) *reinterpret_cast<f32x4 *>(kept + column(v)) = h[v];
      }
      if (kind != kLast) {
#pragma unroll
        for (int v = 0; v < MAXV; ++v) before[v] = h[v];
      }
    }
    if (!more) break;
    row = at = then, kind = kRow;
    if constexpr (SHIFT) {
      if (border) {
        enter(row);
        if (kept && last >= r1) kind = kLast, at = last;
        request(at, raw);
      }
    }
  }
}

template <typename Tag, int S, int MAXV>
void launch(const MvStreamArgs &a, int rows, int cols, int cols_true, int run, int threads, hipStream_t st) {
  const dim3 grid((rows + run - 1) / run);
#define MV_STREAMS(SHIFT, MOE)                                                                                                              \
  hipLaunchKernelGGL((stream_update_kernel<Tag, S, MAXV, SHIFT, MOE>), grid, dim3(threads), 0, st, a, rows, cols, cols_true, run)
  if (a.shift && a.moe_top) MV_STREAMS(true, true);
  else if (a.shift) MV_STREAMS(true, false);
  else if (a.moe_top) MV_STREAMS(false, true);
  else MV_STREAMS(false, false);
#undef MV_STREAMS
}
template <typename Tag, int S>
int launch_width(const MvStreamArgs &a, int rows, int cols, int cols_true, int run, hipStream_t st) {
  const int threads = (cols / 4 + 63) / 64 * 64;
  if (threads <= 1024) launch<Tag, S, 1>(a, rows, cols, cols_true, run, threads, st);
  else if (threads <= 2048) launch<Tag, S, 4>(a, rows, cols, cols_true, run, (cols / 4 + 255) / 256 * 64, st);
  else return MV_E_SHAPE;   // > 8192 columns
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
