// K19 — gated running mean (include/mvhip.h: MvGruArgs): element by element S <- (1 - z) S + z c, out = S silu(g); fp32 from the
// projections on.
//   prompts: the recurrence is a composition of maps S -> A S + B.  Chunks of a sequence give their (A, B) at once (gru_chunk_kernel);
//            then every chunk composes those ahead of it and walks its own tokens (gru_walk_kernel);
//   decode:  mv_gru_step, one launch per step.
#include "vec4.h"

namespace {

constexpr int kAhead = 8;         // tokens whose operands are requested at a time
constexpr int kMaxChunks = 64;    // of one sequence

// tokens of a chunk: short ones where few would leave the chip idle, long ones where a chunk would have too many ahead of it
int chunk_len(int total_q, int max_q, int n) {
  int len = 64;
  while (len > 16 && (int64_t)(total_q / len) * ((n + 255) / 256) < 1024) len /= 2;
  while ((max_q + len - 1) / len > kMaxChunks) len *= 2;
  return len;
}

// one token: the factor a = 1 - sigmoid(z) and what is added, sigmoid(z) c(u)
template <typename Tag>
__device__ __forceinline__ void operands(float z, float u, float &a, float &b) {
  const float s = sigmoid_of<Tag>(z);
  a = 1.0f - s;
  b = s * (u >= 0.f ? u + 0.5f : sigmoid_of<Tag>(u));
}

// fn(token, z, u) for the tokens t0 .. t1 of a thread's four channels
template <typename Tag, typename Fn>
__device__ __forceinline__ void for_tokens(const typename elem<Tag>::T *z, const typename elem<Tag>::T *u, int64_t stride, int t0, int t1,
                                           const Fn &fn) {
  typedef vec4<Tag> V;
  for (int tb = t0; tb < t1; tb += kAhead) {
    typename V::R rz[kAhead], ru[kAhead];
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      const int64_t at = (int64_t)min(tb + i, t1 - 1) * stride;
      rz[i] = V::raw(z + at), ru[i] = V::raw(u + at);
    }
#pragma unroll
    for (int i = 0; i < kAhead; ++i)
      if (tb + i < t1) fn(tb + i, V::unpack(rz[i]), V::unpack(ru[i]));
  }
}

struct Place {   // of a workgroup: 256 channels of one chunk of one sequence
  int q0, len, before, chunks, chunk, c;
  int64_t slot, entry;   // entry: of the chunk's pair in the workspace; those of a sequence lie one behind the other
  bool held;
  __device__ __forceinline__ Place(const MvGruArgs &p, int chunk_tokens) {
    const int s = blockIdx.z;
    q0 = p.cu_q[s], len = p.cu_q[s + 1] - q0, before = p.cu_k[s + 1] - p.cu_k[s] - len;
    chunks = (len + chunk_tokens - 1) / chunk_tokens, chunk = blockIdx.y;
    c = (blockIdx.x * 64 + threadIdx.x) * 4;
    slot = p.state_slots[s], held = slot >= 0 && slot < p.slots;
    entry = q0 / chunk_tokens + s + chunk;
  }
  __device__ __forceinline__ f32x4 start(const MvGruArgs &p) const {
    if (!held || before <= 0) return f32x4{0.f, 0.f, 0.f, 0.f};
    return *reinterpret_cast<const f32x4 *>(p.state + ((before & 1) * p.slots + slot) * p.n + c);
  }
};

// workspace [entries][2][n]: (A, B) of a chunk; of a sequence's first one: the state ahead of it and behind it
template <typename Tag>
__global__ void __launch_bounds__(64) gru_chunk_kernel(MvGruArgs p, int chunk_tokens) {
  typedef typename elem<Tag>::T T;
  const Place at(p, chunk_tokens);
  if (at.c >= p.n || at.chunk >= at.chunks || (at.chunk > 0 && at.chunk + 1 == at.chunks)) return;
  f32x4 a = {1.f, 1.f, 1.f, 1.f}, b = {0.f, 0.f, 0.f, 0.f};
  if (at.chunk == 0) b = at.start(p);
  float *ws = p.workspace + at.entry * 2 * p.n + at.c;
  if (at.chunk == 0) *reinterpret_cast<f32x4 *>(ws) = b;
  if (at.chunks == 1) return;
  const int64_t base = (int64_t)at.q0 * p.stride + at.c;
  const int t0 = at.chunk * chunk_tokens;
  for_tokens<Tag>((const T *)p.z + base, (const T *)p.u + base, p.stride, t0, t0 + chunk_tokens, [&](int, const f32x4 &z, const f32x4 &u) {
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float f, add;
      operands<Tag>(z[e], u[e], f, add);
      a[e] *= f;
      b[e] = fmaf(f, b[e], add);
    }
  });
  if (at.chunk > 0) *reinterpret_cast<f32x4 *>(ws) = a;
  *reinterpret_cast<f32x4 *>(ws + p.n) = b;
}

template <typename Tag>
__global__ void __launch_bounds__(64) gru_walk_kernel(MvGruArgs p, int chunk_tokens, bool chunked) {
  typedef typename elem<Tag>::T T;
  typedef vec4<Tag> V;
  const Place at(p, chunk_tokens);
  if (at.c >= p.n || at.chunk >= at.chunks) return;
  f32x4 s;
  if (!chunked) {
    s = at.start(p);
  } else {
    const float *ws = p.workspace + (at.entry - at.chunk) * 2 * p.n + at.c;
    s = *reinterpret_cast<const f32x4 *>(at.chunk == 0 ? ws : ws + p.n);
    for (int j0 = 1; j0 < at.chunk; j0 += kAhead) {
      f32x4 a[kAhead], b[kAhead];
#pragma unroll
      for (int i = 0; i < kAhead; ++i) {
        const float *e = ws + (int64_t)min(j0 + i, at.chunk - 1) * 2 * p.n;
        a[i] = *reinterpret_cast<const f32x4 *>(e), b[i] = *reinterpret_cast<const f32x4 *>(e + p.n);
      }
#pragma unroll
      for (int i = 0; i < kAhead; ++i)
        if (j0 + i < at.chunk) {
#pragma unroll
          for (int e = 0; e < 4; ++e) s[e] = fmaf(a[i][e], s[e], b[i][e]);
        }
    }
  }
  const int64_t base = (int64_t)at.q0 * p.stride + at.c;
  const int t0 = at.chunk * chunk_tokens, t1 = min(at.len, t0 + chunk_tokens);
  const T *z = (const T *)p.z + base, *u = (const T *)p.u + base, *g = (const T *)p.g + base;
  T *out = (T *)p.out + (int64_t)at.q0 * p.out_stride + at.c;
  for (int tb = t0; tb < t1; tb += kAhead) {
    typename V::R rz[kAhead], ru[kAhead], rg[kAhead];
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      const int64_t row = (int64_t)min(tb + i, t1 - 1) * p.stride;
      rz[i] = V::raw(z + row), ru[i] = V::raw(u + row), rg[i] = V::raw(g + row);
    }
#pragma unroll
    for (int i = 0; i < kAhead; ++i) {
      if (tb + i >= t1) continue;
      const f32x4 zf = V::unpack(rz[i]), uf = V::unpack(ru[i]), gf = V::unpack(rg[i]);
      f32x4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        float f, add;
        operands<Tag>(zf[e], uf[e], f, add);
        s[e] = fmaf(f, s[e], add);
        o[e] = s[e] * gf[e] * sigmoid_of<Tag>(gf[e]);
      }
      V::store(out + (int64_t)(tb + i) * p.out_stride, o);
    }
  }
  if (at.held && at.chunk + 1 == at.chunks)
    *reinterpret_cast<f32x4 *>(p.state + (((at.before + at.len) & 1) * p.slots + at.slot) * p.n + at.c) = s;
}

template <typename Tag>
__global__ void __launch_bounds__(256) gru_step_kernel(MvGruArgs p) {
  typedef typename elem<Tag>::T T;
  typedef vec4<Tag> V;
  const int c = (blockIdx.x * 256 + threadIdx.x) * 4, row = blockIdx.y;
  if (c >= p.n) return;
  const int before = p.context_lens[row] - 1, slot = p.state_slots[row];
  f32x4 s = {0.f, 0.f, 0.f, 0.f}, o = s;
  if (before >= 0) {
    const bool held = slot >= 0 && slot < p.slots;
    const int64_t at = (int64_t)row * p.stride + c;
    if (held && before > 0) s = *reinterpret_cast<const f32x4 *>(p.state + ((before & 1) * p.slots + slot) * p.n + c);
    const f32x4 z = V::load((const T *)p.z + at), u = V::load((const T *)p.u + at), g = V::load((const T *)p.g + at);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      float f, add;
      operands<Tag>(z[e], u[e], f, add);
      s[e] = fmaf(f, s[e], add);
      o[e] = s[e] * g[e] * sigmoid_of<Tag>(g[e]);
    }
    if (held) *reinterpret_cast<f32x4 *>(p.state + (((before + 1) & 1) * p.slots + slot) * p.n + c) = s;
  }
  V::store((T *)p.out + (int64_t)row * p.out_stride + c, o);
}

int check(const MvGruArgs *a, int dtype) {
  if (!a || !a->z || !a->u || !a->g || !a->out || !a->state_slots || (a->slots > 0 && !a->state)) return MV_E_NULLPTR;
  if (dtype != MV_BF16 && dtype != MV_F16 && dtype != MV_F32) return MV_E_DTYPE;
  if (a->n_seqs < 0 || a->n_seqs > 65535 || a->n <= 0 || (a->n & 7) || a->slots < 0 || a->stride < a->n || a->out_stride < a->n)
    return MV_E_SHAPE;
  if (!mv_aligned16(a->z) || !mv_aligned16(a->u) || !mv_aligned16(a->g) || !mv_aligned16(a->out) ||
      (a->state && !mv_aligned16(a->state)) || (a->stride & 7) || (a->out_stride & 7))
    return MV_E_ALIGN;
  return MV_OK;
}

}  // namespace

extern "C" size_t mv_gru_prefill_workspace_bytes(int n_seqs, int total_q, int max_q, int n) {
  if (n_seqs <= 0 || total_q <= 0 || max_q <= 0 || n <= 0) return 0;
  const int len = chunk_len(total_q, max_q, n);
  return max_q <= len ? 0 : (size_t)(total_q / len + n_seqs) * 2 * n * sizeof(float);
}

extern "C" int mv_gru_prefill(const MvGruArgs *a, int dtype, void *stream) {
  if (a && (a->n_seqs == 0 || a->max_q == 0)) return MV_OK;
  if (int e = check(a, dtype)) return e;
  if (!a->cu_q || !a->cu_k) return MV_E_NULLPTR;
  if (a->max_q < 0 || a->total_q < a->max_q) return MV_E_SHAPE;
  const size_t need = mv_gru_prefill_workspace_bytes(a->n_seqs, a->total_q, a->max_q, a->n);
  if (need && (!a->workspace || !mv_aligned16(a->workspace) || a->ws_bytes < (int64_t)need)) return MV_E_WORKSPACE;
  const int len = chunk_len(a->total_q, a->max_q, a->n);
  const dim3 grid((a->n + 255) / 256, (a->max_q + len - 1) / len, a->n_seqs);
  hipStream_t st = (hipStream_t)stream;
  MV_DISPATCH_DTYPE(dtype, {
    if (need) hipLaunchKernelGGL((gru_chunk_kernel<Tag>), grid, dim3(64), 0, st, *a, len);
    hipLaunchKernelGGL((gru_walk_kernel<Tag>), grid, dim3(64), 0, st, *a, len, need != 0);
  });
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_gru_step(const MvGruArgs *a, int dtype, void *stream) {
  if (a && a->n_seqs == 0) return MV_OK;
  if (int e = check(a, dtype)) return e;
  if (!a->context_lens) return MV_E_NULLPTR;
  const dim3 grid((a->n / 4 + 255) / 256, a->n_seqs);
  MV_DISPATCH_DTYPE(dtype, hipLaunchKernelGGL((gru_step_kernel<Tag>), grid, dim3(256), 0, (hipStream_t)stream, *a));
  MV_LAUNCH_CHECK();
  return MV_OK;
}
