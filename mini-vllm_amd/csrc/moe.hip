// K17 — mixture of experts (include/mvhip.h): router, grouping of (token, choice) pairs by expert, products over the groups.
//   mv_moe_route:  logits, softmax, choice by groups, weights; 16 tokens per workgroup;
//   mv_moe_group:  pairs sorted by expert, and the tiles of at most tile_m rows of one expert each;
//   mv_moe_linear: out[place] = W[expert of the place] x[token of the place], with the gate's activation if asked for.
// The weighted sum over a token's choices rides in mv_residual_update.
#include "latent.h"

namespace {

// ---- router ------------------------------------------------------------------------------------------------------------
struct RouteParams {
  const void *x, *w, *correction;
  int32_t *ids;
  float *weights;
  int64_t x_stride;
  int rows, k, outputs, top, groups, keep, flags;
  float scale;
};
constexpr int kRouteTokens = 16, kRouteWaves = 8, kRouteTiles = 4;   // kRouteTiles: tiles of 16 outputs at a time

// largest value of the wave and the lowest index that has it
__device__ __forceinline__ void wave_argmax(float &v, int &i) {
#pragma unroll
  for (int o = 32; o >= 1; o >>= 1) {
    const float u = __shfl_xor(v, o, 64);
    const int j = __shfl_xor(i, o, 64);
    if (u > v || (u == v && j < i)) v = u, i = j;
  }
}

template <typename Tag>
__global__ void __launch_bounds__(kRouteWaves * 64) moe_route_kernel(RouteParams p) {
  typedef typename elem<Tag>::T T;
  extern __shared__ float lds[];   // scores [16][outputs] | choice scores [16][outputs] | (16-bit) partial tiles
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, m0 = blockIdx.x * kRouteTokens, R = p.outputs;
  float *sc = lds, *ch = sc + kRouteTokens * R;
  const T *x = (const T *)p.x, *w = (const T *)p.w;
  if constexpr (__is_same(Tag, f32_tag)) {
    const int l = tid & 15;
    for (int i = tid >> 4; i < kRouteTokens * R; i += kRouteWaves * 4) {
      const int t = i / R, r = i - t * R;
      const T *xr = x + (int64_t)min(m0 + t, p.rows - 1) * p.x_stride, *wr = w + (int64_t)r * p.k;
      float z = 0.f;
      for (int k = l; k < p.k; k += 16) z = fmaf(xr[k], wr[k], z);
      z = row16_sum(z);
      if (l == 0) sc[i] = z;
    }
  } else {
    f32x4 *part = (f32x4 *)(ch + kRouteTokens * R);   // [waves][kRouteTiles][64]
    const int r16 = lane & 15, g = lane >> 4, steps = p.k / 32;
    const T *xr = x + (int64_t)min(m0 + r16, p.rows - 1) * p.x_stride + g * 8;
    for (int rt = 0; rt * 16 < R; rt += kRouteTiles) {
      const T *wr[kRouteTiles];
#pragma unroll
      for (int j = 0; j < kRouteTiles; ++j) wr[j] = w + (int64_t)min((rt + j) * 16 + r16, R - 1) * p.k + g * 8;
      f32x4 acc[kRouteTiles] = {};
      for (int s = wave; s < steps; s += kRouteWaves) {
        const u32x4 b = *(const u32x4 *)(xr + s * 32);
        u32x4 a[kRouteTiles];
#pragma unroll
        for (int j = 0; j < kRouteTiles; ++j) a[j] = *(const u32x4 *)(wr[j] + s * 32);
#pragma unroll
        for (int j = 0; j < kRouteTiles; ++j) acc[j] = mfma16x16x32<Tag>(a[j], b, acc[j]);
      }
#pragma unroll
      for (int j = 0; j < kRouteTiles; ++j) part[(wave * kRouteTiles + j) * 64 + lane] = acc[j];
      __syncthreads();
      if (wave < kRouteTiles) {
        f32x4 z = part[wave * 64 + lane];
#pragma unroll
        for (int v = 1; v < kRouteWaves; ++v) z += part[(v * kRouteTiles + wave) * 64 + lane];
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int r = (rt + wave) * 16 + g * 4 + e;
          if (r < R) sc[r16 * R + r] = z[e];
        }
      }
      __syncthreads();
    }
  }
  __syncthreads();
  const int size = R / p.groups;
  for (int t = wave; t < kRouteTokens; t += kRouteWaves) {
    if (m0 + t >= p.rows) break;   // (uniform in the wave; no barrier below)
    float *s = sc + t * R, *c = ch + t * R;
    const bool sigmoid = p.flags & MV_ROUTE_SIGMOID;
    float mx = -INFINITY, sum = 0.f;
    if (!sigmoid) {
      for (int i = lane; i < R; i += 64) mx = fmaxf(mx, s[i]);
      mx = wave_max(mx);
      for (int i = lane; i < R; i += 64) sum += expf(s[i] - mx);
      sum = wave_sum(sum);
    }
    for (int i = lane; i < R; i += 64) {
      const float v = sigmoid ? 1.0f / (1.0f + expf(-s[i])) : expf(s[i] - mx) / sum;
      s[i] = v;
      c[i] = p.correction ? v + elem<Tag>::ld(((const T *)p.correction)[i]) : v;
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    if (p.keep < p.groups) {   // lane = group (at most 64)
      float best = -INFINITY;
      if (lane < p.groups)
        for (int i = 0; i < size; ++i) best = fmaxf(best, c[lane * size + i]);
      bool kept = false;
      for (int k = 0; k < p.keep; ++k) {
        float v = kept || lane >= p.groups ? -INFINITY : best;
        int i = kept || lane >= p.groups ? 1 << 20 : lane;
        wave_argmax(v, i);
        if (i == lane) kept = true;
      }
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      if (lane < p.groups && !kept)
        for (int i = 0; i < size; ++i) c[lane * size + i] = -INFINITY;
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    }
    int mine = 0;
    float weight = 0.f, total = 0.f;
    for (int k = 0; k < p.top; ++k) {
      float v = -INFINITY;
      int at = 1 << 20;
      for (int i = lane; i < R; i += 64)
        if (c[i] > v || at == 1 << 20) v = c[i], at = i;
      wave_argmax(v, at);
      const float chosen = s[at];
      if (lane == k) mine = at, weight = chosen;
      total += chosen;
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
      if (lane == (at & 63)) c[at] = -INFINITY;   // (the lane that looks at it)
      __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    }
    if (lane < p.top) {
      p.ids[(int64_t)(m0 + t) * p.top + lane] = mine;
      p.weights[(int64_t)(m0 + t) * p.top + lane] = (p.flags & MV_ROUTE_RAW ? weight : weight / (total + 1e-20f)) * p.scale;
    }
  }
}

// ---- grouping.  Workgroup e = expert e: its pairs start behind those of the experts before it.  Each wave walks a part of the
// pairs, in order, so places are the same in every run.
constexpr int kGroupThreads = 1024, kGroupWaves = kGroupThreads / 64, kGroupAhead = 8;   // kGroupAhead: choices of a lane requested at a time

__global__ void __launch_bounds__(kGroupThreads) moe_group_kernel(const int32_t *ids, int pairs, int top, int experts, int tile_m,
                                                                  int max_tiles, int32_t *rows, int32_t *tokens, int32_t *tiles,
                                                                  const float *weights, float *weights_out) {
  __shared__ int less[kGroupWaves], equal[kGroupWaves];
  const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int per = (pairs + kGroupWaves * 64 - 1) / (kGroupWaves * 64) * 64, lo = wave * per, hi = min(pairs, lo + per);
  int nl = 0, ne = 0;
  // the choices i0 + 64 u + lane of this wave's part (-1 behind its end)
  auto choices = [&](int i0, int (&v)[kGroupAhead]) {
#pragma unroll
    for (int u = 0; u < kGroupAhead; ++u) {
      const int i = i0 + 64 * u + lane;
      v[u] = ids[min(i, pairs - 1)];
      if (i >= hi) v[u] = -1;
    }
  };
  for (int i0 = lo; i0 < hi; i0 += 64 * kGroupAhead) {
    int v[kGroupAhead];
    choices(i0, v);
#pragma unroll
    for (int u = 0; u < kGroupAhead; ++u) nl += v[u] >= 0 && v[u] < e, ne += v[u] == e;
  }
#pragma unroll
  for (int o = 32; o >= 1; o >>= 1) nl += __shfl_xor(nl, o, 64), ne += __shfl_xor(ne, o, 64);
  if (lane == 0) less[wave] = nl, equal[wave] = ne;
  __syncthreads();
  int start = 0, count = 0, ahead = 0;
  for (int w = 0; w < kGroupWaves; ++w) {
    start += less[w], count += equal[w];
    if (w < wave) ahead += equal[w];
  }
  int at = start + ahead;
  for (int i0 = lo; i0 < hi; i0 += 64 * kGroupAhead) {
    int v[kGroupAhead];
    float w[kGroupAhead];
    choices(i0, v);
#pragma unroll
    for (int u = 0; u < kGroupAhead; ++u)
      if (weights && v[u] == e) w[u] = weights[i0 + 64 * u + lane];
#pragma unroll
    for (int u = 0; u < kGroupAhead; ++u) {
      const int i = i0 + 64 * u + lane;
      const unsigned long long mask = __ballot(v[u] == e);
      if (v[u] == e) {
        const int place = at + __popcll(mask & ((1ull << lane) - 1));
        rows[i] = place, tokens[place] = i / top;
        if (weights) weights_out[place] = w[u];
      }
      if (e == 0 && v[u] >= experts) rows[i] = -1;
      at += __popcll(mask);
    }
  }
  // tiles of this expert: entries start / tile_m + e on, up to the next expert's; the last expert also clears what is left
  const int t0 = start / tile_m + e, t1 = e + 1 < experts ? (start + count) / tile_m + e + 1 : max_tiles;
  for (int t = t0 + tid; t < t1; t += kGroupThreads) {
    const int first = (t - t0) * tile_m;
    tiles[3 * t] = first < count ? e : -1, tiles[3 * t + 1] = start + first, tiles[3 * t + 2] = min(tile_m, count - first);
  }
}

// ---- products over the groups ---------------------------------------------------------------------------------------------
struct MoeLinear {
  const void *x, *w;
  void *out;
  const int32_t *tokens, *tiles;   // tokens NULL: row = place
  const float *in_scale;           // by place; NULL: 1
  int64_t x_stride, out_stride, w_expert;   // w_expert: elements between two experts' weights
  int n, k;                        // outputs (gated: of the product with up), inputs
  MvGateAct act;
};

__device__ __forceinline__ float in_scale_of(const MoeLinear &p, int place) { return p.in_scale ? p.in_scale[place] : 1.0f; }

// few rows per expert: TM tiles of 16 rows, TN of 16 outputs; the waves split the inputs, weight fragments come straight from
// memory in the order they are stored (1 KiB per instruction)
template <typename Tag, int TM, int TN, bool GATED>
__global__ void __launch_bounds__(256) moe_small_kernel(MoeLinear p) {
  typedef typename elem<Tag>::T T;
  constexpr int NA = GATED ? 2 * TN : TN, U = NA + TM >= 6 ? 2 : 4;
  __shared__ f32x4 red[4][NA * TM][64];
  const int32_t *tile = p.tiles + 3 * blockIdx.y;
  const int e = tile[0], m0 = tile[1], live = tile[2];
  if (e < 0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r16 = lane & 15, g = lane >> 4;
  const int steps = p.k / 32, s_lo = steps * wave / 4, s_hi = steps * (wave + 1) / 4, ntiles = p.n / 16;
  const u32x4 *w[NA];
#pragma unroll
  for (int j = 0; j < NA; ++j) {
    const int t = min((int)blockIdx.x * TN + (GATED ? j >> 1 : j), ntiles - 1) + (GATED && (j & 1) ? ntiles : 0);
    w[j] = (const u32x4 *)((const T *)p.w + e * p.w_expert) + (int64_t)t * steps * 64 + lane;
  }
  const T *x[TM];
#pragma unroll
  for (int i = 0; i < TM; ++i) {
    const int place = m0 + min(i * 16 + r16, live - 1);
    x[i] = (const T *)p.x + (int64_t)(p.tokens ? p.tokens[place] : place) * p.x_stride + g * 8;
  }
  f32x4 acc[NA][TM] = {};
  for (int s = s_lo; s < s_hi; s += U) {
    u32x4 a[U][NA], b[U][TM];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int k = min(s + u, s_hi - 1);
#pragma unroll
      for (int j = 0; j < NA; ++j) a[u][j] = __builtin_nontemporal_load(w[j] + k * 64);
#pragma unroll
      for (int i = 0; i < TM; ++i) b[u][i] = *(const u32x4 *)(x[i] + k * 32);
    }
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (s + u < s_hi) {
#pragma unroll
        for (int j = 0; j < NA; ++j)
#pragma unroll
          for (int i = 0; i < TM; ++i) acc[j][i] = mfma16x16x32<Tag>(a[u][j], b[u][i], acc[j][i]);
      }
  }
#pragma unroll
  for (int j = 0; j < NA; ++j)
#pragma unroll
    for (int i = 0; i < TM; ++i) red[wave][j * TM + i][lane] = acc[j][i];
  __syncthreads();
  auto total = [&](int t) { return (red[0][t][lane] + red[1][t][lane]) + (red[2][t][lane] + red[3][t][lane]); };
  for (int t = wave; t < TN * TM; t += 4) {
    const int j = t / TM, i = t - j * TM, row = i * 16 + r16, n0 = ((int)blockIdx.x * TN + j) * 16;
    if (row >= live || n0 >= p.n) continue;
    const float sc = in_scale_of(p, m0 + row);
    f32x4 o;
    if constexpr (GATED) {
      const f32x4 gate = total(2 * j * TM + i) * sc, up = total((2 * j + 1) * TM + i) * sc;
#pragma unroll
      for (int q = 0; q < 4; ++q) o[q] = gated_act<Tag>(gate[q], up[q], p.act);
    } else {
      o = total(t) * sc;
    }
    *(u32x2 *)((T *)p.out + (int64_t)(m0 + row) * p.out_stride + n0 + g * 4) = pack_quad<Tag>(o);
  }
}

// A fragment of 16 rows x 32 inputs that LDS-DMA brings: four adjacent lanes fetch one row's 64 bytes (16 rows in adjacent lanes would be
// 16 cache lines), in an order that spreads the rows' like pieces over the banks.
__device__ __forceinline__ int row_chunk(int lane) { return (lane & 3) ^ ((lane >> 4) & 3); }              // the piece that a lane fetches
__device__ __forceinline__ int row_place(int row, int chunk) { return row * 4 + (chunk ^ ((row >> 2) & 3)); }  // where a piece lies

// many rows: BM x BN per workgroup of 2 x 2 waves, 64 inputs at a time.  Rows and weights reach LDS by DMA as fragments (16 rows x
// 32 inputs, 1 KiB; weights in the order of the lanes); the next 64 inputs land while these are multiplied.
template <typename Tag, int BM, int BN, bool GATED>
__global__ void __launch_bounds__(256, 2) moe_tile_kernel(MoeLinear p) {
  typedef typename elem<Tag>::T T;
  constexpr int MT = BM / 16, NT = BN / 16, WM = MT / 2, WN = NT / 2, PIECES = 2 * (MT + NT), PER = PIECES / 4;
  constexpr int STAGE = PIECES * 1024;
  extern __shared__ __attribute__((aligned(16))) char smem[];   // 2 stages of [rows: MT][2] | [weights: NT][2] fragments
  const int32_t *tile = p.tiles + 3 * blockIdx.y;
  const int e = tile[0], m0 = tile[1], live = tile[2];
  if (e < 0) return;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r16 = lane & 15, g = lane >> 4;
  const int wm = wave & 1, wn = wave >> 1, ntiles = p.n / 16, steps = p.k / 32, nt0 = blockIdx.x * (GATED ? NT / 2 : NT);
  // this wave's pieces: piece = i * 4 + wave = (tile, half of the 64 inputs); a piece's address moves by a constant per trip
  const T *src[PER];
  int64_t step[PER];
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int piece = i * 4 + wave, half = piece & 1, t = piece >> 1;
    if (t < MT) {
      const int place = m0 + min(t * 16 + (lane >> 2), live - 1);
      src[i] = (const T *)p.x + (int64_t)(p.tokens ? p.tokens[place] : place) * p.x_stride + half * 32 + row_chunk(lane) * 8;
      step[i] = 64;
    } else {
      const int j = t - MT, wt = min(nt0 + (GATED ? j >> 1 : j), ntiles - 1) + (GATED && (j & 1) ? ntiles : 0);
      src[i] = (const T *)p.w + e * p.w_expert + ((int64_t)wt * steps + half) * 512 + lane * 8;
      step[i] = 1024;
    }
  }
  auto fetch = [&](int buf) {
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void *)src[i],
                                       (__attribute__((address_space(3))) void *)(smem + buf * STAGE + (i * 4 + wave) * 1024), 16, 0, 0);
      src[i] += step[i];
    }
  };
  f32x4 acc[WN][WM] = {};
  const uint32_t base = lds_address(smem) + lane * 16, rows = lds_address(smem) + row_place(r16, g) * 16;
  const int trips = p.k / 64;
  fetch(0);
  asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
  lds_barrier();
  for (int t = 0; t < trips; ++t) {
    if (t + 1 < trips) fetch((t + 1) & 1);
    const uint32_t at = (t & 1) * STAGE, xa = rows + at + wm * WM * 2048, wa = base + at + (MT + wn * WN) * 2048;
    u32x4 a[2][WN], b[2][WM];
    static_for<2>([&](auto H) {
      constexpr int h = decltype(H)::value;
      static_for<WM>([&](auto I) { lds_read128<decltype(I)::value * 2048 + h * 1024>(b[h][decltype(I)::value], xa); });
      static_for<WN>([&](auto I) { lds_read128<decltype(I)::value * 2048 + h * 1024>(a[h][decltype(I)::value], wa); });
    });
    static_for<2>([&](auto H) {
      constexpr int h = decltype(H)::value;
      static_for<WM>([&](auto I) { lds_wait<h == 0 ? WM + WN : 0>(b[h][decltype(I)::value]); });
      static_for<WN>([&](auto I) { lds_wait<h == 0 ? WM + WN : 0>(a[h][decltype(I)::value]); });
#pragma unroll
      for (int j = 0; j < WN; ++j)
#pragma unroll
        for (int i = 0; i < WM; ++i) acc[j][i] = mfma16x16x32<Tag>(a[h][j], b[h][i], acc[j][i]);
    });
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    lds_barrier();
  }
#pragma unroll
  for (int i = 0; i < WM; ++i) {
    const int row = (wm * WM + i) * 16 + r16;
    if (row >= live) continue;
    const float sc = in_scale_of(p, m0 + row);
    T *out = (T *)p.out + (int64_t)(m0 + row) * p.out_stride + g * 4;
#pragma unroll
    for (int j = 0; j < (GATED ? WN / 2 : WN); ++j) {
      const int nt = nt0 + (GATED ? wn * (WN / 2) + j : wn * WN + j);
      if (nt >= ntiles) continue;
      f32x4 o;
      if constexpr (GATED) {
#pragma unroll
        for (int q = 0; q < 4; ++q) o[q] = gated_act<Tag>(acc[2 * j][i][q] * sc, acc[2 * j + 1][i][q] * sc, p.act);
      } else {
        o = acc[j][i] * sc;
      }
      *(u32x2 *)(out + nt * 16) = pack_quad<Tag>(o);
    }
  }
}

// very many rows: 256 x 256 per workgroup of 2 x 4 waves, so that a row operand read from LDS serves four products and a weight operand
// eight.  Two stages of 64 inputs; a stage is handed back half way through its products, when all of it is in registers.
template <typename Tag, bool GATED>
__global__ void __launch_bounds__(512, 1) moe_wide_kernel(MoeLinear p, int nx, int max_tiles) {
  typedef typename elem<Tag>::T T;
  constexpr int TILES = 16, WM = 8, WN = 4, PER = 4, STAGE = 4 * TILES * 1024;
  extern __shared__ __attribute__((aligned(16))) char smem[];   // 2 stages of [rows: TILES][2] | [weights: TILES][2] fragments
  // Workgroups are dealt to the XCDs in turn: four row tiles and all their outputs stay on one of them, the row tiles first.
  const int xcd = blockIdx.x & 7, turn = blockIdx.x >> 3, group = turn / (4 * nx) * 8 + xcd, in = turn % (4 * nx);
  const int ty = group * 4 + (in & 3), tx = in >> 2;
  if (ty >= max_tiles) return;
  const int32_t *tile = p.tiles + 3 * ty;
  const int e = tile[0], m0 = tile[1], live = tile[2];
  if (e < 0) return;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), r16 = lane & 15, g = lane >> 4;
  const int wm = wave & 1, wn = wave >> 1, ntiles = p.n / 16, steps = p.k / 32, nt0 = tx * (GATED ? TILES / 2 : TILES);
  // this wave's fragments: one half of the 64 inputs of every fourth tile, of the rows and of the weights
  const int half = wave & 1, first = wave >> 1;
  const T *xs[PER], *ws[PER];
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int j = 4 * i + first, place = m0 + min(j * 16 + (lane >> 2), live - 1);
    xs[i] = (const T *)p.x + (int64_t)(p.tokens ? p.tokens[place] : place) * p.x_stride + half * 32 + row_chunk(lane) * 8;
    const int wt = min(nt0 + (GATED ? j >> 1 : j), ntiles - 1) + (GATED && (j & 1) ? ntiles : 0);
    ws[i] = (const T *)p.w + e * p.w_expert + ((int64_t)wt * steps + half) * 512;
  }
  const int lane8 = lane * 8;
  auto fetch = [&](int t) {
    char *to = smem + (t & 1) * STAGE + (first * 2 + half) * 1024;
    const int64_t kx = (int64_t)t * 64, kw = (int64_t)t * 1024;
#pragma unroll
    for (int i = 0; i < PER; ++i) {
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void *)(xs[i] + kx),
                                       (__attribute__((address_space(3))) void *)(to + i * 8192), 16, 0, 0);
      __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void *)(ws[i] + kw + lane8),
                                       (__attribute__((address_space(3))) void *)(to + (TILES * 2048) + i * 8192), 16, 0, 0);
    }
  };
  f32x4 acc[WN][WM] = {};
  const uint32_t base = lds_address(smem) + lane * 16, rows = lds_address(smem) + row_place(r16, g) * 16;
  const int trips = p.k / 64;
  fetch(0);
  asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
  lds_barrier();
  if (trips > 1) fetch(1);
  for (int t = 0; t < trips; ++t) {
    const uint32_t at = (t & 1) * STAGE, xa = rows + at + wm * WM * 2048, wa = base + at + (TILES + wn * WN) * 2048;
    u32x4 a[2][WN], b[2][WM];
    static_for<2>([&](auto H) {
      constexpr int h = decltype(H)::value;
      static_for<WN>([&](auto I) { lds_read128<decltype(I)::value * 2048 + h * 1024>(a[h][decltype(I)::value], wa); });
      static_for<WM>([&](auto I) { lds_read128<decltype(I)::value * 2048 + h * 1024>(b[h][decltype(I)::value], xa); });
    });
    static_for<2>([&](auto H) {
      constexpr int h = decltype(H)::value;
      static_for<WN>([&](auto I) { lds_wait<h == 0 ? WM + WN : 0>(a[h][decltype(I)::value]); });
      static_for<WM>([&](auto I) { lds_wait<h == 0 ? WM + WN : 0>(b[h][decltype(I)::value]); });
      if (h == 1 && t + 1 < trips) {   // every wave has read this stage; the next has landed
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        lds_barrier();
        if (t + 2 < trips) fetch(t + 2);
      }
#pragma unroll
      for (int i = 0; i < WM; ++i)
#pragma unroll
        for (int j = 0; j < WN; ++j) acc[j][i] = mfma16x16x32<Tag>(a[h][j], b[h][i], acc[j][i]);
    });
  }
#pragma unroll
  for (int i = 0; i < WM; ++i) {
    const int row = (wm * WM + i) * 16 + r16;
    if (row >= live) continue;
    const float sc = in_scale_of(p, m0 + row);
    T *out = (T *)p.out + (int64_t)(m0 + row) * p.out_stride + g * 4;
#pragma unroll
    for (int j = 0; j < (GATED ? WN / 2 : WN); ++j) {
      const int nt = nt0 + (GATED ? wn * (WN / 2) + j : wn * WN + j);
      if (nt >= ntiles) continue;
      f32x4 o;
      if constexpr (GATED) {
#pragma unroll
        for (int q = 0; q < 4; ++q) o[q] = gated_act<Tag>(acc[2 * j][i][q] * sc, acc[2 * j + 1][i][q] * sc, p.act);
      } else {
        o = acc[j][i] * sc;
      }
      *(u32x2 *)(out + nt * 16) = pack_quad<Tag>(o);
    }
  }
}

// fp32: 16 rows x 64 outputs per workgroup, weights [expert][outputs (gate | up)][inputs]
template <bool GATED>
__global__ void __launch_bounds__(256) moe_f32_kernel(MoeLinear p) {
  constexpr int K = 32, NW = GATED ? 128 : 64;
  __shared__ float xs[16][K + 1], ws[NW][K + 1];
  const int32_t *tile = p.tiles + 3 * blockIdx.y;
  const int e = tile[0], m0 = tile[1], live = tile[2], tid = threadIdx.x, n0 = blockIdx.x * 64;
  if (e < 0) return;
  const float *w = (const float *)p.w + e * p.w_expert;
  const int c = tid & 63, r = tid >> 6;   // column; rows r, r + 4, ...
  float acc[4] = {}, up[4] = {};
  for (int k0 = 0; k0 < p.k; k0 += K) {
    __syncthreads();
    for (int i = tid; i < 16 * K; i += 256) {
      const int t = i / K, k = i - t * K, place = m0 + min(t, live - 1);
      xs[t][k] = ((const float *)p.x)[(int64_t)(p.tokens ? p.tokens[place] : place) * p.x_stride + k0 + k];
    }
    for (int i = tid; i < NW * K; i += 256) {
      const int j = i / K, k = i - j * K, n = min(n0 + (j & 63), p.n - 1) + (j >= 64 ? p.n : 0);
      ws[j][k] = w[(int64_t)n * p.k + k0 + k];
    }
    __syncthreads();
    for (int k = 0; k < K; ++k)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        acc[i] = fmaf(xs[r + 4 * i][k], ws[c][k], acc[i]);
        if constexpr (GATED) up[i] = fmaf(xs[r + 4 * i][k], ws[64 + c][k], up[i]);
      }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (r + 4 * i < live && n0 + c < p.n) {
      const float sc = in_scale_of(p, m0 + r + 4 * i);
      ((float *)p.out)[(int64_t)(m0 + r + 4 * i) * p.out_stride + n0 + c] = GATED ? gated_act<f32_tag>(acc[i] * sc, up[i] * sc, p.act) : acc[i] * sc;
    }
}

template <typename Tag, bool GATED>
int launch_linear(const MoeLinear &p, int tile_m, int max_tiles, hipStream_t st) {
  const int nt = p.n / 16;
  constexpr int TN = GATED ? 1 : 2;
  const dim3 small((nt + TN - 1) / TN, max_tiles);
  if (tile_m == 16) hipLaunchKernelGGL((moe_small_kernel<Tag, 1, TN, GATED>), small, dim3(256), 0, st, p);
  else if (tile_m == 32) hipLaunchKernelGGL((moe_small_kernel<Tag, 2, TN, GATED>), small, dim3(256), 0, st, p);
  else if (tile_m == 64 || tile_m == 128) {
    constexpr int BN = 128;
    const dim3 grid((nt * 16 * (GATED ? 2 : 1) + BN - 1) / BN, max_tiles);
    if (tile_m == 64) hipLaunchKernelGGL((moe_tile_kernel<Tag, 64, BN, GATED>), grid, dim3(256), (64 + BN) * 256, st, p);
    else hipLaunchKernelGGL((moe_tile_kernel<Tag, 128, BN, GATED>), grid, dim3(256), (128 + BN) * 256, st, p);
  } else if (tile_m == 256) {
    const int nx = (nt * (GATED ? 2 : 1) + 15) / 16, groups = (max_tiles + 3) / 4;
    if (int rc = mv_allow_lds<moe_wide_kernel<Tag, GATED>>()) return rc;
    hipLaunchKernelGGL((moe_wide_kernel<Tag, GATED>), dim3((unsigned)((groups + 7) / 8 * 8) * 4u * nx), dim3(512), 128 * 1024, st, p, nx, max_tiles);
  } else {
    return MV_E_SHAPE;
  }
  MV_LAUNCH_CHECK();
  return MV_OK;
}

}  // namespace

extern "C" int mv_moe_route(const void *x, int64_t x_stride, const void *w, const void *correction, int32_t *ids, float *weights,
                            int rows, int k, int outputs, int top, int groups, int keep, float scale, int flags, int dtype, void *stream) {
  if (rows == 0) return MV_OK;
  if (!x || !w || !ids || !weights) return MV_E_NULLPTR;
  if (flags & ~(MV_ROUTE_SIGMOID | MV_ROUTE_RAW)) return MV_E_RANGE;
  if (rows < 0 || k <= 0 || (k & 31) || outputs <= 0 || outputs > 512 || top <= 0 || top > 64 || top > outputs || groups <= 0 ||
      groups > 64 || outputs % groups || keep <= 0 || keep > groups || (int64_t)outputs / groups * keep < top || x_stride < k)
    return MV_E_SHAPE;
  if (!mv_aligned16(x) || !mv_aligned16(w) || x_stride % (dtype == MV_F32 ? 4 : 8)) return MV_E_ALIGN;
  const RouteParams p{x, w, correction, ids, weights, x_stride, rows, k, outputs, top, groups, keep, flags, scale};
  const size_t lds = (size_t)2 * kRouteTokens * outputs * 4 + (dtype == MV_F32 ? 0 : kRouteWaves * kRouteTiles * 1024);
  const dim3 grid((rows + kRouteTokens - 1) / kRouteTokens);
  MV_DISPATCH_DTYPE(dtype, {
    if (int rc = mv_allow_lds<moe_route_kernel<Tag>>()) return rc;
    hipLaunchKernelGGL((moe_route_kernel<Tag>), grid, dim3(kRouteWaves * 64), lds, (hipStream_t)stream, p);
  });
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_moe_group(const int32_t *ids, int pairs, int top, int experts, int tile_m, int max_tiles, int32_t *rows,
                            int32_t *tokens, int32_t *tiles, const float *weights, float *weights_out, void *stream) {
  if (pairs == 0) return MV_OK;
  if (!ids || !rows || !tokens || !tiles || (weights && !weights_out)) return MV_E_NULLPTR;
  if (pairs < 0 || top <= 0 || experts <= 0 || experts > 65535 || tile_m <= 0 || max_tiles < pairs / tile_m + experts) return MV_E_SHAPE;
  hipLaunchKernelGGL(moe_group_kernel, dim3(experts), dim3(kGroupThreads), 0, (hipStream_t)stream, ids, pairs, top, experts, tile_m,
                     max_tiles, rows, tokens, tiles, weights, weights_out);
  MV_LAUNCH_CHECK();
  return MV_OK;
}

extern "C" int mv_moe_linear(const MvMoeLinearArgs *a, int dtype, void *stream) {
  if (!a || !a->x || !a->w || !a->out || !a->tiles) return MV_E_NULLPTR;
  if (dtype != MV_BF16 && dtype != MV_F16 && dtype != MV_F32) return MV_E_DTYPE;
  if (a->max_tiles <= 0) return a->max_tiles == 0 ? MV_OK : MV_E_SHAPE;
  if (a->max_tiles > 65535 || a->n <= 0 || a->k <= 0 || (a->k & 63) || (a->n & 15) || a->x_stride < a->k || a->out_stride < a->n)
    return MV_E_SHAPE;
  const int vec = dtype == MV_F32 ? 4 : 8;
  if (!mv_aligned16(a->x) || !mv_aligned16(a->w) || !mv_aligned16(a->out) || a->x_stride % vec || a->out_stride % vec) return MV_E_ALIGN;
  MoeLinear p{a->x, a->w, a->out, a->tokens, a->tiles, a->in_scale, a->x_stride, a->out_stride, (int64_t)a->n * a->k * (a->act ? 2 : 1), a->n, a->k, {}};
  if (a->act) {
    if (int e = mv_check_act(a->act)) return e;
    p.act = *a->act;
  }
  hipStream_t st = (hipStream_t)stream;
  if (dtype == MV_F32) {
    if (a->tile_m != 16) return MV_E_SHAPE;
    const dim3 grid((a->n + 63) / 64, a->max_tiles);
    if (a->act) hipLaunchKernelGGL((moe_f32_kernel<true>), grid, dim3(256), 0, st, p);
    else hipLaunchKernelGGL((moe_f32_kernel<false>), grid, dim3(256), 0, st, p);
    MV_LAUNCH_CHECK();
    return MV_OK;
  }
  if (dtype == MV_BF16) return a->act ? launch_linear<bf16_tag, true>(p, a->tile_m, a->max_tiles, st) : launch_linear<bf16_tag, false>(p, a->tile_m, a->max_tiles, st);
  return a->act ? launch_linear<f16_tag, true>(p, a->tile_m, a->max_tiles, st) : launch_linear<f16_tag, false>(p, a->tile_m, a->max_tiles, st);
}
