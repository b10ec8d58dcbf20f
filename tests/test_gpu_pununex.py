"""Pununex on the GPU: each mechanism's kernel against the plain statement of it, whole models through the engine in every way a
sequence can be cut, batched, paged and given a state slot, and greedy generation through the public entry point."""
import functools

import pytest
import torch

from oracle import pununex as P
from oracle.kugulorn import causal_conv, silu, softplus
from oracle.mofarax import rms
from pununex_configs import CONFIGS, sharp_weights, write_checkpoint

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(scope="module")
def H():
    from minivllm_amd import hip_ops
    return hip_ops


def _close(got, want, dtype, what="", factor=1.0):
    scale = max(want.abs().max().item(), 1e-6)
    err = (got.double().cpu() - want.double()).abs().max().item()
    tol = (2e-5 if dtype == torch.float32 else 1e-2) * factor
    assert err <= tol * scale, f"{what}: {err:.3e} of {scale:.3e}"


def _rand(*shape, dtype=torch.float32, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)).to(dtype)


def _ints(hi, n, seed):
    return torch.randint(0, hi, (n,), generator=torch.Generator().manual_seed(seed))


def _cu(lens):
    return torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32, device=DEV)


def _i32(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


# ---- residual stream, gate ----------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cols, true, splits", [(256, 200, 0), (256, 256, 3), (64, 40, 0), (4160, 4100, 0)])
def test_layer_norms_around_the_stream(H, dtype, cols, true, splits):
    rows, eps = 5, 1e-3
    pad = lambda t: torch.nn.functional.pad(t, (0, cols - true))
    mk = lambda *s, seed: pad(_rand(*s, seed=seed) + 0.7).to(dtype)       # (a mean that matters)
    wy, by, sc, wn, bn = (mk(true, seed=i) for i in (2, 3, 4, 5, 6))
    x0 = pad(_rand(rows, true, seed=7) - 0.4)
    y = pad(_rand(splits, rows, true, seed=1)) if splits else mk(rows, true, seed=1)
    total = (y.double().sum(0) if splits else y.double())[:, :true]
    x, d = x0.clone().to(DEV), lambda t: t.to(DEV)
    out = H.residual_update(x, y=d(y), y_norm_w=d(wy), y_norm_b=d(by), y_scale=d(sc), norm_w=d(wn), norm_b=d(bn), eps=eps, cols_true=true,
                            layer_norm=True)
    t = lambda v: v.double()[:true]
    want = x0.double()[:, :true] + t(sc) * P.layer_norm(total, t(wy), t(by), eps)
    _close(x[:, :true], want, torch.float32, "stream")
    _close(out[:, :true], P.layer_norm(want, t(wn), t(bn), eps), dtype, "norm")
    assert x[:, true:].abs().sum() == 0 and out[:, true:].abs().sum() == 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("with_y", [True, False])
def test_weighted_expert_rows_join_the_stream(H, dtype, with_y):
    rows, cols, top = 9, 128, 3
    x0, eo, w = _rand(rows, cols, seed=1), _rand(20, cols, dtype=dtype, seed=2), _rand(rows, top, seed=3)
    place = _ints(20, rows * top, 4).int()
    place[[2, 7, 8]] = -1                                                 # the stream itself, before the update
    y, nw, nb = _rand(rows, cols, dtype=dtype, seed=5), _rand(cols, dtype=dtype, seed=6), _rand(cols, dtype=dtype, seed=7)
    x = x0.clone().to(DEV)
    H.residual_update(x, y=y.to(DEV) if with_y else None, y_norm_w=nw.to(DEV), y_norm_b=nb.to(DEV), layer_norm=True, eps=1e-4,
                      experts=(eo.to(DEV), place.to(DEV), w.to(DEV)), dtype=dtype)
    total = y.double() if with_y else torch.zeros(rows, cols, dtype=torch.float64)
    for t in range(rows):
        for k in range(top):
            i = int(place[t * top + k])
            total[t] += w[t, k].double() * (eo[i].double() if i >= 0 else x0[t].double())
    _close(x, x0.double() + P.layer_norm(total, nw.double(), nb.double(), 1e-4), torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("buckets, mp, mc", [(97, 13, 7), (1, 0, 1), (509, 100003, 31)])
def test_pair_rows_follow_the_sequence_through_portions_and_steps(H, dtype, buckets, mp, mc):
    """Token by token, in portions beside other sequences, over slots that another sequence used, and a step that runs twice."""
    V, cols = 50, 64
    E, B = _rand(V, cols, dtype=dtype, seed=1), _rand(buckets + 1, cols, dtype=dtype, seed=2)
    prev = torch.full((2, 3), 1 << 20, dtype=torch.int32, device=DEV)
    a, b = _ints(V, 12, 3).tolist(), _ints(V, 6, 4).tolist()

    def run(parts, decode=False):
        """parts: [(tokens, start, stop, slot)]"""
        ids = torch.tensor([t for toks, lo, hi, _ in parts for t in toks[lo:hi]], device=DEV)
        pos = torch.tensor([i for _, lo, hi, _ in parts for i in range(lo, hi)], device=DEV)
        x = torch.empty(ids.numel(), cols, device=DEV)
        H.residual_update(x, embed=E.to(DEV), ids=ids, start=True, want_out=False, pairs=H.PairTable(
            B.to(DEV), mp, mc, pos, prev, _i32([s for *_, s in parts]), None if decode else _cu([hi - lo for _, lo, hi, _ in parts])))
        want = torch.cat([(E.double()[toks] + B.double()[P.bigram_rows(toks, buckets, mp, mc)])[lo:hi] for toks, lo, hi, _ in parts])
        _close(x, want, torch.float32, f"{[p[1:] for p in parts]}")
    run([(a, 0, 12, 0), (b, 0, 6, -1)])
    run([(b, 0, 2, 0), (a, 0, 5, 2)])                                     # slot 0 starts again
    run([(a, 5, 6, 2)], decode=True)
    run([(a, 6, 7, 2), (b, 2, 3, 0)], decode=True)
    run([(a, 6, 7, 2), (b, 2, 3, 0)], decode=True)                        # again
    run([(b, 3, 4, 0), (a, 7, 9, 2)])                                     # a decoded row ahead of a portion
    run([(a, 9, 12, 2), (b, 4, 6, 0)])


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
def test_relu_gate(H, dtype):
    x = _rand(11, 336, dtype=dtype, seed=1)
    want = torch.relu(x.double()[:, :168]) * x.double()[:, 168:]
    _close(H.act_and_mul(x.to(DEV), H.RELU_GLU), want, dtype)


@pytest.mark.parametrize("m, inter, k", [(1, 80, 256), (16, 64, 512), (33, 208, 192)])
def test_relu_gate_in_the_epilogue_of_the_gated_projection(H, m, inter, k):
    dtype = torch.bfloat16
    x, w = _rand(m, k, dtype=dtype, seed=1), (_rand(2 * inter, k, seed=2) * k ** -0.5).to(dtype)
    y = x.double() @ w.double().T
    want, wp = torch.relu(y[:, :inter]) * y[:, inter:], H.pack_weight(w.to(DEV))
    if k >= 256:
        _close(H.gate_up_silu_small_m(x.to(DEV), w.to(DEV), packed=wp, act=H.RELU_GLU), want, dtype)
    _close(H.gate_up_silu_mid_m(x.to(DEV), wp, inter, 0, act=H.RELU_GLU), want, dtype)


# ---- attention ------------------------------------------------------------------------------------------------------------
MASKS = [(0, 0, 0.0), (1, 0, 3.0), (1, 2, 0.0), (33, 4, 30.0), (64, 64, 0.0), (65, 1, 4.0), (130, 70, 8.0)]      # window, kept, cap


def _aimed(nq, k, window, keep, seed):
    """Queries of the last nq of len(k) tokens that point hard at the key just outside their window, the one just inside it, the last
    kept one, the one behind it and the first: a mask that is one off answers with another key's value."""
    nk, dim = k.shape
    q = _rand(nk, dim, seed=seed) * 0.3
    w = window or nk
    for i in range(nk):
        for j in (i - w, i - w + 1, keep - 1, keep, 0):
            if 0 <= j <= i:
                q[i] += 4 * k[j] / k[j].norm()
    return q[nk - nq:]


def _case(nq, nk, heads, kv, dim, vdim, window, keep, dtype, seed):
    k, v = _rand(nk, kv, dim, seed=seed), _rand(nk, kv, vdim, seed=seed + 1)
    q = torch.stack([_aimed(nq, k[:, h * kv // heads], window, keep, seed + 2 + h) for h in range(heads)], 1)
    return q.to(dtype), k.to(dtype), v.to(dtype)


def _attend(q, k, v, scale, cap, sink, window, keep):
    nq, nk = q.shape[0], k.shape[0]
    full = torch.zeros(nk, *q.shape[1:], dtype=torch.float64)
    full[nk - nq:] = q.double()
    return P.sink_attention(full, k.double(), v.double(), scale, cap or None, sink.double(), P.window_mask(nk, window or None, keep))[nk - nq:]


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("heads, kv, d", [(3, 1, 64), (2, 2, 128), (2, 1, 256)])
@pytest.mark.parametrize("window, keep, cap", MASKS, ids=str)
def test_prefill_attention(H, dtype, heads, kv, d, window, keep, cap):
    """Whole sequences and portions (the last queries of a sequence), several in one launch; keys packed and from pages."""
    scale, factor = 0.4, 0.7
    sink = (_rand(heads, seed=3) * 2).to(dtype)
    spans = [(150, 150), (2, 97), (70, 300), (1, 1), (1, 66)]
    cases = [_case(a, b, heads, kv, d, d, window, keep, dtype, 10 * i) for i, (a, b) in enumerate(spans)]
    want = torch.cat([_attend(q, k, v, scale, cap, sink, window, keep) for q, k, v in cases]) * factor
    q, k, v = (torch.cat([c[i] for c in cases]).to(DEV) for i in range(3))
    mask = H.AttnMask(window, keep, cap, factor, sink.to(DEV))
    cq, ck, mq, mk = _cu([a for a, _ in spans]), _cu([b for _, b in spans]), 150, 300
    wide = torch.zeros(q.shape[0], heads * d + 64, dtype=dtype, device=DEV)
    got = H.prefill_varlen(q, k, v, cq, ck, mq, mk, scale, mask=mask, out=wide[:, :heads * d].view(-1, heads, d))
    _close(got, want, dtype, "packed", factor=2.0)
    assert wide[:, heads * d:].abs().sum() == 0
    nb = 5
    pages = torch.randperm(len(spans) * nb, generator=torch.Generator().manual_seed(1)).int().view(-1, nb)
    kc, vc = (torch.zeros(len(spans) * nb, 64, kv, d, dtype=dtype) for _ in range(2))
    for s, (_, kk, vv) in enumerate(cases):
        for i in range(-(-kk.shape[0] // 64)):
            part = slice(i * 64, (i + 1) * 64)
            kc[pages[s, i], :kk[part].shape[0]], vc[pages[s, i], :kk[part].shape[0]] = kk[part], vv[part]
    got = H.prefill_varlen(q, None, None, cq, ck, mq, mk, scale, k_cache=kc.to(DEV), v_cache=vc.to(DEV), block_tables=pages.to(DEV), mask=mask)
    _close(got, want, dtype, "paged", factor=2.0)
    if dtype != torch.float32:
        got = H.prefill_varlen(q, k, v, cq, ck, mq, mk, scale, mask=mask, flags=H.MV_PREFILL_SIMPLE)
        _close(got, want, dtype, "vector kernel", factor=2.0)


def test_long_windowed_prompts_take_the_eight_wave_kernel(H):
    n, window, keep, dtype = 2200, 700, 5, torch.bfloat16
    q, k, v = _case(n, n, 2, 1, 128, 128, window, keep, dtype, 1)
    sink = _rand(2, dtype=dtype, seed=9)
    got = H.prefill_varlen(q.to(DEV), k.to(DEV), v.to(DEV), _cu([n]), _cu([n]), n, n, 0.1, mask=H.AttnMask(window, keep, 6.0, 1.0, sink.to(DEV)))
    _close(got, _attend(q, k, v, 0.1, 6.0, sink, window, keep), dtype, factor=2.0)


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("heads, kv, d", [(3, 3, 64), (8, 1, 64), (8, 4, 64), (8, 1, 128), (34, 2, 128), (4, 4, 128), (2, 1, 256)])
@pytest.mark.parametrize("window, keep, cap", MASKS, ids=str)
def test_decode_attention(H, dtype, heads, kv, d, window, keep, cap):
    """Lengths just inside and just outside a window, a tile and a page; long contexts in parts; an empty row."""
    scale, factor, bs = 0.4, 0.7, 64
    w = window or 33
    lens = sorted({1, 2, w, w + 1, max(w - 1, 1), w + keep, w + keep + 1, 2 * w + 1, 64, 65, 257, 1100}) + [0]
    sink = (_rand(heads, seed=3) * 2).to(dtype)
    nb = -(-max(lens) // bs)
    pages = torch.randperm(len(lens) * nb, generator=torch.Generator().manual_seed(1)).int().view(-1, nb)
    kc, vc = (torch.zeros(len(lens) * nb, bs, kv, d, dtype=dtype) for _ in range(2))
    qs, wants = [], []
    for s, n in enumerate(lens):
        if n == 0:
            qs.append(torch.zeros(1, heads, d, dtype=dtype))
            wants.append(torch.zeros(1, heads, d, dtype=torch.float64))
            continue
        q, k, v = _case(1, n, heads, kv, d, d, window, keep, dtype, 10 * s)
        wants.append(_attend(q, k, v, scale, cap, sink, window, keep) * factor)
        qs.append(q)
        for i in range(-(-n // bs)):
            part = slice(i * bs, (i + 1) * bs)
            kc[pages[s, i], :k[part].shape[0]], vc[pages[s, i], :k[part].shape[0]] = k[part], v[part]
    q, want, mask = torch.cat(qs).to(DEV), torch.cat(wants), H.AttnMask(window, keep, cap, factor, sink.to(DEV))
    args = (kc.to(DEV), vc.to(DEV), pages.to(DEV), _i32(lens), scale)
    for flags in [0] if dtype == torch.float32 else [0, H.MV_DECODE_VECTOR, H.MV_DECODE_MFMA, H.MV_DECODE_MFMA | H.MV_DECODE_KLDS_ON]:
        _close(H.paged_decode(q, *args, flags=flags, mask=mask), want, dtype, f"flags {flags}", factor=2.0)
    # each row alone: the context in many parts
    for s in range(0, len(lens), 3):
        got = H.paged_decode(q[s:s + 1], args[0], args[1], args[2][s:s + 1], args[3][s:s + 1], scale, mask=mask)
        _close(got, want[s:s + 1], dtype, f"length {lens[s]} alone", factor=2.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, kv, dim, d", [(6, 3, 40, 64), (8, 1, 72, 128), (4, 4, 128, 128), (2, 1, 200, 256)])
def test_head_norms_without_rotation_and_the_fused_decode_step(H, dtype, heads, kv, dim, d):
    T, eps, bs, scale = 9, 1e-3, 64, 0.3
    pad = lambda t: torch.nn.functional.pad(t, (0, d - dim)).to(dtype)
    q, k, v = pad(_rand(T, heads, dim, seed=1)), pad(_rand(T, kv, dim, seed=2)), _rand(T, kv, d, dtype=dtype, seed=3)
    wq, wk = pad(_rand(dim, seed=4) + 1), pad(_rand(dim, seed=5) + 1)
    lens = [1, 5, 64, 65, 100, 128, 129, 17, 2]
    pages = torch.arange(T * 3).int().view(T, 3)
    slots = torch.tensor([int(pages[i, (n - 1) // bs]) * bs + (n - 1) % bs for i, n in enumerate(lens)], dtype=torch.int32)
    kc, vc = (_rand(T * 3, bs, kv, d, dtype=dtype, seed=s).to(DEV) for s in (6, 7))
    kc[..., dim:] = 0
    args = (torch.tensor(lens).to(DEV) - 1, None, None, wq.to(DEV), wk.to(DEV), eps)
    k1, v1 = kc.clone(), vc.clone()
    qn, kn = H.rope_qk_store(q.to(DEV), k.to(DEV), v.to(DEV), *args, k_cache=k1, v_cache=v1, slot_mapping=slots.to(DEV), interleaved_pairs=0,
                             norm_dim=dim)
    norm = lambda x, w: rms(x.double()[..., :dim], eps) * w.double()[:dim]
    _close(qn[..., :dim], norm(q, wq), dtype, "q")
    _close(kn[..., :dim], norm(k, wk), dtype, "k")
    assert qn[..., dim:].abs().sum() == 0 and kn[..., dim:].abs().sum() == 0
    flat = slots.long()
    assert torch.equal(k1.view(-1, kv, d)[flat], kn) and torch.equal(v1.view(-1, kv, d)[flat].cpu(), v)
    mask = H.AttnMask(50, 3, 5.0, 0.8, _rand(heads, dtype=dtype, seed=8).to(DEV))
    want = H.paged_decode(qn, k1, v1, pages.to(DEV), _i32(lens), scale, mask=mask)
    got = H.rope_paged_decode(q.to(DEV), k.to(DEV), v.to(DEV), *args, slots.to(DEV), kc, vc, pages.to(DEV), _i32(lens), scale,
                              interleaved_pairs=0, mask=mask, norm_dim=dim)
    if got is not None:                                                   # (layouts that the one launch takes)
        _close(got, want.double().cpu(), dtype)
        assert torch.equal(kc, k1) and torch.equal(vc, v1)
    else:
        assert dtype == torch.float32 or (d != 128 and heads // kv > 4)


# ---- gated delta rule -------------------------------------------------------------------------------------------------------
class _Delta:
    """One rule's operands in the kernels' layout, with the plain computation beside it."""

    def __init__(self, H, heads, kv, dim, vdim, taps, channel_decay, dtype, slots=6, slow=-1.0, fast=1.0, gate="silu"):
        p, n = -(-vdim // 16) * 16, -(-dim // 32) * 32
        up = lambda v: -(-v // 64) * 64
        k_off = up(heads * p)
        q_off = k_off + up(kv * n)
        self.H, self.heads, self.kv, self.dim, self.vdim, self.dtype, self.gate = H, heads, kv, dim, vdim, dtype, gate
        self.shape = H.DeltaShape(heads, kv, p, n, k_off, q_off, vdim, dim ** -0.5, channel_decay, 1e-4)
        cols = lambda off, units, unit, stored: [off + u * stored + i for u in range(units) for i in range(unit)]
        self.places = {"v": cols(0, heads, vdim, p), "k": cols(k_off, kv, dim, n), "q": cols(q_off, kv, dim, n)}
        self.mask = torch.zeros(self.shape.channels)
        for c in self.places.values():
            self.mask[c] = 1
        self.w = (_rand(taps, self.shape.channels, seed=1) * self.mask).to(dtype)
        self.a_cols = cols(0, heads, dim, n) if channel_decay else list(range(heads))
        width = heads * n if channel_decay else heads
        self.bias, self.a_log = torch.zeros(width), _rand(heads, seed=3) * fast
        self.bias[self.a_cols] = _rand(len(self.a_cols), seed=4) + slow
        self.bias, self.a_log = self.bias.to(dtype), self.a_log.to(dtype)
        self.norm = torch.nn.functional.pad(_rand(vdim, seed=5) + 1, (0, p - vdim)).to(dtype)
        self.conv_state = torch.full((2, slots, taps - 1, self.shape.channels), float("nan"), dtype=dtype, device=DEV)
        self.state = torch.full((2, slots, heads, n, p), float("nan"), device=DEV)     # a fresh sequence must not read its slot

    def inputs(self, t, seed):
        s = self.shape
        x = (_rand(t, s.channels, seed=seed) * self.mask).to(self.dtype)
        a = torch.zeros(t, self.bias.numel())
        a[:, self.a_cols] = _rand(t, len(self.a_cols), seed=seed + 1)
        beta = _rand(t, self.heads + 3, seed=seed + 2)
        gate = torch.zeros(t, self.heads, s.p)
        gate[..., :self.vdim] = _rand(t, self.heads, self.vdim, seed=seed + 3)
        return [v.to(self.dtype) for v in (x, beta, a, gate.flatten(1))]

    def want(self, ins, normed):
        """-> [T, heads * p] in fp64; the convolved rows rounded as the kernels hand them on."""
        s, (x, beta, a, gate) = self.shape, ins
        t, zero = x.shape[0], torch.zeros(s.channels, dtype=torch.float64)
        xc = silu(causal_conv(x.double(), self.w.double().T, zero)).to(self.dtype).double()
        v, k, q = (xc[:, self.places[n]].reshape(t, h, -1) for n, h in (("v", self.heads), ("k", self.kv), ("q", self.kv)))
        q, k = P.delta_operands(q, k, self.heads)
        z = (a.double() + self.bias.double())[:, self.a_cols].reshape(t, self.heads, -1).expand(t, self.heads, self.dim)
        decay = torch.exp(-torch.exp(self.a_log.double())[:, None] * softplus(z))
        o = P.delta_scan(q, k, v, P.sigmoid(beta.double()[:, :self.heads]), decay)
        if normed:
            z = gate.double().reshape(t, self.heads, s.p)[..., :self.vdim]
            o = rms(o, s.eps) * self.norm.double()[:self.vdim] * (silu(z) if self.gate == "silu" else P.sigmoid(z)) * 0.7
        return torch.nn.functional.pad(o, (0, s.p - self.vdim)).flatten(1)

    def prefill(self, parts, slots, flags=0):
        """parts: [(inputs, start, stop)] -> o rows"""
        H, s = self.H, self.shape
        x, beta, a, _ = (torch.cat([ins[i][lo:hi] for ins, lo, hi in parts]).to(DEV) for i in range(4))
        lens = [hi - lo for _, lo, hi in parts]
        cq, ck, sl = _cu(lens), _cu([hi for _, _, hi in parts]), _i32(slots)
        xc = H.causal_conv(x, self.w.to(DEV), None, s.conv, self.conv_state, sl, cq, ck, max(lens))
        return H.delta_prefill(s, xc, beta[:, :self.heads], a, self.bias.to(DEV), self.a_log.to(DEV), self.state, sl, cq, ck, max(lens), flags=flags)

    def step(self, rows, lens, slots):
        """rows: [(inputs, token)]"""
        x, beta, a, gate = (torch.stack([ins[i][t] for ins, t in rows]).to(DEV) for i in range(4))
        return self.H.delta_step(self.shape, x, beta[:, :self.heads], a, self.bias.to(DEV), self.a_log.to(DEV), self.w.to(DEV), self.conv_state,
                                 self.state, _i32(slots), _i32(lens), gate, self.norm.to(DEV), self.gate, 0.7)


DELTAS = [(1, 1, 32, 16, 1), (4, 2, 48, 40, 3), (2, 1, 128, 128, 4), (3, 3, 20, 72, 2), (2, 1, 160, 64, 4), (2, 2, 64, 144, 8), (2, 1, 192, 32, 4)]


@pytest.mark.parametrize("scan", [False, True], ids=["chunks", "scan"])
@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("channel_decay", [False, True], ids=["head", "channel"])
@pytest.mark.parametrize("shape", DELTAS, ids=str)
def test_delta_rule_of_prompts_portions_and_steps(H, dtype, shape, channel_decay, scan):
    """Whole prompts side by side; the same sequence cut anywhere beside other sequences, on other slots; its last tokens one by one."""
    if scan and dtype == torch.float16:
        pytest.skip("the vector kernel is covered in two dtypes")
    flags = H.MV_DELTA_SCAN if scan else 0
    s = _Delta(H, *shape, channel_decay, dtype, gate="sigmoid" if channel_decay else "silu")
    a, b, c = (s.inputs(n, 10 * i + 20) for i, n in enumerate((150, 65, 3)))
    wa, wb, wc = (s.want(v, False) for v in (a, b, c))
    tol = dict(factor=1.0 if dtype == torch.float32 else 1.5)
    o = s.prefill([(a, 0, 150), (b, 0, 65), (c, 0, 3)], [3, 0, -1], flags)
    for got, want, what in ((o[:150], wa, "a"), (o[150:215], wb, "b"), (o[215:], wc, "no slot")):
        _close(got, want, dtype, what, **tol)
    o = s.prefill([(b, 0, 2), (a, 0, 71)], [5, 1], flags)
    _close(o[2:], wa[:71], dtype, "first portion", **tol)
    o = s.prefill([(a, 71, 73), (b, 2, 5)], [1, 5], flags)
    _close(o, torch.cat([wa[71:73], wb[2:5]]), dtype, "two tokens", **tol)
    o = s.prefill([(a, 73, 137)], [1], flags)
    _close(o, wa[73:137], dtype, "third portion", **tol)
    wa, wc = s.want(a, True), s.want(c, True)
    for t in range(137, 150):                                            # decoding, beside another sequence that starts with a step
        rows = [(a, t), (c, t - 137)][:2 if t < 140 else 1]
        o = s.step(rows, [t + 1, t - 136][:len(rows)], [1, 4][:len(rows)])
        _close(o[0], wa[t], dtype, f"step {t}", factor=2.0)
        if t < 140:
            _close(o[1], wc[t - 137], dtype, f"fresh step {t - 137}", factor=2.0)


@pytest.mark.parametrize("channel_decay", [False, True], ids=["head", "channel"])
@pytest.mark.parametrize("slow, fast", [(-8.0, 0.1), (2.0, 1.0), (8.0, 3.0)], ids=["slow", "fast", "gone_within_a_token"])
def test_decays_of_every_speed_over_a_long_prompt(H, slow, fast, channel_decay):
    s = _Delta(H, 2, 1, 64, 32, 4, channel_decay, torch.bfloat16, slow=slow, fast=fast)
    ins = s.inputs(900, 5)
    _close(s.prefill([(ins, 0, 900)], [1]), s.want(ins, False), torch.bfloat16, factor=1.5)


@pytest.mark.parametrize("channel_decay", [False, True], ids=["head", "channel"])
def test_many_heads_and_sequences(H, channel_decay):
    """Enough workgroups that a wave takes two column tiles, one wave of them a single one."""
    s = _Delta(H, 32, 16, 64, 112, 3, channel_decay, torch.bfloat16)
    lens = (70, 5, 64, 65, 128, 1, 33, 90, 2)
    ins = [s.inputs(n, i) for i, n in enumerate(lens)]
    o = s.prefill([(v, 0, n) for v, n in zip(ins, lens)], [0, 3, 1, 4, 2, 5, -1, -1, -1])
    at = 0
    for i, (v, n) in enumerate(zip(ins, lens)):
        if i in (0, 3, 4, 5, 7):
            _close(o[at:at + n], s.want(v, False), torch.bfloat16, f"sequence {i}", factor=1.5)
        at += n


@pytest.mark.parametrize("channel_decay", [False, True], ids=["head", "channel"])
def test_equal_keys_that_nothing_forgets(H, channel_decay):
    """Every token writes at the same key at full strength and nothing decays: the triangular system at its worst."""
    s = _Delta(H, 2, 1, 64, 32, 2, channel_decay, torch.bfloat16, slow=8.0, fast=1e-6)
    x, beta, a, gate = s.inputs(200, 3)
    x[:, s.shape.k_off:] = x[:1, s.shape.k_off:]
    ins = (x, torch.full_like(beta, 9.0), torch.full_like(a, -30.0), gate)
    _close(s.prefill([(ins, 0, 200)], [1]), s.want(ins, False), torch.bfloat16, factor=1.5)


def test_a_repeated_step_changes_nothing_and_padding_rows_keep_nothing(H):
    s = _Delta(H, 4, 2, 48, 64, 4, True, torch.bfloat16)
    ins = s.inputs(20, 3)
    want = s.want(ins, True)
    s.prefill([(ins, 0, 18)], [2])
    s.step([(ins, 18)], [19], [2])
    ahead = s.step([(ins, 19)], [20], [2])                               # one step ahead of the host, then the same step again
    rest = [0, 1, 3, 4, 5]
    before = [t[:, rest].clone() for t in (s.conv_state, s.state)]
    o = s.step([(ins, 19), (ins, 0), (ins, 0)], [20, 0, 7], [2, -1, -1])  # and a padding row, and one without a slot
    assert torch.equal(o[:1], ahead) and o[1].abs().sum() == 0
    _close(o[0], want[19], torch.bfloat16, factor=2.0)
    for t, old in zip((s.conv_state, s.state), before):
        assert torch.equal(torch.nan_to_num(t[:, rest], 7.0), torch.nan_to_num(old, 7.0))


def test_states_beyond_the_registers_of_a_step(H):
    s = _Delta(H, 1, 1, 512, 256, 2, False, torch.float32)
    ins = s.inputs(6, 3)
    want = s.want(ins, True)
    for t in range(6):
        _close(s.step([(ins, t)], [t + 1], [2])[0], want[t], torch.float32, f"step {t}", factor=2.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("gate", ["silu", "sigmoid"])
@pytest.mark.parametrize("heads, p_true", [(3, 20), (4, 64), (2, 128), (1, 8), (2, 300), (1, 1000)])
def test_head_norm_and_gate(H, dtype, gate, heads, p_true):
    p, T = -(-p_true // 16) * 16, 7
    y, z, w = torch.zeros(T, heads, p), torch.zeros(T, heads, p), torch.zeros(p)
    y[..., :p_true], z[..., :p_true], w[:p_true] = _rand(T, heads, p_true, seed=1), _rand(T, heads, p_true, seed=2), _rand(p_true, seed=3)
    y, z, w = y.to(dtype), z.to(dtype), w.to(dtype)
    wide = torch.zeros(T, heads * p + 128, dtype=dtype, device=DEV)
    wide[:, 64:64 + heads * p] = z.flatten(1).to(DEV)
    out = torch.zeros(T, heads * p + 64, dtype=dtype, device=DEV)
    H.head_norm_gate(y.flatten(1).to(DEV), wide[:, 64:64 + heads * p], w.to(DEV), heads, p, p_true, 1e-4, gate, 1.3, out=out[:, :heads * p])
    d = lambda t: t.double()[..., :p_true]
    want = rms(d(y), 1e-4) * d(w) * (silu(d(z)) if gate == "silu" else P.sigmoid(d(z))) * 1.3
    g = out[:, :heads * p].view(T, heads, p)
    _close(g[..., :p_true], want, dtype)
    assert g[..., p_true:].abs().sum() == 0 and out[:, heads * p:].abs().sum() == 0


# ---- experts ------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("T, K, R, top, groups, keep", [(1, 64, 2, 1, 1, 1), (37, 256, 18, 2, 2, 1), (16, 192, 9, 3, 3, 2), (50, 128, 96, 8, 8, 4),
                                                        (5, 64, 320, 6, 1, 1), (130, 512, 64, 4, 1, 1), (3, 64, 6, 6, 2, 2)])
def test_router(H, dtype, T, K, R, top, groups, keep):
    x, w = _rand(T, K, dtype=dtype, seed=1), (_rand(R, K, seed=2) * 2 * K ** -0.5).to(dtype)
    corr = (_rand(R, seed=3) * 0.5).to(dtype)                            # (negative choice scores, choices against the score)
    ids, weights = H.moe_route(x.to(DEV), w.to(DEV), corr.to(DEV), top, groups, keep, 1.7)
    want_ids, want = P.route(x.double() @ w.double().T, corr.double(), top, groups, keep, 1.7)
    full = lambda i, v: torch.zeros(T, R, dtype=torch.float64).scatter(1, i.long().cpu(), v.double().cpu())
    _close(full(ids, weights), full(want_ids, want), torch.float32, factor=5.0)


def test_a_group_without_the_best_choice_is_left_out(H):
    """A group's score is its largest choice score, correction included; negative choice scores inside a kept group still count."""
    w, x = torch.zeros(8, 64), torch.zeros(1, 64)
    x[0, 0], w[:, 0] = 1.0, torch.tensor([3.0, 0, 0, 0, 2.9, 2.8, 0, 0])
    corr = torch.tensor([-0.9, -0.9, -0.9, -0.9, -0.95, -0.96, -0.97, -0.98])     # every choice score is negative
    ids, _ = H.moe_route(x.to(DEV), w.to(DEV), corr.to(DEV), 2, 2, 1)
    want, _ = P.route((x @ w.T).double(), corr.double(), 2, 2, 1, 1.0)
    assert sorted(ids[0].tolist()) == sorted(want[0].tolist()) and len({i // 4 for i in ids[0].tolist()}) == 1


@pytest.mark.parametrize("T, top, experts, outputs, tile_m", [(1, 2, 4, 5, 16), (37, 3, 7, 9, 16), (700, 4, 16, 18, 64), (2000, 2, 3, 3, 128), (40, 1, 64, 64, 32)])
def test_grouping_of_choices(H, T, top, experts, outputs, tile_m):
    ids = torch.stack([torch.randperm(outputs, generator=torch.Generator().manual_seed(t))[:top] for t in range(T)]).int()
    if T == 2000:
        ids[:, 0], ids[:, 1] = 1, 2                                      # an expert nobody chose
    g = H.moe_group(ids.to(DEV), experts, tile_m)
    place, tokens, tiles = g.place.cpu().tolist(), g.tokens.cpu().tolist(), g.tiles.cpu().tolist()
    flat = ids.flatten().tolist()
    order = sorted((i for i, e in enumerate(flat) if e < experts), key=lambda i: flat[i])
    assert [place[i] for i in order] == list(range(len(order))) and all(place[i] == -1 for i, e in enumerate(flat) if e >= experts)
    assert [tokens[n] for n in range(len(order))] == [i // top for i in order]
    seen = []
    for e, first, n in tiles:
        if e >= 0:
            assert 0 < n <= tile_m and all(flat[order[first + j]] == e for j in range(n))
            seen += range(first, first + n)
    assert sorted(seen) == list(range(len(order)))


@pytest.mark.parametrize("dtype, tile_m", [(torch.float32, 16)] + [(torch.bfloat16, m) for m in (16, 32, 64, 128, 256)] + [(torch.float16, 128), (torch.float16, 256)])
@pytest.mark.parametrize("T, width, ff, experts, top", [(3, 64, 64, 4, 2), (90, 256, 192, 5, 2), (300, 192, 320, 3, 1)])
def test_products_over_the_experts(H, dtype, tile_m, T, width, ff, experts, top):
    x = _rand(T, width, dtype=dtype, seed=1)
    gu, dn = ((_rand(experts, *s, seed=i) * s[-1] ** -0.5).to(dtype) for i, s in ((2, (2, ff, width)), (3, (width, ff))))
    ids = torch.stack([torch.randperm(experts + 1, generator=torch.Generator().manual_seed(t))[:top] for t in range(T)]).int()
    g = H.moe_group(ids.to(DEV), experts, tile_m)
    form = (lambda t: t.to(DEV)) if dtype == torch.float32 else (lambda t: H.pack_weight(t.to(DEV).view(-1, t.shape[-1])))
    z = H.moe_linear(x.to(DEV), form(gu), ff, g, H.GateAct(0, 0.0, 0.0), gather=True, experts=experts)
    y = H.moe_linear(z, form(dn), width, g, experts=experts)
    place = g.place.cpu().view(T, top)
    zc, yc = z.cpu(), y.cpu()
    for t in range(T):
        for k in range(top):
            e, i = int(ids[t, k]), int(place[t, k])
            if e == experts:
                assert i == -1
                continue
            want = silu(gu[e, 0].double() @ x[t].double()) * (gu[e, 1].double() @ x[t].double())
            _close(zc[i], want, dtype, f"gated {t} {e}", factor=2.0)
            _close(yc[i], dn[e].double() @ zc[i].double(), dtype, f"down {t} {e}", factor=2.0)


# ---- whole models ------------------------------------------------------------------------------------------------------
def _tokens(n, vocab, seed):
    return _ints(vocab, n, seed).tolist()


_ORACLE = {}


def _logits(name, toks, dtype=torch.float32):
    """The plain model's logits (fp64, cached: several tests ask for the same sequences)."""
    calm = dtype != torch.float32
    key = (name, tuple(toks), calm)
    if key not in _ORACLE:
        _ORACLE[key] = P.forward(CONFIGS[name], sharp_weights(name, calm=calm), toks, torch.float64)
    return _ORACLE[key]


@pytest.fixture(scope="module")
def replayers(tmp_path_factory):
    """StepReplayers by (configuration, dtype), made once: 13 pages and 4 state slots for up to 4 live requests."""
    from minivllm_amd.engine.replay import StepReplayer

    made = {}

    def get(name, dtype):
        if (name, dtype) not in made:
            d = write_checkpoint(tmp_path_factory.mktemp(name), CONFIGS[name], sharp_weights(name, calm=dtype != torch.float32))
            made[name, dtype] = StepReplayer(d, str(dtype).split(".")[-1], 13 * 64)
        r = made[name, dtype]
        assert not r.live and r.blocks.get_num_free_blocks() == 13 and r.blocks.states.num_free == 4
        return r
    yield get
    for r in made.values():
        r.close()


def _check(got, want, dtype, what):
    scale = want.pow(2).mean().sqrt().item()
    err = (got.double() - want).pow(2).mean(-1).sqrt() / scale
    worst, typical = (1e-4, 2e-5) if dtype == torch.float32 else (0.25, 0.06)
    assert err.max() <= worst and (len(err) < 20 or err.median() <= typical), f"{what}: {err.max():.2e}, median {err.median():.2e}"


def _alone(r, toks, cuts, dtype, name, rid="x"):
    """Feed ``toks`` in portions of the sizes ``cuts``, the rest one by one; every position is checked."""
    want, at = _logits(name, toks, dtype), 0
    sizes = list(cuts)
    while sum(sizes) < len(toks):
        sizes.append(1)
    for n in sizes:
        got = r.step([{"id": rid, "tokens": toks[at:at + n], "want": list(range(n))}])
        _check(got, want[at:at + n], dtype, f"{name} portion of {n} at {at}")
        at += n
    r.step([], [rid])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompts_and_token_by_token(replayers, name, dtype):
    r, V = replayers(name, dtype), CONFIGS[name]["vocab"]
    _alone(r, _tokens(1, V, 1), [1], dtype, name)
    _alone(r, _tokens(230, V, 2), [230], dtype, name)
    _alone(r, _tokens(140, V, 3), [], dtype, name)                   # every token decoded, from the first on
    _alone(r, _tokens(230, V, 2), [150], dtype, name)                # a prompt, then decoding across pages and windows


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_portions_of_any_size(replayers, name, dtype):
    r, toks = replayers(name, dtype), _tokens(230, CONFIGS[name]["vocab"], 2)
    _alone(r, toks, [2] * 60 + [3, 50, 57], dtype, name)
    _alone(r, toks, [63, 2, 64, 5, 33, 1, 1, 60], dtype, name)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_mixed_batches_with_pages_and_slots_used_again(replayers, name, dtype):
    """Up to four live requests of unlike length in one batch, portions beside single tokens, requests that pause, end and are
    replaced (their pages and slots are handed on): every position as if the request ran alone."""
    r, V = replayers(name, dtype), CONFIGS[name]["vocab"]
    texts = {f"r{i}": _tokens(n, V, 100 + i) for i, n in enumerate([230, 3, 140, 90, 230, 17, 129, 66])}
    texts["r4"] = texts["r0"]                                        # the same request once more, on other pages
    waiting, live, rnd = sorted(texts), {}, torch.Generator().manual_seed(5)
    pick = lambda n: int(torch.randint(0, n, (1,), generator=rnd))
    for _ in range(400):
        if not waiting and not live:
            break
        while waiting and len(live) < 4:
            if sum(-(-len(texts[i]) // 64) for i in list(live) + [waiting[0]]) > 13:
                break
            live[waiting.pop(0)] = 0
        entries, spans, end = [], [], []
        for i in sorted(live):
            if pick(6) == 0:
                continue                                             # paused for this step
            n = min(len(texts[i]) - live[i], [1, 1, 2, 19, 64, 70][pick(6)])
            entries.append({"id": i, "tokens": texts[i][live[i]:live[i] + n], "want": list(range(n))})
            spans.append((i, live[i], n))
            live[i] += n
            if live[i] == len(texts[i]):
                end.append(i)
        if not entries:
            continue
        got, at = r.step(entries, end), 0
        for i, lo, n in spans:
            _check(got[at:at + n], _logits(name, texts[i], dtype)[lo:lo + n], dtype, f"{name} {i} at {lo} (+{n})")
            at += n
        for i in end:
            live.pop(i)
    assert not live and not waiting


def test_long_decoding_stays_exact(replayers):
    name = "ones"
    _alone(replayers(name, torch.float32), _tokens(600, CONFIGS[name]["vocab"], 9), [5], torch.float32, name)


# ---- generation --------------------------------------------------------------------------------------------------------
@functools.lru_cache(None)
def _greedy(name, prompt, n):
    """Greedy continuation by the plain model; every choice must be clear (by a margin fp32 rounding cannot move)."""
    cfg, toks, w = CONFIGS[name], list(prompt), sharp_weights(name)
    for _ in range(n):
        top = P.forward(cfg, w, toks, torch.float64)[-1].topk(2)
        assert top.values[0] - top.values[1] > 1e-4
        toks.append(int(top.indices[0]))
    return toks[len(prompt):]


def _llm(tmp_path, name, **options):
    from minivllm_amd import LLM, Config

    kw = dict(dtype="float32", max_model_len=256, max_num_batched_tokens=512, max_num_seqs=4, num_kvcache_blocks=16)
    kw.update(options)
    return LLM(Config(write_checkpoint(tmp_path / "m", CONFIGS[name], sharp_weights(name)), **kw))


def _prompts(V):
    shared = _tokens(70, V, 40)
    return [_tokens(5, V, 41), shared + _tokens(20, V, 42), _tokens(1, V, 43), shared + _tokens(55, V, 44)]


@pytest.mark.parametrize("options", [{}, {"enforce_eager": True}, {"enable_chunked_prefill": True, "max_num_batched_tokens": 64},
                                     {"enable_mixed_batches": True, "max_num_seqs": 2}, {"max_num_seqs": 3}, {"num_kvcache_blocks": 6}],
                         ids=["graphs", "eager", "chunked", "mixed", "few_slots", "small_pool"])
def test_greedy_generation_through_the_engine(tmp_path, options):
    """LLM.generate (scheduler, state slots, hipGraph decoding, sampler) picks the plain model's tokens."""
    from minivllm_amd import SamplingParams

    name, n = "odd", 12
    prompts, llm = _prompts(CONFIGS[name]["vocab"]), _llm(tmp_path, name, **options)
    try:
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=n, ignore_eos=True), use_tqdm=False)
        if "num_kvcache_blocks" in options:
            assert llm.scheduler.num_preemptions > 0
    finally:
        llm.exit()
    for p, o in zip(prompts, outs):
        assert o["token_ids"] == _greedy(name, tuple(p), n)


def test_a_sequence_that_ends_early_leaves_the_others_states_alone(tmp_path):
    """Decode steps run one ahead of the host; a step that turns out wrong (a sequence ended) runs again for the others."""
    from minivllm_amd import SamplingParams

    name, n = "states", 16
    prompts = _prompts(CONFIGS[name]["vocab"])
    full = [_greedy(name, tuple(p), n) for p in prompts]
    eos = next(t for t in full[0][6:12] if t not in full[0][:6])           # (not where a sequence enters a new page: no step runs ahead there)
    want = [f[:f.index(eos) + 1] if eos in f else f for f in full]
    assert len({len(x) for x in want}) > 1
    llm = _llm(tmp_path, name, eos=eos)
    try:
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=n), use_tqdm=False)
        ex = llm.model_runner.inference_executor
        assert ex.spec_misses > 0 and ex.spec_hits > 0
    finally:
        llm.exit()
    assert [o["token_ids"] for o in outs] == want


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["states", "large_heads"])   # (vocabularies that the head kernel takes)
def test_graph_replays_equal_eager_steps(tmp_path, name, dtype):
    """Every replay of the captured decode step gives the eager step's logits bit for bit, with eager work (prompts of other
    sequences) and synchronizations in between."""
    from minivllm_amd.config import Config
    from minivllm_amd.engine.block_manager import BlockManager
    from minivllm_amd.engine.model_runner import ModelRunner
    from minivllm_amd.engine.sequence import Sequence
    from minivllm_amd.sampling_params import SamplingParams

    d = write_checkpoint(tmp_path / "m", CONFIGS[name], sharp_weights(name))

    def run(eager):
        cfg = Config(d, dtype=str(dtype).split(".")[-1], max_model_len=320, max_num_batched_tokens=640, max_num_seqs=4,
                     num_kvcache_blocks=20, enforce_eager=eager)
        runner = ModelRunner(cfg, 0)
        ex, bm, out = runner.inference_executor, BlockManager(20, 64, state_slots=4), []
        assert eager or ex.graphs
        seqs = [Sequence(_tokens(n, 100, n), SamplingParams(temperature=0.0, max_tokens=99, ignore_eos=True), block_size=64)
                for n in (150, 33, 64)]
        for s in seqs:
            bm.allocate(s)
        ex.execute_batch(seqs, prefill=True)
        for i in range(12):
            for s in seqs:
                s.append_token(int(_tokens(1, 100, 1000 + i)[0]))
                bm.may_append(s)
            logits, _ = ex.execute_batch(seqs, prefill=False)
            out.append(logits.clone().cpu())
            if i % 4 == 1:                                           # eager work between replays
                other = Sequence(_tokens(40 + i, 100, i), SamplingParams(temperature=0.0), block_size=64)
                bm.allocate(other)
                ex.execute_batch([other], prefill=True)
                bm.deallocate(other)
                torch.cuda.synchronize()
        runner.exit()
        return out
    for i, (a, b) in enumerate(zip(run(True), run(False))):
        assert torch.equal(a, b), f"step {i}"


def test_trace_run_program(tmp_path):
    """bin/trace_run, as a user calls it: steps on standard input, files out."""
    import json
    import os
    import subprocess
    import sys

    import numpy as np

    name = "ones"
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    d = write_checkpoint(tmp_path / "m", CONFIGS[name], sharp_weights(name))
    a, b = _tokens(70, 64, 2), _tokens(9, 64, 3)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:68], "want": [0, 67]}, {"id": "b", "tokens": b[:4], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[4:8], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[8:], "want": [0]}, {"id": "a", "tokens": a[68:], "want": [1]}], "end": ["a", "b"]}]
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", d, "--dtype", "float32", "--out",
                        str(tmp_path / "o"), "--max-tokens", "192"], input="\n".join(map(json.dumps, steps)), text=True,
                       capture_output=True, timeout=100)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [x for x in p.stdout.splitlines() if x.startswith("done")] == ["done 0", "done 1", "done 2"]
    la, lb = _logits(name, a), _logits(name, b)
    for n, want in ((0, la[[0, 67]]), (2, torch.stack([lb[8], la[69]]))):
        got = torch.from_numpy(np.fromfile(tmp_path / "o" / f"{n}.f32", dtype="<f4").reshape(-1, 64))
        _check(got, want, torch.float32, f"file {n}")
