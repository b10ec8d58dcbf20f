"""Kugulorn on the GPU: each mechanism's kernel against the plain statement of it, whole models through the engine in every way a
sequence can be cut, batched, paged and given a state slot, and greedy generation through the public entry point."""
import functools

import pytest
import torch

from kugulorn_configs import CONFIGS, sharp_weights, write_checkpoint
from oracle import kugulorn as K
from oracle.mofarax import rms, rms_norm, rotate_interleaved

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


def _tables(rot, base=1e4, n=4096):
    from minivllm_amd.layers.rotary_embedding import RotaryEmbedding

    return RotaryEmbedding(rot, rot, n, base, interleaved=True)._tables(DEV)


def _cu(lens):
    return torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist(), dtype=torch.int32, device=DEV)


# ---- residual, gate ----------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("splits", [0, 3])
def test_scaled_sublayer_output_joins_the_stream(H, dtype, splits):
    rows, cols, true, eps, mult = 9, 256, 200, 1e-3, 0.37
    pad = lambda t: torch.nn.functional.pad(t, (0, cols - true))
    mk = lambda *s, seed: pad(_rand(*s, seed=seed)).to(dtype)
    wy, sc, wn, x0 = mk(true, seed=2), mk(true, seed=3), mk(true, seed=4), pad(_rand(rows, true, seed=5))
    y = pad(_rand(splits, rows, true, seed=1)) if splits else mk(rows, true, seed=1)
    total = (y.double().sum(0) if splits else y.double())[:, :true]
    x = x0.to(DEV)
    out = H.residual_update(x, y=y.to(DEV), y_norm_w=wy.to(DEV), y_scale=sc.to(DEV), y_mult=mult, norm_w=wn.to(DEV), eps=eps, cols_true=true)
    want = x0.double()[:, :true] + mult * sc.double()[:true] * rms_norm(total, wy.double()[:true], eps, 0.0)
    _close(x[:, :true], want, torch.float32, "stream")
    _close(out[:, :true], rms_norm(want, wn.double()[:true], eps, 0.0), dtype, "norm")
    assert x[:, true:].abs().sum() == 0 and out[:, true:].abs().sum() == 0
    x = x0.to(DEV)                                                       # the scale without a norm
    H.residual_update(x, y=y.to(DEV), y_scale=sc.to(DEV), y_mult=mult, dtype=dtype, cols_true=true)
    _close(x[:, :true], x0.double()[:, :true] + mult * sc.double()[:true] * total, torch.float32, "plain")


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
def test_clamped_gate(H, dtype):
    x = _rand(11, 360, dtype=dtype, seed=1) * 4                          # both clamps bite
    wide = torch.zeros(11, 264, dtype=dtype, device=DEV)
    H.act_and_mul(x.to(DEV)[:, 16:16 + 336], H.clamped_glu(1.5), out=wide[:, 64:232])
    want = K.clamped_glu(x.double()[:, 16:184], x.double()[:, 184:352], 1.5)
    _close(wide[:, 64:232], want, dtype)
    assert wide[:, :64].abs().sum() == 0 and wide[:, 232:].abs().sum() == 0
    other = H.act_and_mul(x.to(DEV)[:, :352], H.clamped_glu(1e6, alpha=0.3))      # the constants are parameters
    g, u = x.double()[:, :176], x.double()[:, 176:352]
    _close(other, g * torch.sigmoid(0.3 * g) * (u + 1), dtype)
    with pytest.raises(H.MvHipError):
        H.act_and_mul(x.to(DEV)[:, :352], H.clamped_glu(-1.0))


@pytest.mark.parametrize("m, inter, k", [(1, 80, 256), (5, 192, 320), (16, 64, 512), (33, 208, 192), (200, 144, 256)])
def test_clamped_gate_in_the_epilogue_of_the_gated_projection(H, m, inter, k):
    from minivllm_amd.layers.linear import MID_CFGS

    dtype, act = torch.bfloat16, H.clamped_glu(1.2)
    x, w = _rand(m, k, dtype=dtype, seed=1), (_rand(2 * inter, k, seed=2) * 3 * k ** -0.5).to(dtype)
    y = x.double() @ w.double().T
    want, wp = K.clamped_glu(y[:, :inter], y[:, inter:], 1.2), H.pack_weight(w.to(DEV))
    wide = torch.zeros(m, inter + 96, dtype=dtype, device=DEV)
    out = wide[:, 64:64 + inter]
    if k >= 256 and m <= 64:
        for packed in (None, wp):
            _close(H.gate_up_silu_small_m(x.to(DEV), w.to(DEV), packed=packed, act=act, out=out), want, dtype)
    for cfg in [0] + [c for c, (_, _, gated) in MID_CFGS.items() if gated]:
        wide.zero_()
        _close(H.gate_up_silu_mid_m(x.to(DEV), wp, inter, cfg, act=act, out=out), want, dtype, f"tile {cfg}")
        assert wide[:, :64].abs().sum() == 0 and wide[:, 64 + inter:].abs().sum() == 0


# ---- latent attention around the attention kernels ------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("q_rank, kv_rank, rot", [(40, 48, 12), (96, 512, 64), (300, 70, 2)])
def test_norms_rotation_and_store_of_the_latents(H, dtype, q_rank, kv_rank, rot):
    T, bs, eps = 37, 64, 1e-4
    qc, kc, rc = -(-q_rank // 64) * 64, -(-kv_rank // 64) * 64, -(-rot // 32) * 32
    z = torch.zeros(T, qc + kc + 64)
    z[:, :q_rank], z[:, qc:qc + kv_rank], z[:, qc + kc:qc + kc + rot] = _rand(T, q_rank, seed=1), _rand(T, kv_rank, seed=2), _rand(T, rot, seed=3)
    z = z.to(dtype)
    wq, wk = (torch.nn.functional.pad(_rand(n, seed=s), (0, c - n)).to(dtype) for n, c, s in ((q_rank, qc, 4), (kv_rank, kc, 5)))
    pos = torch.randint(0, 3000, (T,), generator=torch.Generator().manual_seed(6))
    slots = torch.randperm(3 * bs, generator=torch.Generator().manual_seed(7))[:T].int()
    slots[5], slots[6] = -1, 3 * bs                                       # nowhere, and outside the plane
    plane = torch.zeros(3, bs, kc + rc, dtype=dtype, device=DEV)
    cos, sin = _tables(rot, 777.0)
    q, rows = H.latent_prep(z.to(DEV), wq.to(DEV), 0, q_rank, eps, (wk.to(DEV), qc, kv_rank, qc + kc, rot, rc), pos.to(DEV), cos, sin,
                            plane, slots.to(DEV), want_rows=True)
    zd = z.double()
    _close(q[:, :q_rank], rms(zd[:, :q_rank], eps) * wq.double()[:q_rank], dtype, "query latent")
    _close(rows[:, :kv_rank], rms(zd[:, qc:qc + kv_rank], eps) * wk.double()[:kv_rank], dtype, "latent")
    want = rotate_interleaved(zd[:, None, qc + kc:qc + kc + rot], pos, 777.0, rot)[:, 0]
    _close(rows[:, kc:kc + rot], want, dtype, "rotated part")
    assert q[:, q_rank:].abs().sum() == 0 and rows[:, kv_rank:kc].abs().sum() == 0 and rows[:, kc + rot:].abs().sum() == 0
    flat = plane.view(-1, kc + rc)
    for t, s in enumerate(slots.tolist()):
        if 0 <= s < 3 * bs:
            assert torch.equal(flat[s], rows[t])
    assert int((flat.abs().sum(1) > 0).sum()) == T - 2
    q2, none = H.latent_prep(z.to(DEV), wq.to(DEV), 0, q_rank, eps)      # a layer that reads another's latents
    assert none is None and torch.equal(q2, q)


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("T, h, n, k, rot", [(1, 3, 64, 32, 12), (5, 17, 512, 128, 64), (70, 2, 128, 512, 0), (300, 16, 64, 160, 0), (33, 1, 80, 96, 2)])
def test_per_head_products(H, dtype, T, h, n, k, rot):
    rc = -(-rot // 32) * 32
    x, w = _rand(T, h, k + rc + 8, dtype=dtype, seed=1), (_rand(h, n, k, seed=2) * k ** -0.5).to(dtype)
    out = torch.zeros(T, h, n + rc + 16, dtype=dtype, device=DEV)
    pos = torch.arange(T) * 7
    args = None
    if rot:
        cos, sin = _tables(rot)
        args = (rot, rc, pos.to(DEV), cos, sin)
    H.head_linear(x.to(DEV), w.to(DEV), out, args)
    want = torch.stack([x.double()[:, i, :k] @ w.double()[i].T for i in range(h)], 1)
    _close(out[:, :, :n], want, dtype)
    if rot:
        _close(out[:, :, n:n + rot], rotate_interleaved(x.double()[:, :, k:k + rot], pos, 1e4, rot), dtype, "rotated")
    assert out[:, :, n + rot:].abs().sum() == 0


@pytest.mark.parametrize("dtype", DTYPES)
def test_gathered_rows(H, dtype):
    plane = _rand(7, 64, 96, dtype=dtype, seed=1).to(DEV)
    tables = torch.tensor([[4, 2, 0], [1, -1, 6]], dtype=torch.int32)
    first, lens = [60, 0], [100, 190]
    got = H.latent_gather(plane, tables.to(DEV), _cu(lens), torch.tensor(first, dtype=torch.int32, device=DEV), 290, 190)
    at = 0
    for s in range(2):
        for p in range(first[s], first[s] + lens[s]):
            blk = int(tables[s, p // 64])
            want = plane[blk, p % 64] if blk >= 0 else torch.zeros_like(plane[0, 0])
            assert torch.equal(got[at], want)
            at += 1


# ---- the attention kernels -------------------------------------------------------------------------------------------------
def _edge_queries(n, dim, window, keys, seed):
    """Queries that point at the key just outside their window, hard, at the one just inside, and at token 0: a window that is one
    off answers with another key's value."""
    q = _rand(n, dim, seed=seed) * 0.3
    w = window or n
    for i in range(n):
        for j in (i - w, i - w + 1, 0):
            if 0 <= j <= i:
                q[i] += 4 * keys[j] / keys[j].norm()
    return q


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("heads, dim, rot, dv", [(3, 20, 12, 64), (2, 128, 64, 128), (1, 64, 64, 192), (2, 160, 32, 64), (2, 200, 30, 256)])
@pytest.mark.parametrize("window", [0, 1, 31, 64, 65, 129])
def test_prefill_windows(H, dtype, heads, dim, rot, dv, window):
    """Whole sequences and portions (the last queries of a sequence), several in one launch."""
    scale, plain, rc = 0.5, -(-dim // 32) * 32, -(-rot // 32) * 32
    dq = next(d for d in (64, 128, 192, 256) if plain + rc <= d)
    spans = [(150, 150), (2, 97), (70, 200), (1, 1), (1, 66)]            # (queries, keys)
    cos, sin = _tables(rot)
    qs, ks, rs, vs, ps, wants = [], [], [], [], [], []
    for s, (nq, nk) in enumerate(spans):
        k, r, v = _rand(nk, heads, dim, seed=10 + s), _rand(nk, rot, seed=30 + s), _rand(nk, heads, dv, seed=50 + s)
        pos = torch.arange(nk)
        q = torch.zeros(nk, heads, dim + rot)
        for hd in range(heads):
            q[:, hd, :dim] = _edge_queries(nk, dim, window, k[:, hd], 70 + s)
            q[:, hd, dim:] = _rand(nk, rot, seed=90 + s) * 0.3
        q, k, r, v = (t.to(dtype) for t in (q, k, r, v))
        q = q[nk - nq:]
        full = torch.zeros(nk, heads, dim + rot, dtype=torch.float64)
        full[nk - nq:] = q.double()
        full[..., dim:] = rotate_interleaved(full[..., dim:], pos, 1e4, rot)
        wants.append(K.latent_attention(full[..., :dim], full[..., dim:], k.double(), r.double(), v.double(), scale,
                                        K.window_mask(nk, window or None))[nk - nq:])
        qp = torch.zeros(nq, heads, dq, dtype=dtype)
        qp[..., :dim], qp[..., plain:plain + rot] = q[..., :dim], q[..., dim:]
        kp = torch.zeros(nk, heads, plain, dtype=dtype)
        kp[..., :dim] = k
        rp = torch.zeros(nk, rc, dtype=dtype)
        rp[:, :rot] = r
        qs.append(qp), ks.append(kp), rs.append(rp), vs.append(v), ps.append(pos[nk - nq:])
    kv = torch.cat([torch.cat(ks).flatten(1), torch.cat(vs).flatten(1)], 1).to(DEV)     # one matrix, as the model has it
    k, v = kv[:, :heads * plain].unflatten(1, (heads, plain)), kv[:, heads * plain:].unflatten(1, (heads, dv))
    big = torch.zeros(sum(a for a, _ in spans), heads * dv + 64, dtype=dtype, device=DEV)
    H.latent_prefill(torch.cat(qs).to(DEV), k, v, torch.cat(rs).to(DEV), _cu([a for a, _ in spans]), _cu([b for _, b in spans]),
                     max(a for a, _ in spans), max(b for _, b in spans), torch.cat(ps).to(DEV), cos, sin, rot, scale, window,
                     out=big[:, :heads * dv].view(-1, heads, dv))
    got, at = big[:, :heads * dv].view(-1, heads, dv), 0
    for (nq, nk), want in zip(spans, wants):
        _close(got[at:at + nq], want, dtype, f"{nq} of {nk}", factor=2.0)
        at += nq
    assert big[:, heads * dv:].abs().sum() == 0


def test_long_prompts_take_the_eight_wave_kernel(H):
    n, window, heads, dtype = 2200, 700, 1, torch.bfloat16
    q, k, v, r = (_rand(n, *s, dtype=dtype, seed=i) for i, s in enumerate(((heads, 192), (heads, 128), (heads, 128), (64,))))
    cos, sin = _tables(64)
    got = H.latent_prefill(q.to(DEV), k.to(DEV), v.to(DEV), r.to(DEV), _cu([n]), _cu([n]), n, n, torch.arange(n).to(DEV), cos, sin, 64, 0.1,
                           window)
    qd = q.double()
    qd[..., 128:] = rotate_interleaved(qd[..., 128:], torch.arange(n), 1e4, 64)
    want = K.latent_attention(qd[..., :128], qd[..., 128:], k.double(), r.double(), v.double(), 0.1, K.window_mask(n, window))
    _close(got, want, dtype, factor=2.0)


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("heads, kv, rot", [(1, 64, 2), (5, 128, 32), (17, 512, 64), (40, 192, 30), (3, 320, 64), (2, 640, 64), (2, 64, 96)])
@pytest.mark.parametrize("window", [0, 1, 33, 64, 200])
def test_decode_windows(H, dtype, heads, kv, rot, window):
    """Lengths just inside and just outside a window, a tile and a page; long contexts in parts; an empty row."""
    scale, rc, bs = 0.4, -(-rot // 32) * 32, 64
    w = window or 33
    lens = sorted({1, 2, w, w + 1, max(w - 1, 1), 2 * w + 1, 32, 33, 64, 65, 257, 1100}) + [0]
    nb = -(-max(lens) // bs)
    order = torch.randperm(len(lens) * nb, generator=torch.Generator().manual_seed(3)).int().view(len(lens), nb)
    plane = torch.full((len(lens) * nb, bs, kv + rc), float("nan"), dtype=dtype)       # what no sequence wrote must not be read
    q, wants = torch.zeros(len(lens), heads, kv + rc), []
    for b, n in enumerate(lens):
        if n == 0:
            wants.append(torch.zeros(heads, kv, dtype=torch.float64))
            continue
        rows = torch.zeros(n, kv + rc)
        rows[:, :kv + rot] = _rand(n, kv + rot, seed=b)
        rows = rows.to(dtype)
        for i in range(-(-n // bs)):
            part = rows[i * bs:(i + 1) * bs]
            plane[order[b, i], :part.shape[0]] = part
        f = rows.double()
        for hd in range(heads):
            q[b, hd] = _rand(kv + rc, seed=100 + hd) * 0.1
            for j in (n - 1 - w, n - w, 0):                               # just outside, just inside, the first
                if 0 <= j < n:
                    q[b, hd] += 4 * rows[j].float() / rows[j].float().norm()
        qd = q[b].to(dtype).double()
        lo = max(0, n - window) if window else 0
        p = torch.softmax(qd @ f[lo:].T * scale, -1)
        wants.append(p @ f[lo:, :kv])
    got = H.latent_decode(q.to(dtype).to(DEV), plane.to(DEV), order.to(DEV), torch.tensor(lens, dtype=torch.int32, device=DEV), kv, scale, window)
    for b, n in enumerate(lens):
        _close(got[b], wants[b], dtype, f"length {n}", factor=2.0)


def test_decode_skips_pages_that_are_not_there(H):
    dtype, kv = torch.bfloat16, 64
    plane = _rand(4, 64, kv + 32, dtype=dtype, seed=1)
    q = _rand(1, 2, kv + 32, dtype=dtype, seed=2)
    tables = torch.tensor([[2, -1, 3]], dtype=torch.int32, device=DEV)
    rows = torch.cat([plane[2], plane[3][:22]]).double()
    want = torch.softmax(q[0].double() @ rows.T * 0.2, -1) @ rows[:, :kv]
    for flags in (0, H.MV_LATENT_SIMPLE):
        got = H.latent_decode(q.to(DEV), plane.to(DEV), tables, torch.tensor([150], dtype=torch.int32, device=DEV), kv, 0.2, flags=flags)
        _close(got[0], want, dtype, factor=2.0)


# ---- state space layer ------------------------------------------------------------------------------------------------------
class _Ssm:
    """One layer's operands in the kernels' layout, with the plain computation beside it."""

    def __init__(self, heads, groups, p, n, taps, dtype, slots=6, slow=-3.0):
        self.heads, self.groups, self.p, self.n, self.taps, self.dtype = heads, groups, p, n, taps, dtype
        up = lambda v: -(-v // 64) * 64
        self.b_off = up(heads * p)
        self.c_off = up(self.b_off + groups * n)
        self.ch = self.c_off + groups * n
        self.shape = (heads, groups, p, n, self.b_off, self.c_off)
        self.used = torch.cat([torch.arange(heads * p), self.b_off + torch.arange(groups * n), self.c_off + torch.arange(groups * n)])
        mask = torch.zeros(self.ch)
        mask[self.used] = 1
        self.mask = mask
        self.w, self.b = _rand(taps, self.ch, seed=1) * mask, _rand(self.ch, seed=2) * mask
        self.bias, self.a_log, self.d = (_rand(heads, seed=s) for s in (3, 4, 5))
        self.w, self.b, self.bias, self.a_log, self.d = (t.to(dtype) for t in (self.w, self.b, self.bias, self.a_log, self.d))
        self.slow = slow
        self.conv_state = torch.full((2, slots, taps - 1, self.ch), float("nan"), dtype=dtype, device=DEV)
        self.ssm_state = torch.full((2, slots, heads, n, p), float("nan"), device=DEV)     # a fresh sequence must not read its slot

    def inputs(self, t, seed):
        x = (_rand(t, self.ch, seed=seed) * self.mask).to(self.dtype)
        dt = (_rand(t, self.heads, seed=seed + 1) + self.slow).to(self.dtype)
        return x, dt

    def want(self, x, dt):
        """-> y [T, heads * p] in fp64; the convolved rows rounded as the kernels hand them on."""
        xc = K.silu(K.causal_conv(x.double(), self.w.double().T, self.b.double()))
        xc = xc.to(self.dtype).double()
        t = x.shape[0]
        y = K.ssm_scan(xc[:, :self.heads * self.p].reshape(t, self.heads, self.p),
                       xc[:, self.b_off:self.b_off + self.groups * self.n].reshape(t, self.groups, self.n),
                       xc[:, self.c_off:].reshape(t, self.groups, self.n), K.softplus(dt.double() + self.bias.double()),
                       self.a_log.double(), self.d.double())
        return y.reshape(t, -1)

    def prefill(self, H, parts, slots, flags=0):
        """parts: [(x, dt, tokens before)] -> y rows"""
        dev = lambda t: t.to(DEV)
        x, dt = torch.cat([a for a, _, _ in parts]), torch.cat([b for _, b, _ in parts])
        lens = [a.shape[0] for a, _, _ in parts]
        cq, ck = _cu(lens), _cu([n + before for n, (_, _, before) in zip(lens, parts)])
        sl = torch.tensor(slots, dtype=torch.int32, device=DEV)
        xc = H.causal_conv(dev(x), dev(self.w), dev(self.b), self.shape, self.conv_state, sl, cq, ck, max(lens))
        return H.ssm_prefill(xc, dev(dt), dev(self.bias), dev(self.a_log), dev(self.d), self.shape, self.ssm_state, sl, cq, ck, max(lens),
                             flags=flags)

    def step(self, H, x, dt, lens, slots):
        dev = lambda t: t.to(DEV)
        return H.ssm_step(dev(x), dev(dt), dev(self.w), dev(self.b), dev(self.bias), dev(self.a_log), dev(self.d), self.shape, self.conv_state,
                          self.ssm_state, torch.tensor(slots, dtype=torch.int32, device=DEV), torch.tensor(lens, dtype=torch.int32, device=DEV))


SSM_SHAPES = [(1, 1, 16, 32, 1), (4, 2, 48, 32, 3), (6, 3, 64, 128, 4), (3, 1, 32, 96, 2), (2, 2, 80, 160, 8), (2, 1, 16, 256, 4), (2, 1, 128, 64, 5),
              (2, 1, 32, 320, 4)]


@pytest.mark.parametrize("scan", [False, True], ids=["chunks", "scan"])
@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("shape", SSM_SHAPES, ids=str)
def test_recurrence_of_prompts_portions_and_steps(H, dtype, shape, scan):
    """A whole prompt; the same sequence cut anywhere beside other sequences, on other slots; and its last tokens one by one."""
    if scan and dtype == torch.float16:
        pytest.skip("the vector kernel is covered in two dtypes")
    flags = H.MV_SSM_SCAN if scan else 0
    s = _Ssm(*shape, dtype)
    a, b, c = (s.inputs(n, 10 * i) for i, n in enumerate((150, 65, 3)))
    wa, wb, wc = (s.want(*v) for v in (a, b, c))
    tol = dict(factor=1.0 if dtype == torch.float32 else 1.5)
    cut = lambda v, lo, hi: (v[0][lo:hi], v[1][lo:hi], lo)
    y = s.prefill(H, [cut(a, 0, 150), cut(b, 0, 65), cut(c, 0, 3)], [3, 0, -1], flags)
    for got, want, what in ((y[:150], wa, "a"), (y[150:215], wb, "b"), (y[215:], wc, "no slot")):
        _close(got, want, dtype, what, **tol)
    # in portions, slots in another order, another sequence in between
    y = s.prefill(H, [cut(b, 0, 2), cut(a, 0, 71)], [5, 1], flags)
    _close(y[2:], wa[:71], dtype, "first portion", **tol)
    y = s.prefill(H, [cut(a, 71, 73), cut(b, 2, 5)], [1, 5], flags)
    _close(y, torch.cat([wa[71:73], wb[2:5]]), dtype, "two tokens", **tol)
    y = s.prefill(H, [cut(a, 73, 137)], [1], flags)
    _close(y, wa[73:137], dtype, "third portion", **tol)
    for t in range(137, 150):                                            # decoding, beside another sequence that starts with a step
        x, dt = torch.stack([a[0][t], c[0][t - 137]]) if t < 140 else a[0][t:t + 1], torch.stack([a[1][t], c[1][t - 137]]) if t < 140 else a[1][t:t + 1]
        y = s.step(H, x, dt, [t + 1, t - 136][:x.shape[0]], [1, 4][:x.shape[0]])
        _close(y[0], wa[t], dtype, f"step {t}", **tol)
        if t < 140:
            _close(y[1], wc[t - 137], dtype, f"fresh step {t - 137}", **tol)


def test_a_repeated_step_changes_nothing_and_padding_rows_keep_nothing(H):
    s = _Ssm(4, 2, 48, 64, 4, torch.bfloat16)
    x, dt = s.inputs(20, 3)
    want = s.want(x, dt)
    s.prefill(H, [(x[:18], dt[:18], 0)], [2])
    s.step(H, x[18:19], dt[18:19], [19], [2])
    ahead = s.step(H, x[19:20], dt[19:20], [20], [2])                    # one step ahead of the host, then the same step again
    rows = torch.cat([x[19:20], x[:1], x[:1]])
    before = [t for t in (s.conv_state[:, [0, 1, 3, 4, 5]], s.ssm_state[:, [0, 1, 3, 4, 5]])]
    y = s.step(H, rows, torch.cat([dt[19:20], dt[:1], dt[:1]]), [20, 0, 7], [2, -1, -1])   # and a padding row, and one without a slot
    assert torch.equal(y[:1], ahead) and y[1].abs().sum() == 0
    _close(y[0], want[19], torch.bfloat16, factor=1.5)
    for t, old in zip((s.conv_state, s.ssm_state), before):   # (indexing copied them)
        assert torch.equal(torch.nan_to_num(t[:, [0, 1, 3, 4, 5]], 7.0), torch.nan_to_num(old, 7.0))


def test_strong_and_weak_decays_over_a_long_prompt(H):
    for slow in (-8.0, 2.0):
        s = _Ssm(2, 1, 32, 64, 4, torch.bfloat16, slow=slow)
        x, dt = s.inputs(1500, 5)
        _close(s.prefill(H, [(x, dt, 0)], [1]), s.want(x, dt), torch.bfloat16, f"dt {slow}", factor=1.5)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, p_true, groups", [(3, 20, 5), (4, 64, 2), (6, 40, 1), (2, 48, 16), (40, 64, 1), (160, 64, 1)])
def test_gated_norm_in_parts(H, dtype, heads, p_true, groups):
    p, T = -(-p_true // 16) * 16, 7
    y, z, w = torch.zeros(T, heads, p), torch.zeros(T, heads, p), torch.zeros(heads, p)
    y[..., :p_true], z[..., :p_true], w[:, :p_true] = _rand(T, heads, p_true, seed=1), _rand(T, heads, p_true, seed=2), _rand(heads, p_true, seed=3)
    y, z, w = y.to(dtype), z.to(dtype), w.to(dtype)
    wide = torch.zeros(T, heads * p + 128, dtype=dtype, device=DEV)
    wide[:, 64:64 + heads * p] = z.flatten(1).to(DEV)
    got = H.gated_group_norm(y.flatten(1).to(DEV), wide[:, 64:64 + heads * p], w.flatten().to(DEV), heads, p, p_true, groups, 1e-4)
    true = lambda t: t.double()[..., :p_true].flatten(-2)
    want = K.gated_group_norm(true(y), true(z), true(w), groups, 1e-4)
    g = got.view(T, heads, p)
    _close(g[..., :p_true].flatten(1), want, dtype)
    assert g[..., p_true:].abs().sum() == 0


# ---- whole models ------------------------------------------------------------------------------------------------------
def _tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


_ORACLE = {}


def _logits(name, toks):
    """The plain model's logits (fp64, cached: several tests ask for the same sequences)."""
    key = (name, tuple(toks))
    if key not in _ORACLE:
        _ORACLE[key] = K.forward(CONFIGS[name], sharp_weights(CONFIGS[name]), toks, torch.float64)
    return _ORACLE[key]


@pytest.fixture(scope="module")
def replayers(tmp_path_factory):
    """StepReplayers by (configuration, dtype), made once: 13 pages and 4 state slots for up to 4 live requests."""
    from minivllm_amd.engine.replay import StepReplayer

    made = {}

    def get(name, dtype):
        if (name, dtype) not in made:
            d = write_checkpoint(tmp_path_factory.mktemp(name), CONFIGS[name], sharp_weights(CONFIGS[name]))
            made[name, dtype] = StepReplayer(d, str(dtype).split(".")[-1], 13 * 64)
        r = made[name, dtype]
        assert not r.live and r.blocks.get_num_free_blocks() == 13 and r.blocks.states.num_free == 4
        return r
    yield get
    for r in made.values():
        r.close()


def _check(got, want, dtype, what):
    scale = want.pow(2).mean().sqrt().item()
    err = (got.double() - want).pow(2).mean(-1).sqrt().max().item() / scale
    assert err <= (5e-5 if dtype == torch.float32 else 0.1), f"{what}: {err:.2e}"


def _alone(r, toks, cuts, dtype, name, rid="x"):
    """Feed ``toks`` in portions of the sizes ``cuts``, the rest one by one; every position is checked."""
    want, at = _logits(name, toks), 0
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
            _check(got[at:at + n], _logits(name, texts[i])[lo:lo + n], dtype, f"{name} {i} at {lo} (+{n})")
            at += n
        for i in end:
            live.pop(i)
    assert not live and not waiting


def test_long_decoding_stays_exact(replayers):
    name = "ones"
    _alone(replayers(name, torch.float32), _tokens(600, CONFIGS[name]["vocab"], 9), [5], torch.float32, name)


def test_more_live_requests_than_slots_are_refused(replayers):
    r = replayers("states", torch.float32)
    for i in range(4):
        assert r.step([{"id": str(i), "tokens": [1, 2], "want": []}]) is None
    with pytest.raises(ValueError, match="live requests"):
        r.step([{"id": "4", "tokens": [1], "want": []}])
    r.step([], [str(i) for i in range(4)])


# ---- generation --------------------------------------------------------------------------------------------------------
@functools.lru_cache(None)
def _greedy(name, prompt, n):
    """Greedy continuation by the plain model; every choice must be clear (by a margin fp32 rounding cannot move)."""
    cfg, toks = CONFIGS[name], list(prompt)
    w = sharp_weights(cfg)
    for _ in range(n):
        top = K.forward(cfg, w, toks, torch.float64)[-1].topk(2)
        assert top.values[0] - top.values[1] > 1e-4
        toks.append(int(top.indices[0]))
    return toks[len(prompt):]


def _llm(tmp_path, name, **options):
    from minivllm_amd import LLM, Config

    kw = dict(dtype="float32", max_model_len=256, max_num_batched_tokens=512, max_num_seqs=4, num_kvcache_blocks=16)
    kw.update(options)
    return LLM(Config(write_checkpoint(tmp_path / "m", CONFIGS[name], sharp_weights(CONFIGS[name])), **kw))


def _prompts(V):
    shared = _tokens(70, V, 40)
    return [_tokens(5, V, 41), shared + _tokens(20, V, 42), _tokens(1, V, 43), shared + _tokens(55, V, 44)]


@pytest.mark.parametrize("options", [{}, {"enforce_eager": True}, {"enable_chunked_prefill": True, "max_num_batched_tokens": 64},
                                     {"enable_mixed_batches": True, "max_num_seqs": 2}, {"max_num_seqs": 3}, {"num_kvcache_blocks": 6}],
                         ids=["graphs", "eager", "chunked", "mixed", "few_slots", "small_pool"])
def test_greedy_generation_through_the_engine(tmp_path, options):
    """LLM.generate (scheduler, state slots, hipGraph decoding, sampler) picks the plain model's tokens."""
    from minivllm_amd import SamplingParams

    name, n = "odd", 20
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

    name, n = "states", 20
    prompts = _prompts(CONFIGS[name]["vocab"])
    full = [_greedy(name, tuple(p), n) for p in prompts]
    eos = next(t for t in full[0][3:12] if t not in full[0][:3])
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

    d = write_checkpoint(tmp_path / "m", CONFIGS[name], sharp_weights(CONFIGS[name]))

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
    d = write_checkpoint(tmp_path / "m", CONFIGS[name], sharp_weights(CONFIGS[name]))
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
