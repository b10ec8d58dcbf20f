"""Mofarax on the GPU: each mechanism's kernel against the plain statement of it, whole models through the engine in every
way a sequence can be cut, batched and paged, and greedy generation through the public entry point."""
import functools

import pytest
import torch

from mofarax_configs import CONFIGS, config, layer, sharp_weights, write_checkpoint
from oracle import mofarax as M

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(scope="module")
def H():
    from minivllm_amd import hip_ops
    return hip_ops


def _tol(dtype):
    return 2e-5 if dtype == torch.float32 else 1e-2


def _close(got, want, dtype, what=""):
    scale = max(want.abs().max().item(), 1e-6)
    err = (got.double().cpu() - want.double()).abs().max().item()
    assert err <= _tol(dtype) * scale, f"{what}: {err:.3e} of {scale:.3e}"


def _rand(*shape, dtype=torch.float32, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)).to(dtype)


# ---- mechanisms --------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D, pairs", [(64, 32), (64, 9), (128, 64), (128, 20), (256, 100)])
def test_interleaved_rotation_and_store(H, dtype, D, pairs):
    from minivllm_amd.layers.rotary_embedding import RotaryEmbedding

    T, nh, nk, bs = 37, 3, 2, 64
    qk = _rand(T, (nh + nk) * D, dtype=dtype, seed=1)
    pos = torch.randint(0, 3000, (T,), generator=torch.Generator().manual_seed(2))
    slots = torch.randperm(4 * bs, generator=torch.Generator().manual_seed(3))[:T].int()
    slots[5] = -1
    rot = RotaryEmbedding(D, 2 * pairs, 3000, 777.0, interleaved=True)
    cos, sin = rot._tables(DEV)
    d = qk.to(DEV)
    q, k = d[:, :nh * D].view(T, nh, D), d[:, nh * D:].view(T, nk, D)
    kc, vc = (torch.zeros(4, bs, nk, D, dtype=dtype, device=DEV) for _ in range(2))
    qo, ko = H.rope_qk_store(q, k, k, pos.to(DEV), cos, sin, k_cache=kc, v_cache=vc, slot_mapping=slots.to(DEV),
                             interleaved_pairs=pairs)
    qf, kf = qk[:, :nh * D].double().view(T, nh, D), qk[:, nh * D:].double().view(T, nk, D)
    want_q, want_k = (M.rotate_interleaved(t, pos, 777.0, 2 * pairs) for t in (qf, kf))
    _close(qo, want_q, dtype, "q")
    _close(ko, want_k, dtype, "k")
    rows_k, rows_v = kc.view(-1, nk, D).cpu(), vc.view(-1, nk, D).cpu()
    for t, s in enumerate(slots.tolist()):
        if s >= 0:      # rotated keys in one plane, the projected keys themselves in the other
            assert torch.equal(rows_k[s], ko[t].cpu()) and torch.equal(rows_v[s], k[t].cpu())
    assert int((rows_v.abs().sum((1, 2)) > 0).sum()) == T - 1


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cols, true", [(64, 50), (384, 384), (1024, 1000), (2304, 2304)])
def test_residual_update(H, dtype, cols, true):
    rows, V, eps = 9, 13, 1e-3
    mk = lambda *s, seed: torch.nn.functional.pad(_rand(*s, seed=seed), (0, cols - true)).to(dtype)
    y, wy, emb, vec, wn = mk(rows, true, seed=1), mk(true, seed=2), mk(V, true, seed=3), mk(true, seed=4), mk(true, seed=5)
    part = torch.nn.functional.pad(_rand(3, rows, true, seed=6), (0, cols - true))
    x0 = torch.nn.functional.pad(_rand(rows, true, seed=7), (0, cols - true))
    ids = torch.arange(rows) * 5 % V
    d = lambda t: t.to(DEV)
    cut = lambda t: t.double()[..., :true]

    def check(x, out, want, norm):
        _close(x[:, :true], want, torch.float32, "stream")
        assert x[:, true:].abs().sum() == 0
        if out is not None:
            _close(out[:, :true], M.rms_norm(want, cut(wn), eps, 1.0) if norm else want, dtype, "out")
            assert out.dtype == dtype and out[:, true:].abs().sum() == 0

    kw = dict(eps=eps, cols_true=true)
    x = torch.full((rows, cols), float("nan"), device=DEV)                       # a started row does not read the stream
    out = H.residual_update(x, embed=d(emb), ids=d(ids), embed_scale=2.5, start=True, vec=d(vec), norm_w=d(wn), norm_offset=1.0, **kw)
    check(x, out, 2.5 * cut(emb)[ids] + cut(vec), True)
    x = d(x0)
    out = H.residual_update(x, y=d(y), dtype=dtype, **kw)
    check(x, out, cut(x0) + cut(y), False)
    x = d(x0)
    out = H.residual_update(x, y=d(part), norm_w=d(wn), norm_offset=1.0, dtype=dtype, **kw)
    check(x, out, cut(x0) + cut(part).sum(0), True)
    x = d(x0)
    out = H.residual_update(x, y=d(y), y_norm_w=d(wy), embed=d(emb), ids=d(ids), embed_scale=0.7, vec=d(vec), norm_w=d(wn),
                            norm_offset=1.0, **kw)
    check(x, out, cut(x0) + M.rms_norm(cut(y), cut(wy), eps, 0.0) + 0.7 * cut(emb)[ids] + cut(vec), True)
    x = d(x0)
    assert H.residual_update(x, y=d(y), want_out=False, dtype=dtype, **kw) is None
    check(x, None, cut(x0) + cut(y), False)


@pytest.mark.parametrize("dtype", DTYPES)
def test_gelu_and_mul_and_gated_lookup(H, dtype):
    x = _rand(11, 360, dtype=dtype, seed=1) * 3
    wide = torch.zeros(11, 264, dtype=dtype, device=DEV)
    got = H.gelu_and_mul(x.to(DEV)[:, 16:16 + 336], out=wide[:, 64:232])
    want = M.gelu_tanh(x.double()[:, 16:184]) * x.double()[:, 184:352]
    _close(got, want, dtype)
    assert wide[:, :64].abs().sum() == 0 and wide[:, 232:].abs().sum() == 0
    for dim, off, total in ((40, 80, 160), (20, 20, 60), (64, 0, 64)):
        s, table, ids = _rand(11, 64, dtype=dtype, seed=2), _rand(17, total, dtype=dtype, seed=3), torch.arange(11) * 3 % 17
        got = H.gated_lookup(s.to(DEV), table.to(DEV), off, dim, ids.to(DEV))
        _close(got[:, :dim], M.gelu_tanh(s.double()[:, :dim]) * table.double()[ids][:, off:off + dim], dtype)
        assert got[:, dim:].abs().sum() == 0


@pytest.mark.parametrize("m, inter, k", [(1, 80, 256), (5, 192, 320), (16, 64, 512), (33, 208, 192), (200, 144, 256)])
def test_gelu_in_the_epilogue_of_the_gated_projection(H, m, inter, k):
    """Row counts of the small-M and the mid-M kernel, row-major and packed weights, into strided rows."""
    from minivllm_amd.layers.linear import MID_CFGS

    dtype = torch.bfloat16
    x, w = _rand(m, k, dtype=dtype, seed=1), (_rand(2 * inter, k, seed=2) * 3 * k ** -0.5).to(dtype)
    gate, up = x.double() @ w.double().T[:, :inter], x.double() @ w.double().T[:, inter:]
    want, wp = M.gelu_tanh(gate) * up, H.pack_weight(w.to(DEV))
    wide = torch.zeros(m, inter + 96, dtype=dtype, device=DEV)
    out = wide[:, 64:64 + inter]
    if k >= 256 and m <= 64:
        for packed in (None, wp):
            _close(H.gate_up_silu_small_m(x.to(DEV), w.to(DEV), packed=packed, act="gelu_tanh", out=out), want, dtype)
    for cfg in [0] + [c for c, (_, _, gated) in MID_CFGS.items() if gated]:
        wide.zero_()
        _close(H.gate_up_silu_mid_m(x.to(DEV), wp, inter, cfg, act="gelu_tanh", out=out), want, dtype, f"tile {cfg}")
        assert wide[:, :64].abs().sum() == 0 and wide[:, 64 + inter:].abs().sum() == 0


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float16])
@pytest.mark.parametrize("m, n, k", [(17, 64, 256), (64, 52, 2048), (255, 128, 2048), (256, 192, 640), (500, 256, 3584)])
def test_narrow_projection_in_row_groups(H, dtype, m, n, k):
    x, w = _rand(m, k, dtype=dtype, seed=1), (_rand(n, k, seed=2) * k ** -0.5).to(dtype)
    wide = x.new_zeros(m, k + 64)
    wide[:, :k] = x
    b = _rand(n, dtype=dtype, seed=3)
    for bias in (None, b):
        got = H.linear_narrow(wide.to(DEV)[:, :k], H.pack_weight(w.to(DEV)), n, None if bias is None else bias.to(DEV))
        want = x.double() @ w.double().T + (0 if bias is None else bias.double())
        _close(got, want, dtype)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float16])
@pytest.mark.parametrize("rows, dim, k, off, total, n", [(1, 20, 64, 20, 60, 64), (9, 128, 128, 128, 384, 1100), (16, 40, 64, 40, 80, 192),
                                                         (17, 200, 256, 0, 200, 52), (300, 96, 128, 96, 288, 448), (33, 500, 512, 8, 512, 320),
                                                         (2500, 72, 128, 72, 144, 1100), (4099, 190, 192, 0, 190, 64), (2049, 500, 512, 0, 500, 320)])
def test_lookup_and_side_projection_in_one_launch(H, dtype, rows, dim, k, off, total, n):
    s, table, w = _rand(rows, k, dtype=dtype, seed=2), _rand(17, total, dtype=dtype, seed=3), _rand(n, k, dtype=dtype, seed=4)
    ids = torch.arange(rows) * 3 % 17
    got = H.gated_lookup_linear(s.to(DEV), table.to(DEV), off, dim, ids.to(DEV), H.pack_weight(w.to(DEV)), n)
    g = (M.gelu_tanh(s.double()[:, :dim]) * table.double()[ids][:, off:off + dim]).to(dtype).double()
    _close(got, g @ w.double()[:, :dim].T, dtype)


def _paged(kv, lens, nk, D, bs, dtype, seed):
    """Scatter per-sequence rows into shuffled blocks; the other slots hold huge values (a wrong slot shows)."""
    nb = sum(-(-n // bs) for n in lens) + 2
    perm = torch.randperm(nb, generator=torch.Generator().manual_seed(seed)).tolist()
    width = max(-(-n // bs) for n in lens)
    table = torch.full((len(lens), width), -1, dtype=torch.int32)
    caches = [torch.full((nb, bs, nk, D), 30.0, dtype=dtype) for _ in kv]
    for b, n in enumerate(lens):
        for j in range(-(-n // bs)):
            blk = perm.pop()
            table[b, j] = blk
            m = min(bs, n - j * bs)
            for c, rows in zip(caches, kv):
                c[blk, :m] = rows[b][j * bs:j * bs + m]
    return [c.to(DEV) for c in caches], table.to(DEV)


def _qkv(lens, nh, nk, D, dtype, seed, chunk):
    """Per-sequence q, k, v.  The last key of every chunk would win the softmax of the next chunk's queries, and the first
    key of a chunk wins its own: a mask that is off by one at either edge is a gross error."""
    q = [_rand(n, nh, D, dtype=dtype, seed=seed + b) for b, n in enumerate(lens)]
    k = [_rand(n, nk, D, dtype=dtype, seed=seed + 50 + b) for b, n in enumerate(lens)]
    v = [_rand(n, nk, D, dtype=dtype, seed=seed + 90 + b) for b, n in enumerate(lens)]
    for kb, qb in zip(k, q):
        qb[:, :, 0] = 4.0
        kb[:, :, 0] = 0.0
        if chunk:
            kb[chunk - 1::chunk, :, 0] = 40.0 if chunk > 1 else 0.0
            kb[::chunk, :, 0] = 20.0 if chunk > 1 else torch.linspace(-20.0, 20.0, kb.shape[0], dtype=dtype)[:, None]
    return q, k, v


def _want(q, k, v, scale, chunk, last_only=False):
    o = M.grouped_attention(q.double(), k.double(), v.double(), scale, M.chunk_mask(q.shape[0], chunk))
    return o[-1:] if last_only else o


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nh, nk, D, chunk", [(4, 4, 64, 80), (4, 2, 64, 33), (5, 1, 64, 1), (2, 2, 128, 100), (8, 2, 128, 64), (3, 1, 128, 700),
                                              (2, 1, 256, 50), (2, 2, 64, 7), (2, 1, 128, 0)])
def test_chunked_prefill_attention(H, dtype, nh, nk, D, chunk):
    lens = [1, 63, 200, 421]
    scale = D ** -0.5
    q, k, v = _qkv(lens, nh, nk, D, dtype, 7, chunk)
    cu = torch.tensor([0] + lens).cumsum(0).int().to(DEV)
    big = torch.zeros(sum(lens), nh * D + 64, dtype=dtype, device=DEV)     # strided output rows
    out = big[:, :nh * D].view(sum(lens), nh, D)
    H.prefill_varlen(torch.cat(q).to(DEV), torch.cat(k).to(DEV), torch.cat(v).to(DEV), cu, cu, max(lens), max(lens), scale,
                     out=out, chunk=chunk)
    for b, n in enumerate(lens):
        _close(out[int(cu[b]):int(cu[b + 1])], _want(q[b], k[b], v[b], scale, chunk or None), dtype, f"sequence {b}")
    assert big[:, nh * D:].abs().sum() == 0
    # portions over the paged cache: queries from the middle of a page / a chunk on
    (kc, vc), table = _paged((k, v), lens, nk, D, 64, dtype, 3)
    starts = [0, 61, 97, 65]
    qs = [t[s:] for t, s in zip(q, starts)]
    cq = torch.tensor([0] + [t.shape[0] for t in qs]).cumsum(0).int().to(DEV)
    got = H.prefill_varlen(torch.cat(qs).to(DEV), None, None, cq, cu, max(t.shape[0] for t in qs), max(lens), scale, k_cache=kc,
                           v_cache=vc, block_tables=table, chunk=chunk)
    for b, s in enumerate(starts):
        _close(got[int(cq[b]):int(cq[b + 1])], _want(q[b], k[b], v[b], scale, chunk or None)[s:], dtype, f"portion {b}")


@pytest.mark.parametrize("dtype", [torch.bfloat16])
@pytest.mark.parametrize("D", [64, 128])
def test_chunked_prefill_long_rows_take_the_eight_wave_kernel(H, dtype, D):
    n, chunk, scale = 2200, 1000, D ** -0.5
    q, k, v = _qkv([n], 1, 1, D, dtype, 11, chunk)
    cu = torch.tensor([0, n], dtype=torch.int32, device=DEV)
    got = H.prefill_varlen(q[0].to(DEV), k[0].to(DEV), v[0].to(DEV), cu, cu, n, n, scale, chunk=chunk)
    _close(got, _want(q[0], k[0], v[0], scale, chunk), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nh, nk, D", [(16, 16, 64), (3, 3, 64), (4, 2, 64), (6, 1, 64), (16, 1, 64), (4, 4, 128), (8, 2, 128), (11, 1, 128),
                                       (2, 1, 256), (8, 4, 256), (14, 2, 256)])
@pytest.mark.parametrize("chunk", [0, 1, 7, 90, 128, 1000])
def test_chunked_paged_decode(H, dtype, nh, nk, D, chunk):
    """Lengths just inside and just outside a chunk, a page and a tile; long contexts (split over workgroups)."""
    c = chunk or 90
    lens = sorted({1, 2, c, c + 1, c - 1 or 1, 2 * c, 2 * c + 1, 64, 65, 257, 2100})
    scale = D ** -0.5
    q, k, v = _qkv(lens, nh, nk, D, dtype, 23, chunk)
    (kc, vc), table = _paged((k, v), lens, nk, D, 64, dtype, 5)
    big = torch.zeros(len(lens), nh * D + 128, dtype=dtype, device=DEV)
    out = big[:, :nh * D].view(len(lens), nh, D)
    H.paged_decode(torch.stack([t[-1] for t in q]).to(DEV), kc, vc, table, torch.tensor(lens, dtype=torch.int32, device=DEV), scale,
                   out=out, chunk=chunk)
    for b, n in enumerate(lens):
        lo = (n - 1) // chunk * chunk if chunk else 0
        want = M.grouped_attention(q[b][-1:].double(), k[b][lo:].double(), v[b][lo:].double(), scale, torch.ones(1, n - lo, dtype=torch.bool))
        _close(out[b:b + 1], want, dtype, f"length {n}")
    assert big[:, nh * D:].abs().sum() == 0


@pytest.mark.parametrize("nh, nk, D, pairs", [(16, 16, 64, 32), (2, 1, 64, 10), (4, 4, 128, 64), (8, 2, 128, 30), (4, 1, 256, 64)])
def test_rotation_store_and_chunked_decode_in_one_launch(H, nh, nk, D, pairs):
    """The fused launch equals rotation + store, then attention, bit for bit."""
    from minivllm_amd.layers.rotary_embedding import RotaryEmbedding

    dtype, chunk, lens = torch.bfloat16, 90, [1, 90, 91, 300, 2000, 0]
    hist = lens[:-1]
    q, k, v = _qkv(hist, nh, nk, D, dtype, 31, chunk)
    (kc, vc), table = _paged((k, v), hist, nk, D, 64, dtype, 9)
    table = torch.cat([table, torch.full((1, table.shape[1]), -1, dtype=torch.int32, device=DEV)])   # a padding row
    ctx = torch.tensor(lens, dtype=torch.int32, device=DEV)
    pos = (ctx.long() - 1).clamp(min=0)
    slots = torch.tensor([int(table[b, (n - 1) // 64]) * 64 + (n - 1) % 64 if n else -1 for b, n in enumerate(lens)],
                         dtype=torch.int32, device=DEV)
    z = _rand(len(lens), (nh + nk) * D, dtype=dtype, seed=77).to(DEV)
    qn, kn = z[:, :nh * D].view(-1, nh, D), z[:, nh * D:].view(-1, nk, D)
    cos, sin = RotaryEmbedding(D, 2 * pairs, 2048, 1e4, interleaved=True)._tables(DEV)
    kc2, vc2 = kc.clone(), vc.clone()
    q_rot, _ = H.rope_qk_store(qn, kn, kn, pos, cos, sin, k_cache=kc, v_cache=vc, slot_mapping=slots, want_k_out=False,
                               interleaved_pairs=pairs)
    want = H.paged_decode(q_rot, kc, vc, table, ctx, 0.1, chunk=chunk)
    got = H.rope_paged_decode(qn, kn, kn, pos, cos, sin, None, None, 0.0, slots, kc2, vc2, table, ctx, 0.1,
                              interleaved_pairs=pairs, chunk=chunk)
    assert got is not None and torch.equal(got, want)
    assert torch.equal(kc, kc2) and torch.equal(vc, vc2)


# ---- whole models ------------------------------------------------------------------------------------------------------
def _tokens(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


_ORACLE = {}


def _logits(name, toks):
    """The plain model's logits (fp64, cached: several tests ask for the same sequences)."""
    key = (name, tuple(toks))
    if key not in _ORACLE:
        cfg = CONFIGS[name]
        _ORACLE[key] = M.forward(cfg, sharp_weights(cfg), toks, torch.float64)
    return _ORACLE[key]


@pytest.fixture(scope="module")
def replayers(tmp_path_factory):
    """StepReplayers by (configuration, dtype), made once: 13 pages for up to 4 live requests."""
    from minivllm_amd.engine.replay import StepReplayer

    made = {}

    def get(name, dtype):
        if (name, dtype) not in made:
            d = write_checkpoint(tmp_path_factory.mktemp(name), CONFIGS[name], sharp_weights(CONFIGS[name]))
            made[name, dtype] = StepReplayer(d, str(dtype).split(".")[-1], 13 * 64)
        r = made[name, dtype]
        assert not r.live and r.blocks.get_num_free_blocks() == 13
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
    _alone(r, _tokens(230, V, 2), [150], dtype, name)                # a prompt, then decoding across pages and chunks


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_portions_of_any_size(replayers, name, dtype):
    r, toks = replayers(name, dtype), _tokens(230, CONFIGS[name]["vocab"], 2)
    _alone(r, toks, [2] * 60 + [3, 50, 57], dtype, name)
    _alone(r, toks, [63, 2, 64, 5, 33, 1, 1, 60], dtype, name)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_mixed_batches_with_pages_used_again(replayers, name, dtype):
    """Up to four live requests of unlike length in one batch, portions beside single tokens, requests that pause, end and
    are replaced (their pages and places are handed on): every position as if the request ran alone."""
    r, V = replayers(name, dtype), CONFIGS[name]["vocab"]
    texts = {f"r{i}": _tokens(n, V, 100 + i) for i, n in enumerate([230, 3, 140, 90, 230, 17, 129, 66])}
    texts["r4"] = texts["r0"]                                        # the same request once more, on other pages
    waiting, live, rnd = sorted(texts), {}, torch.Generator().manual_seed(5)
    pick = lambda n: int(torch.randint(0, n, (1,), generator=rnd))
    for _ in range(400):
        if not waiting and not live:
            break
        while waiting and len(live) < 4:
            need = sum(-(-len(texts[i]) // 64) for i in list(live) + [waiting[0]])
            if need > 13:
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
    name = "tiny_chunk"
    r, toks = replayers(name, torch.float32), _tokens(600, CONFIGS[name]["vocab"], 9)
    _alone(r, toks, [5], torch.float32, name)


def test_nothing_wanted_and_bad_requests(replayers):
    r = replayers("tiny_chunk", torch.float32)
    assert r.step([{"id": "a", "tokens": [1, 2, 3], "want": []}]) is None
    with pytest.raises(ValueError, match="token ids"):
        r.step([{"id": "a", "tokens": [64], "want": []}])
    with pytest.raises(ValueError, match="wanted places"):
        r.step([{"id": "a", "tokens": [1], "want": [1]}])
    r.step([], ["a"])


# ---- generation --------------------------------------------------------------------------------------------------------
@functools.lru_cache(None)
def _greedy(name, prompt, n):
    """Greedy continuation by the plain model, and whether every choice was clear (by a margin fp32 rounding cannot move)."""
    cfg, toks = CONFIGS[name], list(prompt)
    w = sharp_weights(cfg)
    for _ in range(n):
        top = M.forward(cfg, w, toks, torch.float64)[-1].topk(2)
        assert top.values[0] - top.values[1] > 1e-4
        toks.append(int(top.indices[0]))
    return toks[len(prompt):]


@pytest.mark.parametrize("options", [{}, {"enforce_eager": True}, {"enable_chunked_prefill": True, "max_num_batched_tokens": 64},
                                     {"enable_mixed_batches": True, "max_num_seqs": 2}, {"num_kvcache_blocks": 6}],
                         ids=["graphs", "eager", "chunked", "mixed", "small_pool"])
def test_greedy_generation_through_the_engine(tmp_path, options):
    """LLM.generate (scheduler, prefix cache, hipGraph decoding, sampler) picks the plain model's tokens."""
    from minivllm_amd import LLM, Config, SamplingParams

    name, n = "odd", 24
    V = CONFIGS[name]["vocab"]
    shared = _tokens(70, V, 40)
    prompts = [_tokens(5, V, 41), shared + _tokens(20, V, 42), _tokens(1, V, 43), shared + _tokens(30, V, 44)]
    kw = dict(dtype="float32", max_model_len=256, max_num_batched_tokens=512, max_num_seqs=4, num_kvcache_blocks=16)
    kw.update(options)
    llm = LLM(Config(write_checkpoint(tmp_path / "m", CONFIGS[name], sharp_weights(CONFIGS[name])), **kw))
    try:
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=n, ignore_eos=True), use_tqdm=False)
    finally:
        llm.exit()
    for p, o in zip(prompts, outs):
        assert o["token_ids"] == _greedy(name, tuple(p), n)


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_equal_eager_steps(tmp_path, dtype):
    """Every replay of the captured decode step gives the eager step's logits bit for bit, with eager work (prompts of other
    sequences) and synchronizations in between."""
    from minivllm_amd.config import Config
    from minivllm_amd.engine.block_manager import BlockManager
    from minivllm_amd.engine.model_runner import ModelRunner
    from minivllm_amd.engine.sequence import Sequence
    from minivllm_amd.sampling_params import SamplingParams

    name = "gqa128"
    d = write_checkpoint(tmp_path / "m", CONFIGS[name], sharp_weights(CONFIGS[name]))

    def run(eager):
        cfg = Config(d, dtype=str(dtype).split(".")[-1], max_model_len=320, max_num_batched_tokens=640, max_num_seqs=4,
                     num_kvcache_blocks=20, enforce_eager=eager)
        runner = ModelRunner(cfg, 0)
        ex, bm, out = runner.inference_executor, BlockManager(20, 64), []
        assert eager or ex.graphs
        seqs = [Sequence(_tokens(n, 128, n), SamplingParams(temperature=0.0, max_tokens=99, ignore_eos=True), block_size=64)
                for n in (150, 33, 64)]
        for s in seqs:
            bm.allocate(s)
        ex.execute_batch(seqs, prefill=True)
        for i in range(12):
            for s in seqs:
                s.append_token(int(_tokens(1, 128, 1000 + i)[0]))
                bm.may_append(s)
            logits, _ = ex.execute_batch(seqs, prefill=False)
            out.append(logits.clone().cpu())
            if i % 4 == 1:                                           # eager work between replays
                other = Sequence(_tokens(40 + i, 128, i), SamplingParams(temperature=0.0), block_size=64)
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

    name = "tiny_chunk"
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
    assert sorted(os.listdir(tmp_path / "o")) == ["0.f32", "2.f32"]
    la, lb = _logits(name, a), _logits(name, b)
    for n, want in ((0, la[[0, 67]]), (2, torch.stack([lb[8], la[69]]))):
        got = torch.from_numpy(np.fromfile(tmp_path / "o" / f"{n}.f32", dtype="<f4").reshape(-1, 64))
        _check(got, want, torch.float32, f"file {n}")
