"""Semezen on the GPU: each mechanism's kernel against the plain statement of it, whole models through the engine in every way a
sequence can be cut, batched, paged and given a state slot, and greedy generation through the public entry point."""
import functools

import pytest
import torch

from oracle import semezen as S
from oracle.kugulorn import silu
from oracle.mofarax import rms
from oracle.pununex import sigmoid, window_mask
from semezen_configs import CONFIGS, sharp_weights, write_checkpoint

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


# ---- the streams --------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 8])
@pytest.mark.parametrize("cols, true, how", [(256, 200, "rows"), (64, 64, "splits"), (320, 320, "experts"), (4160, 4100, "rows"), (128, 100, "all"),
                                             (8192, 8190, "splits")])
def test_streams_are_mixed_written_and_read(H, dtype, streams, cols, true, how):
    rows, eps, top, n = 7, 1e-3, 2, streams
    pad = lambda t: torch.nn.functional.pad(t, (0, cols - true))
    mk = lambda *s, seed: pad(_rand(*s, seed=seed)).to(dtype)
    w = {k: _rand(*s, dtype=dtype, seed=i) for i, (k, s) in enumerate({"mix": (n, n), "out": (n,), "in": (n,)}.items())}
    nw, x0 = mk(true, seed=7), pad(_rand(rows, n, true, seed=8))
    y, total = None, torch.zeros(rows, true, dtype=torch.float64)
    if how == "rows":
        wide = torch.zeros(rows, cols + 64, dtype=dtype)
        wide[:, 32:32 + cols] = mk(rows, true, seed=9)
        y = wide.to(DEV)[:, 32:32 + cols]
    elif how != "experts":
        y = pad(_rand(3, rows, true, seed=9)).to(DEV)
    if y is not None:
        total += (y.double().cpu().sum(0) if y.dim() == 3 else y.double().cpu())[:, :true]
    experts = None
    if how in ("experts", "all"):
        eo, place, ew = mk(20, true, seed=10), _ints(20, rows * top, 4).int(), _rand(rows, top, seed=3)
        place[3] = -1                                                         # no product: nothing
        weighed = how == "all"
        experts = (eo.to(DEV), place.to(DEV), ew.to(DEV) if weighed else None)
        for t in range(rows):
            for k in range(top):
                if place[t * top + k] >= 0:
                    total[t] += (ew[t, k].double() if weighed else 1.0) * eo.double()[place[t * top + k], :true]
    x, new = x0.to(DEV), torch.full((rows, n, cols), 7.0, device=DEV)
    out = H.stream_update(n, nw.to(DEV), eps, x=x, x_out=new, y=y, mix=w["mix"].to(DEV), out_w=w["out"].to(DEV), in_w=w["in"].to(DEV),
                          experts=experts, cols_true=true)
    want = S.write_streams(x0.double()[..., :true], w["mix"].double(), w["out"].double(), total)
    _close(new[..., :true], want, torch.float32, "streams")
    _close(out[:, :true], rms(S.read_streams(want, w["in"].double()), eps) * nw.double()[:true], dtype, "norm")
    assert new[..., true:].abs().sum() == 0 and out[:, true:].abs().sum() == 0 and torch.equal(x.cpu(), x0)
    out = H.stream_update(n, nw.to(DEV), eps, x=x, y=y, mix=w["mix"].to(DEV), out_w=w["out"].to(DEV), experts=experts, cols_true=true)
    _close(out[:, :true], rms(want.sum(1), eps) * nw.double()[:true], dtype, "the sum at the end")
    H.stream_update(n, nw.to(DEV), eps, x=x, x_out=x, y=y, mix=w["mix"].to(DEV), out_w=w["out"].to(DEV), experts=experts, cols_true=true)
    assert torch.equal(x, new)                                                # in place


@pytest.mark.parametrize("dtype", DTYPES)
def test_streams_start_from_the_embedding(H, dtype):
    E, ids, nw, a = _rand(50, 64, dtype=dtype, seed=1), _ints(50, 9, 2), _rand(64, dtype=dtype, seed=3), _rand(3, dtype=dtype, seed=4)
    x = torch.empty(9, 3, 64, device=DEV)
    h = H.stream_update(3, nw.to(DEV), 1e-4, embed=E.to(DEV), ids=ids.to(DEV), x_out=x, in_w=a.to(DEV))
    assert torch.equal(x.cpu(), E.float()[ids][:, None].expand(9, 3, 64))
    _close(h, rms(E.double()[ids] * a.double().sum(), 1e-4) * nw.double(), dtype)


class _Shift:
    """Token-shifted reads of random streams, with the plain computation beside it."""

    def __init__(self, H, dtype, cols=64, streams=2, slots=4):
        self.H, self.dtype, self.n, self.cols = H, dtype, streams, cols
        self.nw, self.a, self.share = (_rand(k, dtype=dtype, seed=i) for i, k in enumerate((cols, streams, cols)))
        self.mix, self.out = _rand(streams, streams, dtype=dtype, seed=3), _rand(streams, dtype=dtype, seed=4)
        self.prev = torch.full((2, slots, cols), float("nan"), device=DEV)       # a fresh sequence must not read its slot

    def sequence(self, n, seed):
        x, y = _rand(n, self.n, self.cols, seed=seed), _rand(n, self.cols, dtype=self.dtype, seed=seed + 1)
        new = S.write_streams(x.double(), self.mix.double(), self.out.double(), y.double())
        h = rms(S.read_streams(new, self.a.double()), 1e-4) * self.nw.double()
        return x, y, new, S.token_shift(h, self.share.double())

    def run(self, parts, decode=False, check=True):
        """parts: [(sequence, start, stop, slot)]"""
        cat = lambda i: torch.cat([s[i][lo:hi] for s, lo, hi, _ in parts])
        x, new = cat(0).to(DEV), torch.full((sum(hi - lo for _, lo, hi, _ in parts), self.n, self.cols), 7.0, device=DEV)
        pos = torch.cat([torch.arange(lo, hi) for _, lo, hi, _ in parts]).to(DEV)
        shift = self.H.StreamShift(self.share.to(DEV), self.prev, pos, _i32([s for *_, s in parts]),
                                   None if decode else _cu([hi - lo for _, lo, hi, _ in parts]))
        got = self.H.stream_update(self.n, self.nw.to(DEV), 1e-4, x=x, x_out=new, y=cat(1).to(DEV), mix=self.mix.to(DEV),
                                   out_w=self.out.to(DEV), in_w=self.a.to(DEV), shift=shift)
        if check:
            _close(got, cat(3), self.dtype, f"{[p[1:] for p in parts]}")
            _close(new, cat(2), torch.float32, "streams")
        return got


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cols", [64, 1088])
def test_shift_follows_the_sequence_through_portions_and_steps(H, dtype, cols):
    s = _Shift(H, dtype, cols)
    a, b = s.sequence(14, 10), s.sequence(7, 20)
    s.run([(a, 0, 14, 0), (b, 0, 7, 3)])
    s.run([(b, 0, 2, 0), (a, 0, 5, 2)])                                   # slot 0 starts again; both halves of a slot in turn
    s.run([(a, 5, 6, 2)], decode=True)
    s.run([(a, 6, 7, 2), (b, 2, 3, 0)], decode=True)
    s.run([(a, 6, 7, 2), (b, 2, 3, 0)], decode=True)                      # again
    s.run([(b, 3, 4, 0), (a, 7, 9, 2)])                                   # a decoded row ahead of a portion of two
    s.run([(a, 9, 11, 2), (b, 4, 7, 0)])
    s.run([(a, 11, 14, 2)])
    kept = s.prev.clone()
    s.run([(a, 0, 1, -1), (b, 0, 1, -1)], decode=True)                    # padding rows and rows without a slot keep nothing
    assert torch.equal(torch.nan_to_num(s.prev, 7.0), torch.nan_to_num(kept, 7.0))


@pytest.mark.parametrize("lens", [(5000,), (3, 4096, 1, 1, 2000, 2), (2049, 2047), tuple([1, 2, 3, 70] * 60)], ids=str)
def test_shift_over_runs_of_rows(H, lens):
    """Enough rows that a workgroup takes a run of them: sequences that begin, end and lie inside runs; the next step reads what this
    one kept."""
    s = _Shift(H, torch.float32, slots=len(lens))
    seqs = [s.sequence(n + 1, 10 * i) for i, n in enumerate(lens)]
    s.run([(q, 0, n, i) for i, (q, n) in enumerate(zip(seqs, lens))])
    s.run([(q, n, n + 1, i) for i, (q, n) in enumerate(zip(seqs, lens))], decode=True)


def test_shifted_streams_need_a_buffer_of_their_own(H):
    s = _Shift(H, torch.float32)
    x, y, *_ = s.sequence(4, 1)
    x, shift = x.to(DEV), H.StreamShift(s.share.to(DEV), s.prev, torch.arange(4, device=DEV), _i32([0]), _cu([4]))
    with pytest.raises(H.MvHipError, match="alias"):
        H.stream_update(2, s.nw.to(DEV), 1e-4, x=x, x_out=x, y=y.to(DEV), mix=s.mix.to(DEV), out_w=s.out.to(DEV), shift=shift)


# ---- gated running mean --------------------------------------------------------------------------------------------------
class _Gru:
    def __init__(self, H, n, dtype, slots=6, slow=0.0):
        self.H, self.n, self.dtype, self.slow = H, n, dtype, slow
        self.state = torch.full((2, slots, n), float("nan"), device=DEV)

    def inputs(self, t, seed):
        z = 3 * _rand(t, 3, self.n, seed=seed)
        z[:, 0] += self.slow
        return z.to(self.dtype)

    def want(self, ins):
        z, u, g = ins.double().unbind(1)
        return S.gru_scan(sigmoid(z), u) * silu(g)

    def _split(self, ins):
        wide = torch.zeros(ins.shape[0], 3 * self.n + 64, dtype=self.dtype, device=DEV)
        wide[:, :3 * self.n] = ins.flatten(1).to(DEV)
        out = torch.zeros(ins.shape[0], self.n + 64, dtype=self.dtype, device=DEV)[:, :self.n]
        return [wide[:, i * self.n:(i + 1) * self.n] for i in range(3)], out

    def prefill(self, parts, slots):
        """parts: [(inputs, start, stop)]"""
        lens = [hi - lo for _, lo, hi in parts]
        zug, out = self._split(torch.cat([ins[lo:hi] for ins, lo, hi in parts]))
        return self.H.gru_prefill(*zug, self.state, _i32(slots), _cu(lens), _cu([hi for _, _, hi in parts]), max(lens), out)

    def step(self, rows, lens, slots):
        zug, out = self._split(torch.stack([ins[t] for ins, t in rows]))
        return self.H.gru_step(*zug, self.state, _i32(slots), _i32(lens), out)


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("n", [64, 320, 1024])
def test_running_mean_of_prompts_portions_and_steps(H, dtype, n):
    """Whole prompts side by side; the same sequence cut anywhere beside others, on other slots; its last tokens one by one."""
    s = _Gru(H, n, dtype)
    a, b, c = (s.inputs(k, i) for i, k in enumerate((150, 65, 3)))
    wa, wb, wc = (s.want(v) for v in (a, b, c))
    o = s.prefill([(a, 0, 150), (b, 0, 65), (c, 0, 3)], [3, 0, -1])
    for got, want, what in ((o[:150], wa, "a"), (o[150:215], wb, "b"), (o[215:], wc, "no slot")):
        _close(got, want, dtype, what)
    o = s.prefill([(b, 0, 2), (a, 0, 71)], [5, 1])
    _close(o[2:], wa[:71], dtype, "first portion")
    _close(s.prefill([(a, 71, 73), (b, 2, 5)], [1, 5]), torch.cat([wa[71:73], wb[2:5]]), dtype, "two tokens")
    _close(s.prefill([(a, 73, 137)], [1]), wa[73:137], dtype, "third portion")
    for t in range(137, 150):                                             # decoding, beside another sequence that starts with a step
        rows = [(a, t), (c, t - 137)][:2 if t < 140 else 1]
        o = s.step(rows, [t + 1, t - 136][:len(rows)], [1, 4][:len(rows)])
        _close(o[0], wa[t], dtype, f"step {t}")
        if t < 140:
            _close(o[1], wc[t - 137], dtype, f"fresh step {t - 137}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("slow", [-9.0, 0.0, 9.0], ids=["slow", "medium", "nothing_kept"])
@pytest.mark.parametrize("lens", [(2000,), (5000, 17, 64, 1), (15, 16, 17, 31, 32, 33, 63, 64, 65, 127, 128, 129)], ids=str)
def test_running_mean_over_many_chunks(H, dtype, lens, slow):
    """What is remembered for thousands of tokens crosses every chunk's edge; many chunks ahead of the last one."""
    s = _Gru(H, 64, dtype, slots=16, slow=slow)
    ins = [s.inputs(n + 3, i) for i, n in enumerate(lens)]
    o = s.prefill([(v, 0, n) for v, n in zip(ins, lens)], list(range(len(lens))))
    _close(o, torch.cat([s.want(v)[:n] for v, n in zip(ins, lens)]), dtype, factor=3.0 if dtype == torch.float32 else 1.0)
    o = s.prefill([(v, n, n + 3) for v, n in zip(ins, lens)], list(range(len(lens))))   # the state they left
    _close(o, torch.cat([s.want(v)[n:] for v, n in zip(ins, lens)]), dtype, "after", factor=3.0 if dtype == torch.float32 else 1.0)


def test_a_first_token_is_remembered_to_the_end(H):
    """Gates that shut behind the first token: the state is that token's at every later position, whatever the chunks."""
    s = _Gru(H, 64, torch.float32)
    ins = s.inputs(1500, 1)
    ins[0, 0], ins[0, 1], ins[1:, 0] = 50.0, 3.0, -60.0
    g = ins[:, 2].double()
    o = s.prefill([(ins, 0, 1500)], [1])
    _close(o, 3.5 * silu(g), torch.float32)


def test_a_repeated_step_changes_nothing_and_padding_rows_keep_nothing(H):
    s = _Gru(H, 64, torch.bfloat16)
    ins = s.inputs(20, 3)
    want = s.want(ins)
    s.prefill([(ins, 0, 18)], [2])
    s.step([(ins, 18)], [19], [2])
    ahead = s.step([(ins, 19)], [20], [2])
    rest = [0, 1, 3, 4, 5]
    before = s.state[:, rest].clone()
    o = s.step([(ins, 19), (ins, 0), (ins, 0)], [20, 0, 7], [2, -1, -1])
    assert torch.equal(o[:1], ahead) and o[1].abs().sum() == 0
    _close(o[0], want[19], torch.bfloat16)
    assert torch.equal(torch.nan_to_num(s.state[:, rest], 7.0), torch.nan_to_num(before, 7.0))


# ---- attention ------------------------------------------------------------------------------------------------------------
def _aimed(nq, k, window, seed):
    """Queries of the last nq of len(k) tokens that point hard at the key just outside their window, the one just inside it and the
    first: a mask that is one off answers with another key's value."""
    nk, dim = k.shape
    q = _rand(nk, dim, seed=seed) * 0.3
    w = window or nk
    for i in range(nk):
        for j in (i - w, i - w + 1, 0):
            if 0 <= j <= i:
                q[i] += 4 * k[j] / k[j].norm()
    return q[nk - nq:]


def _case(nq, nk, heads, kv, d, window, dtype, seed):
    k, v = _rand(nk, kv, d, seed=seed), _rand(nk, kv, d, seed=seed + 1)
    q = torch.stack([_aimed(nq, k[:, h * kv // heads], window, seed + 2 + h) for h in range(heads)], 1)
    return q.to(dtype), k.to(dtype), v.to(dtype)


def _attend(q, k, v, scale, window):
    nq, nk = q.shape[0], k.shape[0]
    full = torch.zeros(nk, *q.shape[1:], dtype=torch.float64)
    full[nk - nq:] = q.double()
    return S.attend(full, k.double(), v.double(), scale, window_mask(nk, window or None))[nk - nq:]


def _paged(cases, bs, kv, d, dtype):
    nb = -(-max(k.shape[0] for _, k, _ in cases) // bs)
    pages = torch.randperm(len(cases) * nb, generator=torch.Generator().manual_seed(1)).int().view(-1, nb)
    kc, vc = (torch.zeros(len(cases) * nb, bs, kv, d, dtype=dtype) for _ in range(2))
    for s, (_, k, v) in enumerate(cases):
        for i in range(-(-k.shape[0] // bs)):
            part = slice(i * bs, (i + 1) * bs)
            kc[pages[s, i], :k[part].shape[0]], vc[pages[s, i], :k[part].shape[0]] = k[part], v[part]
    return kc.to(DEV), vc.to(DEV), pages.to(DEV)


def _gates(rows, heads, d, dtype, seed=77):
    """Gate rows inside wider ones; -> (device view, what the output is multiplied by)."""
    wide = _rand(rows, heads * d + 128, dtype=dtype, seed=seed) * 3
    return wide.to(DEV)[:, 64:64 + heads * d], sigmoid(wide.double()[:, 64:64 + heads * d]).view(rows, heads, d)


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("heads, kv, d", [(3, 1, 64), (2, 2, 128), (2, 1, 256)])
@pytest.mark.parametrize("window", [0, 1, 2, 33, 64, 65, 130])
def test_gated_prefill_attention(H, dtype, heads, kv, d, window):
    """Whole sequences and portions (the last queries of a sequence), several in one launch; keys packed and from pages."""
    scale, spans = 0.4, [(150, 150), (2, 97), (70, 300), (1, 1), (1, 66)]
    cases = [_case(a, b, heads, kv, d, window, dtype, 10 * i) for i, (a, b) in enumerate(spans)]
    q, k, v = (torch.cat([c[i] for c in cases]).to(DEV) for i in range(3))
    gate, open_ = _gates(q.shape[0], heads, d, dtype)
    want = torch.cat([_attend(*c, scale, window) for c in cases]) * open_
    mask = H.AttnMask(window, gate=gate)
    cq, ck = _cu([a for a, _ in spans]), _cu([b for _, b in spans])
    wide = torch.zeros(q.shape[0], heads * d + 64, dtype=dtype, device=DEV)
    got = H.prefill_varlen(q, k, v, cq, ck, 150, 300, scale, mask=mask, out=wide[:, :heads * d].view(-1, heads, d))
    _close(got, want, dtype, "packed", factor=2.0)
    assert wide[:, heads * d:].abs().sum() == 0
    kc, vc, pages = _paged(cases, 64, kv, d, dtype)
    got = H.prefill_varlen(q, None, None, cq, ck, 150, 300, scale, k_cache=kc, v_cache=vc, block_tables=pages, mask=mask)
    _close(got, want, dtype, "paged", factor=2.0)
    if dtype != torch.float32:
        got = H.prefill_varlen(q, k, v, cq, ck, 150, 300, scale, mask=mask, flags=H.MV_PREFILL_SIMPLE)
        _close(got, want, dtype, "vector kernel", factor=2.0)


def test_long_gated_prompts_take_the_eight_wave_kernel(H):
    n, window, dtype = 2200, 700, torch.bfloat16
    c = _case(n, n, 2, 1, 128, window, dtype, 1)
    gate, open_ = _gates(n, 2, 128, dtype)
    q, k, v = (t.to(DEV) for t in c)
    _close(H.prefill_varlen(q, k, v, _cu([n]), _cu([n]), n, n, 0.1, mask=H.AttnMask(window, gate=gate)), _attend(*c, 0.1, window) * open_, dtype, factor=2.0)


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("heads, kv, d", [(3, 3, 64), (8, 1, 64), (8, 1, 128), (34, 2, 128), (4, 4, 128), (2, 1, 256)])
@pytest.mark.parametrize("window", [0, 1, 33, 64, 65])
def test_gated_decode_attention(H, dtype, heads, kv, d, window):
    """Lengths just inside and just outside a window, a tile and a page; long contexts in parts; an empty row."""
    scale, w = 0.4, window or 33
    lens = sorted({1, 2, w, w + 1, max(w - 1, 1), 2 * w + 1, 64, 65, 257, 1100})
    cases = [_case(1, n, heads, kv, d, window, dtype, 10 * s) for s, n in enumerate(lens)]
    gate, open_ = _gates(len(lens) + 1, heads, d, dtype)
    want = torch.cat([_attend(*c, scale, window) for c in cases] + [torch.zeros(1, heads, d, dtype=torch.float64)]) * open_
    kc, vc, pages = _paged(cases, 64, kv, d, dtype)
    q = torch.cat([c[0] for c in cases] + [torch.ones(1, heads, d, dtype=dtype)]).to(DEV)
    tables, ctx, mask = torch.cat([pages, pages[:1]]), _i32(lens + [0]), H.AttnMask(window, gate=gate)
    for flags in [0] if dtype == torch.float32 else [0, H.MV_DECODE_VECTOR, H.MV_DECODE_MFMA, H.MV_DECODE_MFMA | H.MV_DECODE_KLDS_ON]:
        _close(H.paged_decode(q, kc, vc, tables, ctx, scale, flags=flags, mask=mask), want, dtype, f"flags {flags}", factor=2.0)
    for s in range(0, len(lens), 3):                                      # each row alone: the context in many parts
        got = H.paged_decode(q[s:s + 1], kc, vc, tables[s:s + 1], ctx[s:s + 1], scale, mask=H.AttnMask(window, gate=gate[s:s + 1]))
        _close(got, want[s:s + 1], dtype, f"length {lens[s]} alone", factor=2.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, kv, dim, d, pairs", [(6, 3, 40, 64, 11), (8, 1, 72, 128, 36), (4, 4, 128, 128, 16), (8, 2, 128, 128, None),
                                                      (2, 1, 200, 256, 1), (3, 1, 64, 64, None)])
def test_unit_length_behind_the_rotation_and_the_fused_decode_step(H, dtype, heads, kv, dim, d, pairs):
    """pairs None: the layout of whole halves.  The values are the keys as they came."""
    T, eps, scale = 9, 0.3, 0.3                                           # (an eps that matters)
    pad = lambda t: torch.nn.functional.pad(t, (0, d - dim)).to(dtype)
    q, k = pad(_rand(T, heads, dim, seed=1) * 2), pad(_rand(T, kv, dim, seed=2))
    lens = [1, 5, 64, 65, 100, 128, 129, 17, 2]
    n = d // 2 if pairs is None else pairs
    angle = torch.rand(140, n, generator=torch.Generator().manual_seed(3)) * 6.3
    pages = torch.arange(T * 3).int().view(T, 3)
    slots = torch.tensor([int(pages[i, (m - 1) // 64]) * 64 + (m - 1) % 64 for i, m in enumerate(lens)], dtype=torch.int32)
    kc, vc = (_rand(T * 3, 64, kv, d, dtype=dtype, seed=s).to(DEV) for s in (6, 7))
    kc[..., dim:] = 0
    pos = torch.tensor(lens) - 1
    args = (pos.to(DEV), angle.cos().to(DEV), angle.sin().to(DEV), None, None, eps)
    how = {"interleaved_pairs": pairs, "norm_dim": dim, "unit_norm": True}

    def want(x):
        x, c, s = x.double()[..., :dim], angle[pos].double().cos()[:, None], angle[pos].double().sin()[:, None]
        y = x.clone()
        u, v = (slice(0, n), slice(n, 2 * n)) if pairs is None else (slice(0, 2 * n, 2), slice(1, 2 * n, 2))
        y[..., u], y[..., v] = x[..., u] * c - x[..., v] * s, x[..., v] * c + x[..., u] * s
        return rms(y, eps)
    k1, v1 = kc.clone(), vc.clone()
    qr, kr = H.rope_qk_store(q.to(DEV), k.to(DEV), k.to(DEV), *args, k_cache=k1, v_cache=v1, slot_mapping=slots.to(DEV), **how)
    _close(qr[..., :dim], want(q), dtype, "q")
    _close(kr[..., :dim], want(k), dtype, "k")
    assert qr[..., dim:].abs().sum() == 0 and kr[..., dim:].abs().sum() == 0
    flat = slots.long()
    assert torch.equal(k1.view(-1, kv, d)[flat], kr) and torch.equal(v1.view(-1, kv, d)[flat].cpu(), k)
    gate, _ = _gates(T, heads, d, dtype)
    mask = H.AttnMask(50, gate=gate)
    base = H.paged_decode(qr, k1, v1, pages.to(DEV), _i32(lens), scale, mask=mask)
    got = H.rope_paged_decode(q.to(DEV), k.to(DEV), k.to(DEV), *args, slots.to(DEV), kc, vc, pages.to(DEV), _i32(lens), scale, mask=mask, **how)
    if got is not None:                                                   # (layouts that the one launch takes)
        _close(got, base.double().cpu(), dtype)
        assert torch.equal(kc, k1) and torch.equal(vc, v1)
    else:
        assert dtype == torch.float32 or (d != 128 and heads // kv > 4)
    with pytest.raises(H.MvHipError):                                     # a weight belongs to the other norm
        H.rope_qk_store(q.to(DEV), k.to(DEV), k.to(DEV), *args[:3], torch.ones(d, dtype=dtype, device=DEV),
                        torch.ones(d, dtype=dtype, device=DEV), eps, **how)


# ---- feed-forward ---------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
def test_gelu_with_the_error_function(H, dtype):
    z = torch.cat([torch.linspace(-9, 9, 1600), torch.tensor([0.0, 1e-4, -1e-4, 40.0, -40.0, 300.0, -300.0, 1e-20])]).view(8, -1)[:, :200].to(dtype)
    want = S.gelu(z.double())
    x = z.to(DEV)
    got = H.gelu_erf(x)
    tol = 1e-6 if dtype == torch.float32 else 1e-2 if dtype == torch.bfloat16 else 2e-3
    assert ((got.double().cpu() - want).abs() <= tol * want.abs() + 4e-7).all()
    assert torch.equal(H.gelu_erf(x, out=x), got) and torch.equal(x, got)


@pytest.mark.parametrize("m, n, k", [(1, 80, 256), (16, 64, 512), (33, 208, 192), (200, 512, 320), (40, 128, 256), (600, 96, 64)])
@pytest.mark.parametrize("bias", [False, True])
def test_projections_with_gelu_behind_them(H, m, n, k, bias):
    from minivllm_amd.layers import Segment, SegmentedLinear
    from minivllm_amd.layers.linear import gelu_linear

    dtype = torch.bfloat16
    lin = SegmentedLinear(k, [Segment("up", n)], split="out", bias=bias)
    x, w, b = _rand(m, k, dtype=dtype, seed=1), _rand(n, k, seed=2) * k ** -0.5, _rand(n, seed=3)
    lin.weight_loader(lin.weight, w, "up")
    if bias:
        lin.weight_loader(lin.bias, b, "up")
    lin = lin.to(DEV, dtype)
    lin.pack_for_decode()
    want = S.gelu(torch.nn.functional.pad(x, (0, lin.weight.shape[1] - k)).double() @ lin.weight.double().cpu().T + (lin.bias.double().cpu() if bias else 0))
    xp = torch.nn.functional.pad(x, (0, lin.weight.shape[1] - k)).to(DEV)
    _close(gelu_linear(xp, lin), want, dtype)
    _close(lin(xp), xp.double().cpu() @ lin.weight.double().cpu().T + (lin.bias.double().cpu() if bias else 0), dtype, "plain")
    wp, full = lin.weight_packed, lin.weight.shape
    for got in ([H.linear_small_m(xp, lin.weight, lin.bias, shape=H.MV_LINEAR_GELU_ERF, packed=p) for p in (None, wp)] if m <= 64 and k >= 256 else []) + (
            [H.linear_narrow(xp, wp, full[0], lin.bias, shape=H.MV_LINEAR_GELU_ERF)] if full[0] <= 256 and full[1] >= 256 else []) + (
            [H.linear_mid_m(xp, wp, full[0], lin.bias, H.MV_LINEAR_GELU_ERF)] if m <= 512 else []):
        _close(got, want, dtype, "epilogue")


@pytest.mark.parametrize("dtype", DTYPES + [torch.float16])
@pytest.mark.parametrize("T, K, R, top", [(1, 64, 1, 1), (37, 256, 12, 1), (16, 192, 9, 3), (50, 128, 96, 8), (5, 64, 320, 6), (3, 64, 6, 6)])
def test_sigmoid_router_without_a_correction(H, dtype, T, K, R, top):
    x, w = _rand(T, K, dtype=dtype, seed=1), (_rand(R, K, seed=2) * 2 * K ** -0.5).to(dtype)
    ids, weights = H.moe_route(x.to(DEV), w.to(DEV), None, top, sigmoid=True, raw=True)
    want_ids, want = S.route(x.double() @ w.double().T, top)
    full = lambda i, v: torch.zeros(T, R, dtype=torch.float64).scatter(1, i.long().cpu(), v.double().cpu())
    _close(full(ids, weights), full(want_ids, want), torch.float32, factor=5.0)
    ids2, weights2 = H.moe_route(x.to(DEV), w.to(DEV), None, top, sigmoid=True, scale=1.5)     # divided by their sum
    assert torch.equal(ids, ids2)
    _close(weights2, (weights / weights.sum(-1, keepdim=True) * 1.5).double().cpu(), torch.float32)


@pytest.mark.parametrize("dtype, tile_m", [(torch.float32, 16)] + [(torch.bfloat16, m) for m in (16, 32, 64, 128, 256)] + [(torch.float16, 128), (torch.float16, 256)])
@pytest.mark.parametrize("T, width, ff, experts, top", [(3, 64, 64, 4, 2), (90, 256, 192, 5, 2), (300, 192, 320, 3, 1)])
def test_weighed_inputs_of_clamped_experts(H, dtype, tile_m, T, width, ff, experts, top):
    """The weight is inside the clamps and the gate: on the output it would give something else."""
    limit, x = 0.8, _rand(T, width, dtype=dtype, seed=1) * 2
    gu, dn = ((_rand(experts, *s, seed=i) * s[-1] ** -0.5).to(dtype) for i, s in ((2, (2, ff, width)), (3, (width, ff))))
    ids = torch.stack([torch.randperm(experts, generator=torch.Generator().manual_seed(t))[:top] for t in range(T)]).int()
    weights = torch.rand(T, top, generator=torch.Generator().manual_seed(5)) + 0.05
    g = H.moe_group(ids.to(DEV), experts, tile_m, weights.to(DEV))
    place = g.place.cpu().view(T, top)
    assert torch.equal(g.weights.cpu()[place.long()], weights)
    form = (lambda t: t.to(DEV)) if dtype == torch.float32 else (lambda t: H.pack_weight(t.to(DEV).view(-1, t.shape[-1])))
    z = H.moe_linear(x.to(DEV), form(gu), ff, g, H.clamped_glu(limit), gather=True, experts=experts, in_scale=g.weights)
    y = H.moe_linear(z, form(dn), width, g, experts=experts, in_scale=g.weights)             # (any product takes a factor)
    zc, yc = z.cpu(), y.cpu()
    for t in range(0, T, 7):
        for k in range(top):
            e, i, c = int(ids[t, k]), int(place[t, k]), weights[t, k].double()
            a, b = (gu[e, j].double() @ (c * x[t].double()) for j in (0, 1))
            a, b = a.clamp(max=limit), b.clamp(-limit, limit)
            _close(zc[i], a * sigmoid(1.702 * a) * (b + 1), dtype, f"gated {t} {e}", factor=2.0)
            _close(yc[i], c * (dn[e].double() @ zc[i].double()), dtype, f"down {t} {e}", factor=2.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [1, 20, 700])
def test_an_expert_layer_as_a_whole(H, dtype, T):
    from minivllm_amd.layers import ExpertMLP

    width, ff, experts, top, limit = 100, 40, 6, 2, 1.2
    cfg = {"router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}
    w = {"router": _rand(experts, width, seed=1) * 0.2}
    layer = ExpertMLP(width, experts, 0, top, 1, 1, 1.0, ff, act=H.clamped_glu(limit), sigmoid=True, corrected=False, raw_weights=True, weigh_inputs=True)
    for e in range(experts):
        for i, (n, s) in enumerate({"gate": (ff, width), "up": (ff, width), "down": (width, ff)}.items()):
            w[f"e{e}.{n}"] = _rand(*s, seed=10 * e + i + 2) * s[1] ** -0.5
            layer._load(layer.down if n == "down" else layer.gate_up, w[f"e{e}.{n}"].bfloat16().float(), (e, n))
    layer.router.data[:, :width] = w["router"].bfloat16()
    layer = layer.to(DEV, dtype)
    layer.finish_weights()
    x = torch.nn.functional.pad(_rand(T, width, seed=99), (0, 28)).to(dtype)
    shared, (y, place, weights) = layer(x.to(DEV))
    assert shared is None and weights is None
    got = y.double().cpu()[place.long().cpu()].view(T, top, -1).sum(1)[:, :width]
    want = S.moe(x.double()[:, :width], cfg, {k: v.bfloat16().double() for k, v in w.items()}, "")
    _close(got, want, dtype, factor=2.0)


# ---- whole models ------------------------------------------------------------------------------------------------------
def _tokens(n, vocab, seed):
    return _ints(vocab, n, seed).tolist()


_ORACLE = {}


def _logits(name, toks, dtype=torch.float32):
    """The plain model's logits (fp64, cached: several tests ask for the same sequences)."""
    calm = dtype != torch.float32
    key = (name, tuple(toks), calm)
    if key not in _ORACLE:
        _ORACLE[key] = S.forward(CONFIGS[name], sharp_weights(name, calm=calm), toks, torch.float64)
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
    name = "large_heads"
    _alone(replayers(name, torch.float32), _tokens(600, CONFIGS[name]["vocab"], 9), [5], torch.float32, name)


# ---- generation --------------------------------------------------------------------------------------------------------
@functools.lru_cache(None)
def _greedy(name, prompt, n):
    """Greedy continuation by the plain model; every choice must be clear (by a margin fp32 rounding cannot move)."""
    cfg, toks, w = CONFIGS[name], list(prompt), sharp_weights(name)
    for _ in range(n):
        top = S.forward(cfg, w, toks, torch.float64)[-1].topk(2)
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
    eos = next(t for f in full for t in f[6:12] if t not in f[:6] and any(t not in g for g in full))
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
