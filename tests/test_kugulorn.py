"""Kugulorn without a GPU: configuration, weight placement (padding, tensor-parallel shards), state slots beside cache blocks, the
executor's key spans, and the plain implementation's own consistency."""
import copy
import math

import pytest
import torch

from kugulorn_configs import CONFIGS, config, latent, mamba, sharp_weights, write_checkpoint
from oracle import kugulorn as K


@pytest.fixture(autouse=True)
def _single_rank():
    from minivllm_amd import parallel_state

    parallel_state.reset_tensor_parallel()
    yield
    parallel_state.reset_tensor_parallel()


def _rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


# ---- the plain implementation ------------------------------------------------------------------------------------------
def test_window_counts_the_query_itself():
    m = K.window_mask(6, 3)
    assert m[0].nonzero().flatten().tolist() == [0] and m[4].nonzero().flatten().tolist() == [2, 3, 4]
    assert K.window_mask(4, 1).equal(torch.eye(4, dtype=torch.bool)) and K.window_mask(5, None)[4].all()


def test_convolution_by_hand():
    x, w, b = _rand(7, 3, seed=1), _rand(3, 4, seed=2), _rand(3, seed=3)
    y = K.causal_conv(x, w, b)
    for t in range(7):
        for c in range(3):
            want = b[c] + sum(x[t - k, c] * w[c, 3 - k] for k in range(4) if t - k >= 0)
            assert y[t, c].item() == pytest.approx(want.item())


def test_recurrence_equals_its_unrolled_sum():
    """y_t = sum_j exp(sum of log decays j+1..t) dt_j (c_t . b_j) x_j + d x_t, per head with its group's b and c."""
    T, H, P, G, N = 9, 4, 3, 2, 5
    x, b, c, dt = _rand(T, H, P, seed=1), _rand(T, G, N, seed=2), _rand(T, G, N, seed=3), _rand(T, H, seed=4).abs()
    a, d = _rand(H, seed=5), _rand(H, seed=6)
    y = K.ssm_scan(x, b, c, dt, a, d)
    for t in (0, 1, 8):
        for h in range(H):
            want = d[h] * x[t, h]
            for j in range(t + 1):
                decay = torch.exp(-torch.exp(a[h]) * dt[j + 1:t + 1, h].sum())
                want = want + decay * dt[j, h] * (c[t, h // 2] @ b[j, h // 2]) * x[j, h]
            assert torch.allclose(y[t, h], want, atol=1e-12)


def test_gate_comes_before_the_parted_norm():
    y, z, w = _rand(2, 12, seed=1), _rand(2, 12, seed=2), _rand(12, seed=3)
    got = K.gated_group_norm(y, z, w, 3, 1e-3)
    g = y * z * torch.sigmoid(z)
    for i in range(3):
        part = g[:, 4 * i:4 * i + 4]
        want = part / (part.pow(2).mean(1, keepdim=True) + 1e-3).sqrt() * w[4 * i:4 * i + 4]
        assert torch.allclose(got[:, 4 * i:4 * i + 4], want)


def test_clamped_gate_by_hand():
    g, u = torch.tensor([-30.0, 0.5, 9.0]).double(), torch.tensor([-9.0, 0.25, 9.0]).double()
    y = K.clamped_glu(g, u, 2.0)
    sig = lambda v: 1 / (1 + math.exp(-1.702 * v))
    assert y.tolist() == pytest.approx([-30 * sig(-30) * -1, 0.5 * sig(0.5) * 1.25, 2 * sig(2) * 3])


def test_a_shared_layer_uses_the_other_layers_rows():
    cfg = config(32, 40, [latent(2, 8, 4, 8, 8, 16), latent(3, 12, 4, 20, 8, 16, kv_from=0)])
    w, toks = K.random_model(cfg), list(range(20))
    assert "l1.mix.dkv" not in w and "l1.mix.uk" in w
    a = K.forward(cfg, w, toks)
    w2 = dict(w, **{"l0.mix.dkv.norm": w["l0.mix.dkv.norm"] * 2})
    w3 = dict(w2, **{"l0.mix.uk": w["l0.mix.uk"] / 2, "l0.mix.uv": w["l0.mix.uv"] / 2})     # layer 0 itself unchanged
    assert not torch.allclose(a, K.forward(cfg, w3, toks), atol=1e-3)
    w4 = dict(w3, **{"l1.mix.uk": w["l1.mix.uk"] / 2, "l1.mix.uv": w["l1.mix.uv"] / 2})
    assert torch.allclose(a, K.forward(cfg, w4, toks), atol=1e-9)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_longer_sequence_does_not_change_earlier_logits(name):
    cfg = CONFIGS[name]
    toks, w = torch.arange(75) % cfg["vocab"], sharp_weights(cfg)
    a, b = K.forward(cfg, w, toks), K.forward(cfg, w, toks[:51])
    assert torch.allclose(a[:51], b, atol=1e-9)


# ---- configuration -----------------------------------------------------------------------------------------------------
def test_config_is_read_and_served_by_the_registry(tmp_path):
    from minivllm_amd.config import Config
    from minivllm_amd.engine.inference_executor import kv_planes, latent_modules, state_modules
    from minivllm_amd.glue import create_model

    cfg = CONFIGS["odd"]
    c = Config(write_checkpoint(tmp_path / "m", cfg, K.random_model(cfg)), max_model_len=640)
    h = c.hf_config
    assert (h.vocab_size, h.hidden_size, h.residual_mult, h.norm_eps) == (301, 200, 0.37, 3e-5)
    assert h.num_hidden_layers == 5 and h.max_position_embeddings == 640 and h.recurrent_state
    a = h.layers[0].mixer
    assert (a.heads, a.dim, a.rot_dim, a.vdim, a.q_rank, a.kv_rank, a.window, a.rot_base, a.scale) == (5, 20, 12, 24, 40, 48, 37, 500.0, 0.2)
    s = h.layers[1].mixer
    assert (s.heads, s.vdim, s.state, s.groups, s.taps, s.norm_groups) == (3, 20, 24, 1, 4, 5)
    assert h.layers[0].mlp.limit == 1.5 and h.layers[2].mlp is None and h.layers[3].mlp.ff == 72 and h.layers[2].mixer.kv_from == 0
    assert h.weight_shapes() == K.tensor_shapes(cfg)
    m = create_model(h)
    assert type(m).__name__ == "KugulornForCausalLM" and not kv_planes(m)
    # one plane per layer with latents of its own; a shared plane reaches as far back as the widest of its readers
    assert [(x.row_cols, x.span_window) for x in latent_modules(m)] == [(64 + 32, 90), (128 + 32, 0)]
    assert m.l2.mix.owner is m.l0.mix
    assert [x.state_shapes(torch.bfloat16)["ssm_state"][0] for x in state_modules(m)] == [(3, 32, 32), (6, 64, 48)]
    assert not create_model_config_is_recurrent(config(32, 40, [latent(2, 8, 4, 8, 8, 16)]))


def create_model_config_is_recurrent(raw):
    from minivllm_amd.native_configs import KugulornConfig

    return KugulornConfig(raw).recurrent_state


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][0].update(type="other"), "layer type"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "feed-forward"),
    (lambda c: c["layers"][0]["mlp"].pop("limit"), "missing 'limit'"),
    (lambda c: c["layers"][0]["mlp"].update(limit=-1.0), "limit must be positive"),
    (lambda c: c["layers"][0]["mixer"].update(rot_dim=11), "rot_dim must be even"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "positive integer"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "missing 'scale'"),
    (lambda c: c["layers"][1]["mixer"].update(groups=2), "do not divide"),
    (lambda c: c["layers"][1]["mixer"].update(norm_groups=7), "norm groups"),
    (lambda c: c["layers"][1]["mixer"].pop("conv"), "missing 'conv'"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=4), "kv_from"),
    (lambda c: c["layers"][4]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=50), "must equal"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(base=1.5), "must equal"),
])
def test_config_errors_name_the_field(tmp_path, change, text):
    from minivllm_amd.native_configs import load_native_config

    cfg = copy.deepcopy(CONFIGS["odd"])
    change(cfg)
    with pytest.raises(ValueError, match=text):
        load_native_config(write_checkpoint(tmp_path / "m", cfg, {}))


# ---- weights -----------------------------------------------------------------------------------------------------------
def _built(tmp_path, cfg, weights):
    from minivllm_amd.glue import create_model
    from minivllm_amd.native_configs import load_native_config
    from minivllm_amd.utils.loader import load_model

    d = write_checkpoint(tmp_path / "m", cfg, weights)
    c = load_native_config(d)
    c.max_position_embeddings = 128
    m = create_model(c)
    load_model(m, d)
    return m


def test_weights_land_in_the_merged_matrices_with_zero_padding(tmp_path):
    cfg = CONFIGS["odd"]
    w = K.random_model(cfg, 3)
    m = _built(tmp_path, cfg, w)
    f = {k: v.float() for k, v in w.items()}
    a = m.l0.mix                                   # 5 heads of 20 + 12, rows [20 -> 32 | 12 -> 32], width 200 at 256
    assert a.down.offsets == {"dq": 0, "latent": 64, "rot": 128} and a.down.weight.shape == (192, 256)
    assert torch.equal(a.down.weight[:40, :200], f["l0.mix.dq"]) and torch.equal(a.down.weight[64:112, :200], f["l0.mix.dkv"][:48])
    assert torch.equal(a.down.weight[128:140, :200], f["l0.mix.dkv"][48:]) and a.down.weight[140:].abs().sum() == 0
    uq = a.uq.weight[:5 * 64, :40].view(5, 64, 40)
    want = f["l0.mix.uq"].view(5, 32, 40)
    assert torch.equal(uq[:, :20], want[:, :20]) and torch.equal(uq[:, 32:44], want[:, 20:])
    assert uq[:, 20:32].abs().sum() == 0 and uq[:, 44:].abs().sum() == 0
    a.finish_weights()
    assert a.uk_t.shape == (5, 64, 32) and torch.equal(a.uk_t[:, :48, :20], f["l0.mix.uk"].view(5, 20, 48).transpose(1, 2))
    assert a.uv.shape == (5, 64, 64) and torch.equal(a.uv[:, :24, :48], f["l0.mix.uv"].view(5, 24, 48)) and a.uv[:, 24:].abs().sum() == 0
    s = m.l1.mix                                   # 3 heads of 20 -> 32, state 24 -> 32
    at, src = s.in_proj.offsets, f["l1.mix.in"]
    assert at == {"z": 0, "x": 128, "b": 256, "c": 320, "dt": 384} and s.shape == (3, 1, 32, 32, 128, 192)
    x = s.in_proj.weight[128:224, :200].view(3, 32, 200)
    assert torch.equal(x[:, :20], src[60:120].view(3, 20, 200)) and x[:, 20:].abs().sum() == 0
    assert torch.equal(s.in_proj.weight[256:280, :200], src[120:144]) and torch.equal(s.in_proj.weight[320:344, :200], src[144:168])
    assert torch.equal(s.in_proj.weight[384:387, :200], src[168:]) and s.in_proj.weight[387:].abs().sum() == 0
    conv = f["l1.mix.conv"]
    assert s.conv.shape == (4, 224) and torch.equal(s.conv[:, 32:52], conv[20:40].T) and s.conv[:, 20:32].abs().sum() == 0
    assert torch.equal(s.conv[:, 128:152], conv[60:84].T) and torch.equal(s.conv_b[192:216], f["l1.mix.conv.b"][84:])
    assert torch.equal(s.norm.view(3, 32)[:, :20].reshape(-1), f["l1.mix.norm"]) and torch.equal(s.A_log, f["l1.mix.A_log"])
    assert torch.equal(m.l0.ls1[:200], f["l0.ls1"]) and torch.equal(m.l0.norm2b[:200], f["l0.norm2b"]) and m.l1.mlp is None
    assert torch.equal(m.head.weight[:, :200], f["head"]) and torch.equal(m.final_norm[:200], f["final.norm"])


def test_a_missing_or_misshapen_tensor_is_an_error(tmp_path):
    cfg = CONFIGS["states"]
    w = K.random_model(cfg)
    with pytest.raises(ValueError, match="l1.mix.A_log"):
        _built(tmp_path / "a", cfg, {k: v for k, v in w.items() if k != "l1.mix.A_log"})
    with pytest.raises(ValueError, match="l0.mix.in"):
        _built(tmp_path / "b", cfg, dict(w, **{"l0.mix.in": w["l0.mix.in"][:-1].contiguous()}))


def test_tensor_parallel_shards_are_the_whole_layer(tmp_path):
    """Two ranks' shards hold each head, group and channel of the unsharded layer once; what cannot be split is refused."""
    from minivllm_amd import parallel_state as ps

    cfg = config(96, 40, [mamba(4, 16, 32, 2, 4, 2), latent(4, 32, 8, 32, 24, 48, 20, ff=48)])
    w = K.random_model(cfg, 5)
    f = {k: v.float() for k, v in w.items()}
    parts = []
    for rank in range(2):
        ps.init_tensor_parallel(rank, 2)
        try:
            parts.append(_built(tmp_path / str(rank), cfg, w))
        finally:
            ps.reset_tensor_parallel()
    inner = 64
    for rank, m in enumerate(parts):
        s, a = m.l0.mix, m.l1.mix
        assert (s.heads, s.groups, s.norm_groups, a.heads) == (2, 1, 1, 2)
        half = slice(32 * rank, 32 * rank + 32)
        src, at = f["l0.mix.in"], s.in_proj.offsets
        assert torch.equal(s.in_proj.weight[:32, :96], src[half]) and torch.equal(s.in_proj.weight[at["x"]:at["x"] + 32, :96], src[inner:2 * inner][half])
        assert torch.equal(s.in_proj.weight[at["b"]:at["b"] + 32, :96], src[2 * inner:][half])
        assert torch.equal(s.in_proj.weight[at["dt"]:at["dt"] + 2, :96], src[-4:][2 * rank:2 * rank + 2])
        assert torch.equal(s.conv[:, :32], f["l0.mix.conv"][half].T) and torch.equal(s.D, f["l0.mix.D"][2 * rank:2 * rank + 2])
        assert torch.equal(s.norm, f["l0.mix.norm"][half]) and torch.equal(s.o.weight[:96, :32], f["l0.mix.o"][:, half])
        assert torch.equal(a.down.weight[:24, :96], f["l1.mix.dq"])                        # the latents are replicated
        uk = a.ukv.weight[:64].view(2, 32, 64)[:, :, :48]
        assert torch.equal(uk, f["l1.mix.uk"].view(4, 32, 48)[2 * rank:2 * rank + 2])
        assert torch.equal(a.o.weight[:96].view(96, 2, 64)[:, :, :32], f["l1.mix.o"].view(96, 4, 32)[:, 2 * rank:2 * rank + 2])
    ps.init_tensor_parallel(0, 2)
    with pytest.raises(ValueError):
        _built(tmp_path / "g", config(96, 40, [mamba(4, 16, 32, 1)]), w)


# ---- sequences, blocks and state slots -----------------------------------------------------------------------------------
def _seq(n, tok=1):
    from minivllm_amd.engine.sequence import Sequence

    return Sequence([tok] * n, block_size=64)


def test_state_slots_come_and_go_with_the_blocks():
    from minivllm_amd.engine.block_manager import BlockManager

    bm = BlockManager(8, 64, state_slots=2)
    a, b, c = _seq(70), _seq(3), _seq(3)
    bm.reserve(a)
    bm.allocate(b)
    assert (a.state_slot, b.state_slot) == (0, 1) and not bm.can_allocate(c)
    with pytest.raises(RuntimeError, match="state slots"):
        bm.reserve(c)
    assert c.block_table == []
    a.extend([2] * 3)
    bm.reserve(a)
    assert a.state_slot == 0                                             # kept while the sequence lives
    bm.deallocate(a)
    assert a.state_slot == -1 and bm.can_allocate(c)
    bm.allocate(c)
    assert c.state_slot == 0


def test_prompts_of_recurrent_models_share_no_blocks():
    from minivllm_amd.engine.block_manager import BlockManager

    for slots, cached in ((0, 64), (4, 0)):
        bm = BlockManager(8, 64, state_slots=slots)
        a, b = _seq(100), _seq(100)
        bm.allocate(a)
        bm.allocate(b)
        assert b.num_cached_tokens == cached and (a.block_table[0] == b.block_table[0]) == bool(cached)


def test_the_scheduler_waits_for_a_slot_and_preemption_gives_one_back():
    from types import SimpleNamespace

    from minivllm_amd.engine.scheduler import Scheduler

    cfg = SimpleNamespace(max_num_seqs=2, max_num_batched_tokens=512, eos=-1, num_kvcache_blocks=16, kvcache_block_size=64,
                          max_model_len=512, hf_config=SimpleNamespace(recurrent_state=True))
    s = Scheduler(cfg)
    seqs = [_seq(10) for _ in range(3)]
    for q in seqs:
        s.add(q)
    batch, prefill = s.schedule()
    assert prefill and batch == seqs[:2]
    s.postprocess(batch, [1, 1])
    assert s.schedule() == (seqs[:2], False)                             # the third waits
    s.running.remove(seqs[1])
    s.preempt(seqs[1])
    assert seqs[1].state_slot == -1 and s.block_manager.states.num_free == 1


def test_batch_inputs_carry_the_slots_and_padding_rows_have_none():
    import pickle

    from minivllm_amd.engine.block_manager import BlockManager
    from minivllm_amd.engine.input_builder import InputBuilder

    bm, ib = BlockManager(8, 64, state_slots=4), InputBuilder(64, 4, 256, 512)
    seqs = [_seq(5), _seq(70)]
    for q in reversed(seqs):
        bm.allocate(q)
    assert ib.prefill(seqs).state_slots.tolist() == [1, 0]
    inp = ib.decode(seqs, pad_to=4)
    assert inp.state_slots.tolist() == [1, 0] and ib.pack_view(ib.decode_pack, "state").tolist() == [1, 0, -1, -1]
    assert pickle.loads(pickle.dumps(seqs[0])).state_slot == 1


def test_key_spans_reach_exactly_as_far_as_the_window():
    from minivllm_amd.engine.inference_executor import InferenceExecutor

    ex = object.__new__(InferenceExecutor)
    ex.latents, ex.span_windows, ex.device = [object()], [0, 10], torch.device("cpu")
    a, b = _seq(50), _seq(7)
    a.num_cached_tokens = 30
    spans = ex._key_spans([a, b], 0)
    cu, first, total, longest = spans[10]                                # token 30 sees 21 .. 30
    assert cu.tolist() == [0, 29, 36] and first.tolist() == [21, 0] and (total, longest) == (36, 29)
    assert spans[0][0].tolist() == [0, 50, 57] and spans[0][1].tolist() == [0, 0]
    assert ex._key_spans([b], 0) is None and ex._key_spans([a], 1) is None
