"""Pununex without a GPU: configuration, weight placement (padding, low-rank blocks, experts), state shapes, and the plain
implementation's own consistency."""
import copy
import math

import pytest
import torch

from oracle import pununex as P
from pununex_configs import CONFIGS, RANKS, attention, config, delta, dense, layer, moe, parallel, sharp_weights, write_checkpoint


@pytest.fixture(autouse=True)
def _single_rank():
    from minivllm_amd import parallel_state

    parallel_state.reset_tensor_parallel()
    yield
    parallel_state.reset_tensor_parallel()


def _rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


# ---- the plain implementation ------------------------------------------------------------------------------------------
def test_window_keeps_the_first_tokens():
    m = P.window_mask(8, 3, 2)
    assert m[1].nonzero().flatten().tolist() == [0, 1] and m[7].nonzero().flatten().tolist() == [0, 1, 5, 6, 7]
    assert P.window_mask(4, 1).equal(torch.eye(4, dtype=torch.bool)) and P.window_mask(5, None, 3)[4].all()


def test_the_sink_takes_weight_and_gives_nothing():
    q, k, v = _rand(1, 2, 4, seed=1), _rand(5, 1, 4, seed=2), _rand(5, 1, 3, seed=3)
    q = torch.cat([torch.zeros(4, 2, 4, dtype=torch.float64), q])
    sink, mask = torch.tensor([0.7, -40.0], dtype=torch.float64), P.window_mask(5, None)
    o = P.sink_attention(q, k, v, 0.5, 2.0, sink, mask)[4]
    for h in range(2):
        s = 2.0 * torch.tanh((k[:, 0] @ q[4, h]) * 0.5 / 2.0)
        e = torch.exp(s)
        assert torch.allclose(o[h], (e @ v[:, 0]) / (e.sum() + math.exp(sink[h])))
    assert not torch.allclose(o[0] / o[0].norm(), o[0]) and o[0].norm() < P.sink_attention(q, k, v, 0.5, 2.0, sink - 99, mask)[4, 0].norm()


def test_delta_rule_replaces_what_a_key_holds():
    """beta 1, no decay, orthogonal keys: a state that answers with the last value written under a key."""
    k = torch.eye(4, dtype=torch.float64)[[0, 1, 0, 2]][:, None]
    v, one = _rand(4, 1, 3, seed=1), torch.ones(4, 1, dtype=torch.float64)
    o = P.delta_scan(k[[0, 1, 1, 0]], k, v, one, torch.ones(4, 1, 4, dtype=torch.float64))[:, 0]
    assert torch.allclose(o[0], v[0, 0]) and torch.allclose(o[1], v[1, 0]) and torch.allclose(o[2], v[1, 0]) and torch.allclose(o[3], v[2, 0])


def test_delta_rule_equals_its_matrix_form():
    """S_t = (I - beta k k^T) diag(g) S_{t-1} + beta k v^T, and the read-out behind the write."""
    T, H, D, V = 7, 2, 4, 3
    q, k, v, beta, g = _rand(T, H, D, seed=1), P.unit(_rand(T, H, D, seed=2)), _rand(T, H, V, seed=3), torch.sigmoid(_rand(T, H, seed=4)), torch.sigmoid(_rand(T, H, D, seed=5))
    o = P.delta_scan(q, k, v, beta, g)
    for h in range(H):
        s = torch.zeros(D, V, dtype=torch.float64)
        for t in range(T):
            b, kk = beta[t, h], k[t, h][:, None]
            s = (torch.eye(D) - b * kk @ kk.T) @ (g[t, h][:, None] * s) + b * kk @ v[t, h][None]
            assert torch.allclose(o[t, h], s.T @ q[t, h])


def test_layer_norm_and_pairs_by_hand():
    x, w, b = torch.tensor([[1.0, 3.0]]).double(), torch.tensor([2.0, 1.0]).double(), torch.tensor([0.5, 0.0]).double()
    d = 1 / math.sqrt(1 + 0.25)
    assert P.layer_norm(x, w, b, 0.25)[0].tolist() == pytest.approx([-2 * d + 0.5, d])
    assert P.bigram_rows([5, 2, 9], 7, 3, 10) == [7, (5 * 3 + 2 * 10) % 7, (2 * 3 + 9 * 10) % 7]


def test_routing_by_groups():
    s = torch.tensor([[0.05, 0.30, 0.25, 0.10, 0.20, 0.10]]).double()
    z, none = s.log(), torch.zeros(6).double()
    ids, w = P.route(z, none, 2, 1, 1, 3.0)
    assert ids.tolist() == [[1, 2]] and w[0].tolist() == pytest.approx([0.9 / 0.55, 0.75 / 0.55])
    ids, _ = P.route(z, none, 2, 3, 1, 1.0)                              # groups (0 1) (2 3) (4 5)
    assert ids.tolist() == [[1, 0]]
    corr = torch.tensor([-1.0, -1.0, -1.0, -1.0, -0.9, -1.0]).double()    # every choice score negative; the weights do not see it
    ids, w = P.route(z, corr, 2, 3, 1, 1.0)
    assert ids.tolist() == [[4, 5]] and w[0].tolist() == pytest.approx([2 / 3, 1 / 3])


def test_identity_experts_return_their_input():
    cfg = config(32, 16, [layer(delta(1, 1, 8, 8), moe(2, 2, 16, identity=1, scale=0.5))])
    w = {k: v.double() for k, v in P.random_model(cfg).items()}
    w["l0.mlp.correction"] = torch.tensor([0.0, -9.0, 9.0]).double()       # expert 0 and the identity
    h = _rand(3, 32, seed=1)
    s = torch.softmax(h @ w["l0.mlp.router"].T, -1)[:, [0, 2]]
    s = s / s.sum(1, keepdim=True) * 0.5
    want = s[:, :1] * P.gated_mlp(h, w, "l0.mlp.e0.", P.silu) + s[:, 1:] * h
    assert torch.allclose(P.moe(h, cfg["layers"][0]["mlp"], w, "l0.mlp."), want)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_longer_sequence_does_not_change_earlier_logits(name):
    cfg = CONFIGS[name]
    toks, w = torch.arange(75) % cfg["vocab"], sharp_weights(name)
    a, b = P.forward(cfg, w, toks), P.forward(cfg, w, toks[:51])
    assert torch.allclose(a[:51], b, atol=1e-9)


# ---- configuration -----------------------------------------------------------------------------------------------------
def test_config_is_read_and_served_by_the_registry(tmp_path):
    from minivllm_amd.config import Config
    from minivllm_amd.engine.inference_executor import kv_planes, state_modules
    from minivllm_amd.glue import create_model

    cfg = CONFIGS["odd"]
    c = Config(write_checkpoint(tmp_path / "m", cfg, P.random_model(cfg, 0, RANKS["odd"])), max_model_len=640)
    h = c.hf_config
    assert (h.vocab_size, h.hidden_size, h.norm_eps, h.pair_buckets, h.pair_muls) == (301, 200, 3e-5, 97, (13, 7))
    assert h.num_hidden_layers == 4 and h.max_position_embeddings == 640 and h.recurrent_state
    d, m = h.layers[0].mixer, h.layers[0].mlp
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.taps, d.channel_decay) == (6, 3, 24, 40, 3, False)
    assert (m.experts, m.identity, m.top, m.groups, m.keep, m.scale, m.ff, m.shared_ff) == (7, 2, 3, 3, 2, 1.5, 40, 72)
    p = h.layers[1].mixer
    assert (p.left.window, p.left.keep_first, p.left.softcap, p.left.scale) == (37, 3, 5.0, 0.3) and (p.left_scale, p.right_scale) == (0.6, 1.2)
    assert p.right.channel_decay and (p.right.decay_rank, p.right.gate_rank) == RANKS["odd"]     # from the checkpoint's tensors
    assert h.layers[1].mlp.ff == 120 and h.layers[2].mlp is None and h.layers[3].mixer.left.softcap == 0.0
    assert h.layers[3].mlp.groups == h.layers[3].mlp.keep == 1
    assert h.weight_shapes() == P.tensor_shapes(cfg, RANKS["odd"])
    model = create_model(h)
    assert type(model).__name__ == "PununexForCausalLM" and kv_planes(model) == [(6, 3, 64, 0), (4, 1, 128, 0)]
    shapes = [m.state_shapes(torch.bfloat16) for m in state_modules(model)]
    assert shapes[0] == {"prev_tokens": ((), torch.int32)}
    assert [s["state"][0] for s in shapes[1:]] == [(6, 32, 48), (3, 64, 32), (2, 64, 16), (4, 32, 64)]
    assert shapes[1]["conv_state"] == ((2, 320 + 128 + 96), torch.bfloat16)
    plain = create_model(Config(write_checkpoint(tmp_path / "p", CONFIGS["plain"], P.random_model(CONFIGS["plain"], 0, RANKS["plain"]))).hf_config)
    assert plain.bigram is None and plain.l1.mix.attn.mask.window == 0


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][0].update(type="other"), "layer type"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "feed-forward"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "do not divide"),
    (lambda c: c["layers"][0]["mixer"].pop("conv"), "missing 'conv'"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=7), "cannot give 7 choices"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=2), "9 outputs in 2 groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=4), "cannot give"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(identity=-1), "non-negative"),
    (lambda c: c["layers"][0]["mlp"].pop("expert"), "missing 'expert'"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=4), "do not divide"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(scale=-1.0), "scale must be positive"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0), "positive integer"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(keep_first=-2), "non-negative"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "missing 'right'"),
    (lambda c: c["layers"][1]["mlp"].pop("ff"), "missing 'ff'"),
    (lambda c: c["embedding"]["bigram"].pop("mul_prev"), "missing 'mul_prev'"),
    (lambda c: c.update(layers=[]), "non-empty"),
])
def test_config_errors_name_the_field(tmp_path, change, text):
    from minivllm_amd.native_configs import load_native_config

    cfg = copy.deepcopy(CONFIGS["odd"])
    change(cfg)
    with pytest.raises(ValueError, match=text):
        load_native_config(write_checkpoint(tmp_path / "m", cfg, {}))


def test_ranks_without_a_checkpoint_come_from_the_configuration():
    from minivllm_amd.native_configs import PununexConfig

    cfg = config(64, 32, [layer(parallel(attention(1, 1, 8, 8), delta(1, 1, 8, 8)))])
    with pytest.raises(ValueError, match="ranks"):
        PununexConfig(cfg).weight_shapes()
    cfg = copy.deepcopy(cfg)
    cfg["layers"][0]["mixer"]["right"]["rank"] = 5
    assert PununexConfig(cfg).weight_shapes()["l0.mix.right.a2"] == (8, 5)


# ---- weights -----------------------------------------------------------------------------------------------------------
def _built(path, cfg, weights):
    from minivllm_amd.glue import create_model
    from minivllm_amd.native_configs import load_native_config
    from minivllm_amd.utils.loader import load_model

    d = write_checkpoint(path / "m", cfg, weights)
    c = load_native_config(d)
    c.max_position_embeddings = 128
    m = create_model(c)
    load_model(m, d)
    return m


def test_weights_land_in_the_merged_matrices_with_zero_padding(tmp_path):
    cfg = CONFIGS["odd"]
    w = P.random_model(cfg, 3, RANKS["odd"])
    m = _built(tmp_path, cfg, w)
    f = {k: v.float() for k, v in w.items()}
    d = m.l0.mix                                   # 6 heads of 40 -> 48, 3 key heads of 24 -> 32, width 200 at 256
    assert d.in_proj.offsets == {"v": 0, "k": 320, "q": 448, "b": 576, "a": 640, "g": 704} and d.in_proj.weight.shape == (1024, 256)
    v = d.in_proj.weight[:288, :200].view(6, 48, 200)
    assert torch.equal(v[:, :40], f["l0.mix.v"].view(6, 40, 200)) and v[:, 40:].abs().sum() == 0
    assert torch.equal(d.in_proj.weight[320:416, :200].view(3, 32, 200)[:, :24], f["l0.mix.k"].view(3, 24, 200))
    assert torch.equal(d.in_proj.weight[576:582, :200], f["l0.mix.b"]) and torch.equal(d.in_proj.weight[640:646, :200], f["l0.mix.a"])
    r = d.rule
    assert r.shape.channels == 448 + 96 and r.conv.shape == (3, 544) and r.shape.q_scale == 24 ** -0.5
    assert torch.equal(r.conv[:, 448:544].view(3, 3, 32)[:, :, :24], f["l0.mix.q.conv"].T.reshape(3, 3, 24)) and r.conv[:, 472:480].abs().sum() == 0
    assert torch.equal(r.norm[:40], f["l0.mix.norm"]) and torch.equal(r.A_log, f["l0.mix.A_log"]) and torch.equal(r.dt_bias, f["l0.mix.dt_bias"])
    e = m.l0.mlp                                   # 7 experts of 40 -> 64
    assert e.gate_up.shape == (7, 2, 64, 256) and torch.equal(e.gate_up[4, 0, :40, :200], f["l0.mlp.e4.gate"])
    assert torch.equal(e.gate_up[6, 1, :40, :200], f["l0.mlp.e6.up"]) and torch.equal(e.down[5, :200, :40], f["l0.mlp.e5.down"])
    assert e.gate_up[:, :, 40:].abs().sum() == 0 and e.down[:, :, 40:].abs().sum() == 0
    assert torch.equal(e.router[:, :200], f["l0.mlp.router"]) and torch.equal(e.correction, f["l0.mlp.correction"])
    assert torch.equal(e.shared_gate_up.weight[128:200, :200], f["l0.mlp.shared.up"]) and torch.equal(e.shared_down.weight[:200, :72], f["l0.mlp.shared.down"])
    p = m.l1.mix                                   # attention heads of 40 | 24 -> 64; rule: 3 heads, keys 40 -> 64, values 20 -> 32
    at = p.in_proj.offsets
    assert torch.equal(p.in_proj.weight[:384, :200].view(6, 64, 200)[:, :40], f["l1.mix.left.q"].view(6, 40, 200))
    assert torch.equal(p.in_proj.weight[at["left.v"]:at["left.v"] + 192, :200].view(3, 64, 200)[:, :24], f["l1.mix.left.v"].view(3, 24, 200))
    assert torch.equal(p.in_proj.weight[at["right.g1"]:at["right.g1"] + 40, :200], f["l1.mix.right.g1"])
    assert torch.equal(p.q_norm[:40], f["l1.mix.left.q.norm"]) and torch.equal(p.sink, f["l1.mix.left.sink"]) and p.k_norm[40:].abs().sum() == 0
    lift = p.rule.lift                             # [decay rank 24 -> 64 | gate rank 40 -> 64] -> [3 x 64 | 3 x 32]
    assert lift.weight.shape == (192 + 128, 128) and lift.offsets == {"a2": 0, "g2": 192}
    a2, g2 = lift.weight[:192].view(3, 64, 128), lift.weight[192:288].view(3, 32, 128)
    assert torch.equal(a2[:, :40, :24], f["l1.mix.right.a2"].view(3, 40, 24)) and torch.equal(g2[:, :20, 64:104], f["l1.mix.right.g2"].view(3, 20, 40))
    assert lift.weight.abs().sum() == a2[:, :40, :24].abs().sum() + g2[:, :20, 64:104].abs().sum()
    assert torch.equal(p.rule.dt_bias.view(3, 64)[:, :40], f["l1.mix.right.dt_bias"].view(3, 40))
    assert torch.equal(p.o.weight[:200, :384].view(200, 6, 64)[:, :, :24], f["l1.mix.left.o"].view(200, 6, 24))
    assert torch.equal(p.o.weight[:200, 384:480].view(200, 3, 32)[:, :, :20], f["l1.mix.right.o"].view(200, 3, 20))
    assert torch.equal(m.bigram.weight[:, :200], f["bigram"]) and torch.equal(m.l1.norm2_b[:200], f["l1.norm2.b"])
    assert torch.equal(m.l0.ls1[:200], f["l0.ls1"]) and m.l2.mlp is None and torch.equal(m.final_norm_b[:200], f["final.norm.b"])
    assert torch.equal(m.head.weight[:, :200], f["head"]) and torch.equal(m.l1.mlp.gate_up.weight[128:248, :200], f["l1.mlp.up"])


def test_a_missing_or_misshapen_tensor_is_an_error(tmp_path):
    cfg = CONFIGS["states"]
    w = P.random_model(cfg, 0, RANKS["states"])
    with pytest.raises(ValueError, match="l0.mlp.e3.up"):
        _built(tmp_path / "a", cfg, {k: v for k, v in w.items() if k != "l0.mlp.e3.up"})
    with pytest.raises(ValueError, match="l0.mix.k.conv"):
        _built(tmp_path / "b", cfg, dict(w, **{"l0.mix.k.conv": w["l0.mix.k.conv"][:-1].contiguous()}))


def test_head_sizes_above_the_kernels_and_several_ranks_are_refused(tmp_path):
    from minivllm_amd import parallel_state as ps
    from minivllm_amd.glue import create_model
    from minivllm_amd.native_configs import PununexConfig

    big = config(64, 32, [layer(parallel(attention(1, 1, 300, 8), dict(delta(1, 1, 8, 8), rank=4)))])
    with pytest.raises(ValueError, match="above 256"):
        create_model(PununexConfig(big))
    ps.init_tensor_parallel(0, 2)
    with pytest.raises(ValueError, match="one GPU"):
        create_model(PununexConfig(config(64, 32, [layer(delta(2, 2, 8, 8), dense(64))])))


def test_tiles_follow_the_pairs_per_expert():
    from minivllm_amd.layers import ExpertMLP

    e = ExpertMLP(64, 16, 0, 4, 1, 1, 1.0, 64)
    assert e.tile_rows(1) == 16                                          # (fp32: the only form)
    e = e.to(torch.bfloat16)
    rows = [e.tile_rows(t) for t in (1, 16, 256, 16384)]
    assert rows == sorted(rows) and rows[0] == 16 and rows[-1] == 256


def test_header_shapes_of_a_checkpoint(tmp_path):
    from minivllm_amd.native_configs import checkpoint_shapes

    d = write_checkpoint(tmp_path / "m", {}, {"a.b": torch.zeros(3, 5), "c": torch.zeros(2, dtype=torch.int32)})
    assert checkpoint_shapes(d) == {"a.b": (3, 5), "c": (2,)} and checkpoint_shapes(tmp_path) == {}
