"""Semezen without a GPU: configuration, weight placement (order, padding, biases, experts), rotary tables, state shapes, and the
plain implementation's own consistency."""
import copy
import math

import pytest
import torch

from oracle import semezen as S
from semezen_configs import CONFIGS, attention, config, dense, layer, mingru, moe, sharp_weights, write_checkpoint


@pytest.fixture(autouse=True)
def _single_rank():
    from minivllm_amd import parallel_state

    parallel_state.reset_tensor_parallel()
    yield
    parallel_state.reset_tensor_parallel()


def _rand(*shape, seed=0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64)


# ---- the plain implementation ------------------------------------------------------------------------------------------
def test_long_wavelengths_are_stretched_and_short_ones_kept():
    m = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 100}
    f, g = (S.scaled_frequencies(50.0, 16, x) for x in (None, m))
    turns = 100 * f / (2 * math.pi)
    assert (turns > 4).any() and (turns < 1).any() and ((turns > 1) & (turns < 4)).any()
    for a, b, t in zip(f.tolist(), g.tolist(), turns.tolist()):
        s = min(max((t - 1) / 3, 0.0), 1.0)
        assert b == pytest.approx((1 - s) * a / 4 + s * a)
    assert g[0] == f[0] and g[-1] == pytest.approx(f[-1] / 4)


def test_rotation_by_hand():
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 5.0]]]).double()
    y = S.rotate_halves(x, torch.tensor([2]), torch.tensor([0.25, 1.0]).double())[0, 0]
    c, s = math.cos(0.5), math.sin(0.5)
    assert y[[0, 2]].tolist() == pytest.approx([c - 3 * s, 3 * c + s]) and y[4] == 5
    assert y[[1, 3]].tolist() == pytest.approx([2 * math.cos(2) - 4 * math.sin(2), 4 * math.cos(2) + 2 * math.sin(2)])


def test_running_mean_by_hand():
    z, u = torch.tensor([[0.25], [1.0], [0.0]]).double(), torch.tensor([[2.0], [-1.0], [9.0]]).double()
    sig = 1 / (1 + math.e)
    assert S.gru_scan(z, u).flatten().tolist() == pytest.approx([0.625, sig, sig])
    assert S.gru_scan(z, u, torch.tensor([4.0]).double())[0].item() == pytest.approx(3.625)
    assert S.gru_scan(torch.ones(1, 1).double(), torch.zeros(1, 1).double()).item() == 0.5          # both halves meet


def test_token_shift_and_streams_by_hand():
    h = torch.tensor([[1.0, 2.0], [3.0, 5.0]]).double()
    assert S.token_shift(h, torch.tensor([0.5, -1.0]).double()).tolist() == [[0.5, 4.0], [2.0, 8.0]]
    x, mix = torch.tensor([[[1.0], [10.0]]]).double(), torch.tensor([[2.0, 3.0], [5.0, 7.0]]).double()
    new = S.write_streams(x, mix, torch.tensor([1.0, -1.0]).double(), torch.tensor([[100.0]]).double())
    assert new.flatten().tolist() == [2 + 50 + 100, 3 + 70 - 100]        # [from, to]
    assert S.read_streams(x, torch.tensor([0.5, 2.0]).double()).item() == 20.5


def test_an_expert_clamps_and_its_input_is_weighed():
    w = {"e0.gate": torch.tensor([[3.0]]).double(), "e0.up": torch.tensor([[-4.0]]).double(), "e0.down": torch.tensor([[2.0]]).double(),
         "router": torch.tensor([[1.0]]).double()}
    f = lambda g, u: 2 * g / (1 + math.exp(-1.702 * g)) * (u + 1)
    assert S.expert(torch.tensor([[0.5]]).double(), w, "e0.", 1.75).item() == pytest.approx(f(1.5, -1.75))
    assert S.expert(torch.tensor([[-2.0]]).double(), w, "e0.", 1.75).item() == pytest.approx(f(-6.0, 1.75))
    m = {"router": {"top": 1}, "expert": {"limit": 100.0}}
    c = 1 / (1 + math.exp(-0.5))
    assert S.moe(torch.tensor([[0.5]]).double(), m, w, "").item() == pytest.approx(f(1.5 * c, -2 * c))


def test_the_exact_gelu():
    z = torch.tensor([-3.0, -0.5, 0.0, 1.0, 4.0]).double()
    assert torch.allclose(S.gelu(z), torch.nn.functional.gelu(z))


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_a_longer_sequence_does_not_change_earlier_logits(name):
    cfg = CONFIGS[name]
    toks, w = torch.arange(75) % cfg["vocab"], sharp_weights(name)
    a, b = S.forward(cfg, w, toks), S.forward(cfg, w, toks[:51])
    assert torch.allclose(a[:51], b, atol=1e-9)


# ---- configuration -----------------------------------------------------------------------------------------------------
def test_config_is_read_and_served_by_the_registry(tmp_path):
    from minivllm_amd.config import Config
    from minivllm_amd.engine.inference_executor import kv_planes, state_modules
    from minivllm_amd.glue import create_model

    cfg = CONFIGS["odd"]
    c = Config(write_checkpoint(tmp_path / "m", cfg, S.random_model(cfg)), max_model_len=640)
    h = c.hf_config
    assert (h.vocab_size, h.hidden_size, h.norm_eps, h.streams) == (301, 200, 3e-4, 5)
    assert h.num_hidden_layers == 4 and h.max_position_embeddings == 640 and h.recurrent_state
    assert h.layers[0].mixer.width == 72 and h.layers[2].mlp is None and h.layers[1].mlp.ff == 120
    m = h.layers[0].mlp
    assert (m.experts, m.top, m.ff, m.limit) == (7, 3, 40, 0.7)
    a = h.layers[1].mixer
    assert (a.heads, a.kv_heads, a.dim, a.window, a.rot_dims, a.rot_base, a.scale) == (6, 3, 40, 37, 22, 500.0, 3.0 * 40 ** -0.5)
    assert (a.scaling.factor, a.scaling.low, a.scaling.high, a.scaling.original) == (8.0, 1.0, 4.0, 60)
    assert h.weight_shapes() == S.tensor_shapes(cfg)
    model = create_model(h)
    assert type(model).__name__ == "SemezenForCausalLM" and kv_planes(model) == [(6, 3, 64, 0), (4, 1, 64, 0)]
    assert model.l1.mix.attn.mask.window == 37 and model.l1.mix.attn.scale == a.scale
    e = model.l0.mlp
    assert (e.act.kind, e.act.limit, e.act.alpha) == (2, pytest.approx(0.7), pytest.approx(1.702))
    assert e.sigmoid and e.raw_weights and e.weigh_inputs and e.correction is None
    shapes = [m.state_shapes(torch.bfloat16) for m in state_modules(model)]
    assert sorted(str(s) for s in shapes) == sorted(str(s) for s in [{"prev": ((256,), torch.float32)}] * 4 + [
        {"state": ((128,), torch.float32)}, {"state": ((320,), torch.float32)}])
    plain = create_model(Config(write_checkpoint(tmp_path / "p", CONFIGS["plain"], S.random_model(CONFIGS["plain"]))).hf_config)
    assert plain.l0.mix.attn.mask.window == 0 and plain.l0.mlp is None and not hasattr(plain.l0, "hc2")
    assert plain.config.layers[0].mixer.scaling is None


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][0].update(type="other"), "layer type"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "feed-forward"),
    (lambda c: c["layers"][0]["mixer"].pop("width"), "missing 'width'"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=8), "cannot give 8 choices"),
    (lambda c: c["layers"][0]["mlp"].pop("expert"), "missing 'expert'"),
    (lambda c: c["layers"][0]["mlp"]["expert"].update(limit=0.0), "limit must be positive"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=4), "do not divide"),
    (lambda c: c["layers"][1]["mixer"].update(vdim=24), "the values are the keys"),
    (lambda c: c["layers"][1]["mixer"].update(scale=-1.0), "must be positive"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=23), "even"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=42), "at most dim"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("low"), "missing 'low'"),
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(high=0.5), "high at least low"),
    (lambda c: c["layers"][1]["mixer"]["mask"].update(size=0), "positive integer"),
    (lambda c: c["layers"][1]["mlp"].pop("ff"), "missing 'ff'"),
    (lambda c: c.pop("streams"), "missing 'streams'"),
    (lambda c: c.update(streams=9), "at most 8"),
    (lambda c: c.update(layers=[]), "non-empty"),
])
def test_config_errors_name_the_field(tmp_path, change, text):
    from minivllm_amd.native_configs import load_native_config

    cfg = copy.deepcopy(CONFIGS["odd"])
    change(cfg)
    with pytest.raises(ValueError, match=text):
        load_native_config(write_checkpoint(tmp_path / "m", cfg, {}))


# ---- rotation ----------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("scaling", [None, (8.0, 1.0, 4.0, 60), (2.0, 2.0, 2.0, 100), (3.0, 0.01, 0.02, 50), (3.0, 900.0, 990.0, 50)], ids=str)
@pytest.mark.parametrize("dim, rot, base", [(40, 22, 500.0), (24, 24, 100.0), (8, 2, 1e4), (64, 32, 5e5)])
def test_pairs_side_by_side_give_the_same_scores_as_halves(dim, rot, base, scaling):
    """The stored order and the table against the plain rotation of halves."""
    from minivllm_amd.layers import get_rope, halves_as_pairs

    names = ("factor", "low", "high", "original")
    plain = dict(zip(names, scaling)) if scaling else None
    rope = get_rope(64, rot, 50, base, dict(plain, type="wavelength") if plain else None, interleaved=True)
    cos, sin = rope._cos32.double(), rope._sin32.double()
    x, pos, order = _rand(50, 1, dim, seed=1), torch.arange(50), torch.tensor(halves_as_pairs(dim, rot))
    assert sorted(order.tolist()) == list(range(dim))
    want = S.rotate_halves(x, pos, S.scaled_frequencies(base, rot, plain))[:, 0]
    y = torch.empty(50, dim, dtype=torch.float64)
    y[:, order] = x[:, 0]
    u, v = y[:, 0:rot:2].clone(), y[:, 1:rot:2].clone()
    y[:, 0:rot:2], y[:, 1:rot:2] = u * cos - v * sin, v * cos + u * sin
    assert torch.allclose(y[:, order], want, atol=1e-5)


def test_other_scalings_are_refused_for_pairs():
    from minivllm_amd.layers import get_rope

    with pytest.raises(ValueError, match="wavelength"):
        get_rope(64, 32, 50, 1e4, {"type": "linear", "factor": 2.0}, interleaved=True)


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


def test_weights_land_in_the_merged_matrices(tmp_path):
    from minivllm_amd.layers import halves_as_pairs

    cfg = CONFIGS["odd"]
    w = S.random_model(cfg, 3)
    m = _built(tmp_path, cfg, w)
    f = {k: v.float() for k, v in w.items()}
    g = m.l0.mix                                   # 72 -> 128 channels, width 200 at 256
    assert g.in_proj.offsets == {"z": 0, "x": 128, "g": 256} and g.in_proj.weight.shape == (384, 256)
    assert torch.equal(g.in_proj.weight[128:200, :200], f["l0.mix.x"]) and torch.equal(g.in_proj.weight[256:328, :200], f["l0.mix.g"])
    assert torch.equal(g.in_proj.bias[:72], f["l0.mix.z.b"]) and torch.equal(g.in_proj.bias[128:200], f["l0.mix.x.b"])
    assert g.in_proj.bias[256:].abs().sum() == 0 and g.in_proj.bias[72:128].abs().sum() == 0
    assert torch.equal(g.o.weight[:200, :72], f["l0.mix.o"]) and g.o.weight[:, 72:].abs().sum() == 0
    a, order = m.l1.mix, torch.tensor(halves_as_pairs(40, 22))     # 6 | 3 heads of 40 -> 64, pairs side by side
    assert a.in_proj.offsets == {"q": 0, "k": 384, "g": 576}
    q = a.in_proj.weight[:384, :200].view(6, 64, 200)
    assert torch.equal(q[:, order], f["l1.mix.q"].view(6, 40, 200)) and q[:, 40:].abs().sum() == 0
    assert torch.equal(a.in_proj.weight[576:960, :200].view(6, 64, 200)[:, order], f["l1.mix.g"].view(6, 40, 200))
    assert torch.equal(a.in_proj.bias[384:576].view(3, 64)[:, order], f["l1.mix.k.b"].view(3, 40)) and a.in_proj.bias[576:].abs().sum() == 0
    assert torch.equal(a.o.weight[:200].view(200, 6, 64)[:, :, order], f["l1.mix.o"].view(200, 6, 40))
    e = m.l0.mlp
    assert torch.equal(e.gate_up[4, 0, :40, :200], f["l0.mlp.e4.gate"]) and torch.equal(e.gate_up[6, 1, :40, :200], f["l0.mlp.e6.up"])
    assert torch.equal(e.down[5, :200, :40], f["l0.mlp.e5.down"]) and torch.equal(e.router[:, :200], f["l0.mlp.router"])
    assert torch.equal(m.l1.mlp.up.weight[:120, :200], f["l1.mlp.up"]) and torch.equal(m.l1.mlp.down.weight[:200, :120], f["l1.mlp.down"])
    for i in range(4):
        la = getattr(m, f"l{i}")
        assert torch.equal(la.shift.share[:200], f[f"l{i}.shift"]) and torch.equal(la.norm1[:200], f[f"l{i}.norm1"])
        for c in ("hc1", "hc2") if i != 2 else ("hc1",):
            h = getattr(la, c)
            assert torch.equal(h.read, f[f"l{i}.{c}.in"]) and torch.equal(h.write, f[f"l{i}.{c}.out"]) and torch.equal(h.mix, f[f"l{i}.{c}.mix"])
    assert torch.equal(m.embed[:, :200], f["embed"]) and torch.equal(m.final_norm[:200], f["final.norm"]) and torch.equal(m.head.weight[:, :200], f["head"])


def test_a_missing_or_misshapen_tensor_is_an_error(tmp_path):
    cfg = CONFIGS["states"]
    w = S.random_model(cfg)
    with pytest.raises(ValueError, match="l0.mlp.e3.up"):
        _built(tmp_path / "a", cfg, {k: v for k, v in w.items() if k != "l0.mlp.e3.up"})
    with pytest.raises(ValueError, match="l1.mix.z.b"):
        _built(tmp_path / "b", cfg, dict(w, **{"l1.mix.z.b": w["l1.mix.z.b"][:-1].contiguous()}))
    with pytest.raises(ValueError, match="l2.shift"):
        _built(tmp_path / "c", cfg, {k: v for k, v in w.items() if k != "l2.shift"})


def test_sizes_beyond_the_kernels_and_several_ranks_are_refused():
    from minivllm_amd import parallel_state as ps
    from minivllm_amd.glue import create_model
    from minivllm_amd.layers import ExpertMLP, Segment, SegmentedLinear
    from minivllm_amd.native_configs import SemezenConfig

    with pytest.raises(ValueError, match="above 256"):
        create_model(SemezenConfig(config(64, 32, 2, [layer(attention(1, 1, 300))])))
    with pytest.raises(ValueError, match="identity"):
        ExpertMLP(64, 4, 1, 2, 1, 1, 1.0, 64, weigh_inputs=True)
    with pytest.raises(ValueError, match="bias"):
        SegmentedLinear(64, [Segment("o", 64)], split="in", bias=True)
    ps.init_tensor_parallel(0, 2)
    with pytest.raises(ValueError, match="one GPU"):
        create_model(SemezenConfig(config(64, 32, 2, [layer(mingru(64), dense(64))])))


def test_random_weights_of_every_name(tmp_path):
    from minivllm_amd.glue import create_model
    from minivllm_amd.native_configs import SemezenConfig

    c = SemezenConfig(config(64, 32, 3, [layer(mingru(64), moe(3, 1, 64)), layer(attention(2, 1, 32, 9), dense(64))]))
    m = create_model(c)
    w = m.dummy_weights(torch.Generator().manual_seed(0))
    assert set(w) == set(c.weight_shapes())
    m.load_weights(w)
    assert torch.equal(m.l0.hc1.mix, torch.eye(3)) and m.l0.mix.in_proj.bias[:64].mean() < -1.5
