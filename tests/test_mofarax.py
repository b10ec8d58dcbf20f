"""Mofarax without a GPU: configuration, weight placement (padding, tensor-parallel shards), rotation tables, the block
pool's portion-wise growth, and the plain implementation's own consistency."""
import copy
import math

import pytest
import torch

from mofarax_configs import CONFIGS, config, layer, sharp_weights, write_checkpoint
from oracle import mofarax as M


@pytest.fixture(autouse=True)
def _single_rank():
    """The models are built for one rank, whatever earlier tests of this process left behind."""
    from minivllm_amd import parallel_state

    parallel_state.reset_tensor_parallel()
    yield
    parallel_state.reset_tensor_parallel()


# ---- the plain implementation ------------------------------------------------------------------------------------------
def test_rotation_is_relative_and_leaves_the_tail():
    g = torch.Generator().manual_seed(0)
    x, y = (torch.randn(1, 1, 12, generator=g, dtype=torch.float64) for _ in range(2))

    def dot(p, q):
        a = M.rotate_interleaved(x, torch.tensor([p]), 300.0, 8)
        b = M.rotate_interleaved(y, torch.tensor([q]), 300.0, 8)
        return (a[..., :8] * b[..., :8]).sum().item()
    assert dot(5, 3) == pytest.approx(dot(105, 103), rel=1e-9) and abs(dot(5, 3) - dot(5, 4)) > 1e-3
    assert torch.equal(M.rotate_interleaved(x, torch.tensor([9]), 300.0, 8)[..., 8:], x[..., 8:])
    # the first pair by hand: (u cos a - v sin a, v cos a + u sin a), a = position
    u, v = x[0, 0, 0].item(), x[0, 0, 1].item()
    r = M.rotate_interleaved(x, torch.tensor([2]), 300.0, 8)[0, 0]
    assert r[0].item() == pytest.approx(u * math.cos(2) - v * math.sin(2)) and r[1].item() == pytest.approx(v * math.cos(2) + u * math.sin(2))


def test_chunk_mask_counts_from_the_start_of_the_sequence():
    m = M.chunk_mask(10, 4)
    assert m[3].nonzero().flatten().tolist() == [0, 1, 2, 3] and m[4].nonzero().flatten().tolist() == [4]
    assert m[9].nonzero().flatten().tolist() == [8, 9]
    assert M.chunk_mask(5, None)[4].all()


def test_layer_schedule_of_a_loop():
    assert M.layer_schedule(4, {"start": 1, "stop": 3, "times": 2}) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert M.layer_schedule(2, None) == [(0, None), (1, None)]


def test_a_longer_sequence_does_not_change_earlier_logits():
    cfg, toks = CONFIGS["odd"], torch.arange(75) % 301
    w = sharp_weights(cfg)
    a, b = M.forward(cfg, w, toks, torch.float64), M.forward(cfg, w, toks[:51], torch.float64)
    assert torch.allclose(a[:51], b, atol=1e-10)


# ---- configuration -----------------------------------------------------------------------------------------------------
def test_config_is_read_and_served_by_the_registry(tmp_path):
    from minivllm_amd.config import Config
    from minivllm_amd.glue import create_model

    cfg = CONFIGS["odd"]
    c = Config(write_checkpoint(tmp_path / "m", cfg, M.random_model(cfg)), max_model_len=640)
    h = c.hf_config
    assert (h.vocab_size, h.hidden_size, h.side_dim, h.loop) == (301, 200, 20, (1, 3, 2))
    assert h.layer_runs() == [(0, 0, False), (1, 0, True), (2, 0, False), (1, 1, True), (2, 1, False), (3, 0, False)]
    assert h.num_hidden_layers == 6 and h.max_position_embeddings == 640
    a = h.layers[0].attention
    assert (a.heads, a.kv_heads, a.dim, a.rot_dims, a.rot_base, a.chunk, a.scale) == (6, 2, 48, 32, 500.0, 50, 0.2)
    assert h.layers[1].ff == 0 and h.weight_shapes() == M.tensor_shapes(cfg)
    m = create_model(h)
    assert type(m).__name__ == "MofaraxForCausalLM"
    # a K/V plane pair per pass of the looped layers, one for the others
    from minivllm_amd.engine.inference_executor import kv_planes
    assert [p[1:] for p in kv_planes(m)] == [(2, 64, 50), (4, 64, 33), (4, 64, 33), (1, 64, 100), (1, 64, 100), (3, 64, 70)]


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][0].update(type="other"), "layer type"),
    (lambda c: c["layers"][0]["mlp"].update(kind="sparse"), "feed-forward"),
    (lambda c: c["layers"][0]["mixer"].update(vdim=16), "vdim"),
    (lambda c: c["layers"][0]["mixer"].update(heads=5), "do not divide"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=50), "at most dim"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "positive integer"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "missing 'scale'"),
    (lambda c: c["loop"].update(stop=9), "loop"),
    (lambda c: c.update(architecture="Unheard"), "unsupported architecture"),
])
def test_config_errors_name_the_field(tmp_path, change, text):
    from minivllm_amd.native_configs import load_native_config

    cfg = copy.deepcopy(CONFIGS["odd"])
    change(cfg)
    with pytest.raises(ValueError, match=text):
        load_native_config(write_checkpoint(tmp_path / "m", cfg, {}))


def test_other_model_directories_are_left_to_their_own_loader(tmp_path):
    from minivllm_amd.native_configs import load_native_config

    (tmp_path / "config.json").write_text('{"model_type": "qwen3"}')
    assert load_native_config(str(tmp_path)) is None and load_native_config(str(tmp_path / "none")) is None


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
    w = M.random_model(cfg, 3)
    m = _built(tmp_path, cfg, w)
    f = {k: v.float() for k, v in w.items()}
    lin, ffn = m.l0.qk, m.l0.gate_up                                   # q: 6 heads of 48 stored at 64; width 200 at 256
    assert lin.weight.shape == (6 * 64 + 2 * 64, 256) and lin.offsets == {"q": 0, "k": 384}
    assert ffn.weight.shape == (128 + 128, 256) and ffn.offsets == {"gate": 0, "up": 128}
    q = lin.weight[:384].view(6, 64, 256)
    assert torch.equal(q[:, :48, :200], f["l0.mix.q"].view(6, 48, 200)) and q[:, 48:].abs().sum() == 0
    assert torch.equal(ffn.weight[:120, :200], f["l0.mlp.gate"]) and ffn.weight[120:128].abs().sum() == 0
    assert torch.equal(ffn.weight[128:248, :200], f["l0.mlp.up"])
    assert lin.weight[:, 200:].abs().sum() == 0
    o = m.l0.proj_out.weight[:200, :384].view(200, 6, 64)
    assert torch.equal(o[:, :, :48], f["l0.mix.o"].view(200, 6, 48)) and o[:, :, 48:].abs().sum() == 0
    assert torch.equal(m.l0.proj_out.weight[:200, 384:504], f["l0.mlp.down"])
    assert m.l1.proj_out.weight.shape == (256, 256) and m.l1.ff == 0   # no feed-forward: 4 heads of 32 stored at 64
    assert torch.equal(m.l2.side.gate.weight[:20, :200], f["l2.side.gate"]) and torch.equal(m.l2.side.norm[:200], f["l2.side.norm"])
    assert torch.equal(m.head.weight[:, :200], f["head"]) and m.head.weight[:, 200:].abs().sum() == 0
    assert torch.equal(m.loop_step[:, :200], f["loop.step"]) and torch.equal(m.side_embed, f["side.embed"])


def test_a_missing_or_foreign_tensor_is_an_error(tmp_path):
    cfg = CONFIGS["tiny_chunk"]
    w = M.random_model(cfg)
    short = {k: v for k, v in w.items() if k != "l1.mix.k"}
    with pytest.raises(ValueError, match="l1.mix.k"):
        _built(tmp_path / "a", cfg, short)
    bad = dict(w, **{"l0.mix.o": w["l0.mix.o"][:, :32].contiguous()})
    with pytest.raises(ValueError, match="l0.mix.o"):
        _built(tmp_path / "b", cfg, bad)


def test_tensor_parallel_shards_sum_to_the_whole(tmp_path):
    """Two ranks' shards of a layer, put through plain products, add up to the unsharded layer's."""
    from minivllm_amd import parallel_state as ps

    cfg = config(96, 40, [layer(4, 2, 32, 16, ff=48)], side=16)
    w = M.random_model(cfg, 5)
    h = torch.randn(7, 96)
    h_pad = torch.nn.functional.pad(h, (0, 32))
    f = {k: v.float() for k, v in w.items()}
    total, qs = torch.zeros(7, 96), []
    for rank in range(2):
        ps.init_tensor_parallel(rank, 2)
        try:
            m = _built(tmp_path / str(rank), cfg, w)
        finally:
            ps.reset_tensor_parallel()
        lay = m.l0
        assert (lay.heads, lay.kv_heads) == (2, 1) and m.head.weight.shape[0] == 20
        z, y = h_pad @ lay.qk.weight.T, h_pad @ lay.gate_up.weight.T
        qs.append(z[:, :128].view(7, 2, 64)[:, :, :32])
        up = lay.gate_up.offsets["up"]
        act = M.gelu_tanh(y[:, :up]) * y[:, up:]
        mixed = torch.cat([z[:, :128], act], 1)                        # (the queries stand in for the attention output)
        total += (mixed @ lay.proj_out.weight.T)[:, :96]
    q = h @ f["l0.mix.q"].T
    assert torch.allclose(torch.cat(qs, 1).reshape(7, 128), q, atol=1e-4)
    assert torch.allclose(total, q @ f["l0.mix.o"].T + M.gated_mlp(h, {k: f[f"l0.mlp.{k}"] for k in ("gate", "up", "down")}), atol=1e-3)


def test_interleaved_tables_hold_the_exact_angles():
    from minivllm_amd.layers.rotary_embedding import RotaryEmbedding

    r = RotaryEmbedding(64, 24, 4096, 5000.0, interleaved=True)
    cos, sin = r._tables("cpu")
    assert cos.shape == (4096, 12) and r.interleaved_pairs == 12
    for p, i in ((0, 0), (4095, 0), (4095, 3), (1234, 11)):
        a = p * 5000.0 ** (-2 * i / 24)
        assert cos[p, i].item() == pytest.approx(math.cos(a), abs=1e-7) and sin[p, i].item() == pytest.approx(math.sin(a), abs=1e-7)
    with pytest.raises(ValueError):
        RotaryEmbedding(64, 66, 16, 1e4, interleaved=True)


# ---- sequences and blocks ----------------------------------------------------------------------------------------------
def test_portions_reserve_blocks_and_give_them_back():
    from minivllm_amd.engine.block_manager import BlockManager
    from minivllm_amd.engine.sequence import Sequence

    bm = BlockManager(4, 64)
    a = Sequence([1] * 70, block_size=64)
    bm.reserve(a)
    assert len(a.block_table) == 2 and a.num_cached_tokens == 0
    a.extend([2] * 58)
    bm.reserve(a)
    assert len(a.block_table) == 2 and a.num_cached_tokens == 70 and a.prefill_stop == 128 and a.last_token == 2
    a.extend([3])
    bm.reserve(a)
    assert len(a.block_table) == 3
    b = Sequence([1] * 65, block_size=64)
    with pytest.raises(RuntimeError, match="No free blocks"):
        bm.reserve(b)
    assert b.block_table == [] and bm.get_num_free_blocks() == 1        # all or nothing
    bm.deallocate(a)
    bm.reserve(b)
    assert bm.get_num_free_blocks() == 2
