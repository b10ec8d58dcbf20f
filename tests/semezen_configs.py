"""Small Semezen configurations for the tests, and checkpoints of them with random weights."""
from mofarax_configs import write_checkpoint  # noqa: F401  (the same checkpoint layout)
from oracle import semezen as S


def attention(heads, kv_heads, dim, window=None, rot=None, base=10000.0, scaling=None, sharp=3.0):
    """``sharp``: queries and keys have a length of sqrt(dim), so scores are about ``sharp`` times a normal number; ``scaling``:
    (factor, low, high, original)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": sharp * dim ** -0.5,
         "rot": {"base": base, "dims": rot or dim}}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    if window:
        m["mask"] = {"size": window}
    return m


def mingru(width):
    return {"width": width}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit=1.5):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}


def layer(mixer, mlp=None):
    return {"type": "mingru" if "width" in mixer else "attention", "mixer": mixer, "mlp": mlp}


def config(width, vocab, streams, layers, eps=1e-5):
    return {"architecture": "Semezen", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # odd sizes everywhere, layers of unlike shape, partial rotation, every part of a frequency scaling, several choices of an expert
    "odd": config(200, 301, 5, [layer(mingru(72), moe(7, 3, 40, 0.7)),
                                layer(attention(6, 3, 40, 37, 22, 500.0, (8.0, 1.0, 4.0, 60)), dense(120)),
                                layer(mingru(301)),
                                layer(attention(4, 1, 24, 90, 24, 100.0, (2.5, 0.5, 9.0, 200)), moe(5, 1, 72))], eps=3e-4),
    # heads at the kernels' own sizes (the matrix-core decode kernel); as many choices as experts
    "large_heads": config(256, 128, 2, [layer(attention(8, 1, 128, 100, 32), moe(4, 4, 64, 3.0)), layer(mingru(512), dense(192)),
                                        layer(attention(4, 4, 64, 33, 64), dense(64))]),
    # one of everything: a stream, a window of one token, a head, an expert, two rotated dims
    "ones": config(64, 64, 1, [layer(attention(1, 1, 8, 1, 2), moe(1, 1, 64)), layer(mingru(1), moe(2, 1, 64)),
                               layer(attention(2, 1, 64, 2, 64), dense(64))]),
    # no window, no scaling, no feed-forward in places; heads wider than 128; attention only
    "plain": config(96, 104, 4, [layer(attention(2, 1, 160, None, 100)), layer(attention(4, 2, 32), dense(96))], eps=1e-6),
    # recurrent layers only: no cache plane at all
    "states": config(96, 104, 8, [layer(mingru(128), moe(6, 2, 32, 2.0)), layer(mingru(640), dense(64)), layer(mingru(64))]),
}


def sharp_weights(name, seed=0, calm=False):
    """Random weights.  ``calm``: experts weigh little, for 16-bit runs of whole models, where a close call of a router may go either
    way and a state carries it on."""
    cfg, w = CONFIGS[name], S.random_model(CONFIGS[name], seed)
    for i, la in enumerate(cfg["layers"]):
        if calm and la["mlp"] and la["mlp"]["kind"] == "moe":
            w[f"l{i}.hc2.out"] = (w[f"l{i}.hc2.out"].float() * 0.05).bfloat16()
    return w
