"""Small Pununex configurations for the tests, and checkpoints of them with random weights."""
from mofarax_configs import write_checkpoint  # noqa: F401  (the same checkpoint layout)
from oracle import pununex as P


def attention(heads, kv_heads, dim, vdim, window=None, keep=0, softcap=None, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale}
    if softcap:
        m["softcap"] = softcap
    if window:
        m["mask"] = {"size": window, "keep_first": keep}
    return m


def delta(heads, kv_heads, dim, vdim, conv=4):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def parallel(left, right, left_scale=0.6, right_scale=1.2):
    return {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, identity=0, groups=None, scale=1.0, shared=None):
    r = {"experts": experts, "top": top, "identity": identity, "scale": scale}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    m = {"kind": "moe", "router": r, "expert": {"ff": ff}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def layer(mixer, mlp=None):
    return {"type": "parallel" if "left" in mixer else "delta", "mixer": mixer, "mlp": mlp}


def config(width, vocab, layers, pairs=None, eps=1e-5):
    e = {"bigram": {"buckets": pairs[0], "mul_prev": pairs[1], "mul_cur": pairs[2]}} if pairs else {}
    return {"architecture": "Pununex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": e, "layers": layers}


CONFIGS = {
    # odd sizes everywhere; several key heads; unlike query / key and value sizes either way round; groups across identity experts
    "odd": config(200, 301, [layer(delta(6, 3, 24, 40, 3), moe(7, 3, 40, identity=2, groups=(3, 2), scale=1.5, shared=72)),
                             layer(parallel(attention(6, 3, 40, 24, 37, 3, 5.0, 0.3), delta(3, 1, 40, 20, 2)), dense(120)),
                             layer(delta(2, 2, 33, 16, 5)),
                             layer(parallel(attention(4, 1, 24, 72, 90, 70, None, 0.5), delta(4, 2, 20, 50, 8), 1.0, -0.5),
                                   moe(5, 1, 72, identity=1, shared=24))], pairs=(97, 13, 7), eps=3e-5),
    # head and state sizes of a large model; experts without a shared one, identity experts or groups
    "large_heads": config(256, 128, [layer(parallel(attention(8, 1, 128, 128, 100, 5, 20.0), delta(4, 2, 128, 128)), moe(8, 2, 64)),
                                     layer(delta(2, 1, 160, 64), dense(192))], pairs=(61, 5, 3)),
    # one of everything: a window of one token, no convolution history, one head, one expert beside the identity, one bucket
    "ones": config(64, 64, [layer(delta(1, 1, 32, 16, 1), moe(1, 1, 64, identity=1)),
                            layer(parallel(attention(1, 1, 8, 8, 1, 0, 2.0), delta(1, 1, 8, 8, 1)), moe(2, 2, 64, groups=(2, 2))),
                            layer(parallel(attention(2, 1, 64, 64, 2, 1), delta(1, 1, 16, 16, 1)), dense(64))], pairs=(1, 0, 1)),
    # no pair table, no window, no cap, no feed-forward in places; states larger than the chunked kernel takes
    "plain": config(96, 104, [layer(delta(2, 1, 192, 48, 4)),
                              layer(parallel(attention(4, 2, 64, 32), delta(4, 4, 32, 32, 4), 0.8, 0.8), dense(96))]),
    # recurrent layers only: no cache plane at all
    "states": config(96, 104, [layer(delta(4, 2, 48, 32, 3), moe(6, 2, 32, identity=2, groups=(4, 2), scale=2.0)),
                               layer(delta(2, 1, 96, 160, 4), dense(64))], pairs=(50, 3, 11)),
}
RANKS = {"odd": (24, 40), "large_heads": (64, 96), "ones": (1, 2), "plain": (16, 16), "states": (8, 8)}


def sharp_weights(name, seed=0, gain=4.0, calm=False):
    """Random weights whose attention queries (through their norm) are scaled up: attention picks few keys, so a wrong key shows.
    ``calm``: experts weigh little, for 16-bit runs of whole models, where a close call of a router may go either way and a state
    carries it on."""
    w = P.random_model(CONFIGS[name], seed, RANKS[name])
    for i, layer in enumerate(CONFIGS[name]["layers"]):
        if calm and layer["mlp"] and layer["mlp"]["kind"] == "moe":
            w[f"l{i}.ls2"] = (w[f"l{i}.ls2"].float() * 0.05).bfloat16()
    for k in w:
        if k.endswith(".mix.left.q.norm"):
            w[k] = (w[k].float() * gain).bfloat16()
    return w
