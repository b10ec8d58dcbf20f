"""Small Kugulorn configurations for the tests, and checkpoints of them with random weights."""
from mofarax_configs import write_checkpoint  # noqa: F401  (the same checkpoint layout)
from oracle import kugulorn as K


def latent(heads, dim, rot, vdim, q_rank, kv_rank, window=None, base=10000.0, scale=None, kv_from=None, ff=None, limit=2.5):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "rot": {"base": base, "dims": rot}, "scale": (dim + rot) ** -0.5 if scale is None else scale}
    if window:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff, "limit": limit} if ff else None}


def mamba(heads, vdim, state, groups=1, conv=4, norm_groups=1, ff=None, limit=2.5):
    m = {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}
    return {"type": "mamba2", "mixer": m, "mlp": {"kind": "dense", "ff": ff, "limit": limit} if ff else None}


def config(width, vocab, layers, mult=0.7, eps=1e-5):
    return {"architecture": "Kugulorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "layers": layers}


CONFIGS = {
    # odd sizes everywhere: norm parts across heads, shared latents under another window and other head sizes, a feed-forward behind
    # a state space layer and none behind an attention layer, one layer without a window
    "odd": config(200, 301, [latent(5, 20, 12, 24, 40, 48, 37, 500.0, 0.2, ff=120, limit=1.5), mamba(3, 20, 24, 1, 4, 5),
                             latent(3, 40, 12, 72, 56, 48, 90, 500.0, 0.13, kv_from=0), mamba(6, 40, 40, 3, 2, 1, ff=72, limit=0.8),
                             latent(2, 70, 30, 100, 33, 100, None, 1e5, ff=250)], mult=0.37, eps=3e-5),
    # head and state sizes of a large model, more heads than one workgroup of the decode kernel takes
    "large_heads": config(256, 128, [mamba(4, 64, 128, 2, 4, 2), latent(17, 128, 64, 128, 96, 512, 70, ff=192),
                                     latent(20, 96, 64, 160, 64, 512, 130, kv_from=1, ff=64)]),
    # one of everything: a window of one token, no convolution history, one head, one group, multiplier 1
    "ones": config(64, 64, [mamba(1, 16, 32, 1, 1, 1), latent(1, 32, 2, 16, 16, 32, 1, ff=64, limit=50.0),
                            latent(1, 8, 8, 8, 8, 16, 2, ff=64), mamba(2, 8, 8, 2, 8, 2)], mult=1.0),
    # recurrent layers only: no cache plane at all
    "states": config(96, 104, [mamba(4, 48, 64, 4, 3, 4, ff=64), mamba(6, 80, 160, 2, 5, 3)], mult=0.5),
}


def sharp_weights(cfg, seed=0, gain=4.0):
    """Random weights whose queries are scaled up: attention picks few keys, so a wrong key shows."""
    w = K.random_model(cfg, seed)
    for name in w:
        if name.endswith(".mix.uq"):
            w[name] = (w[name].float() * gain).bfloat16()
    return w
