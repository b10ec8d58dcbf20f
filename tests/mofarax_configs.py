"""Small Mofarax configurations for the tests, and checkpoints of them with random weights."""
import json

from oracle import mofarax as M


def layer(heads, kv, dim, size=None, base=10000.0, dims=None, scale=None, ff=None):
    m = {"dim": dim, "vdim": dim, "heads": heads, "kv_heads": kv, "rot": {"base": base, "dims": dim if dims is None else dims},
         "scale": dim ** -0.5 if scale is None else scale}
    if size:
        m["mask"] = {"size": size}
    return {"type": "attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(width, vocab, layers, loop=None, side=None, scale=3.0, eps=1e-6):
    c = {"architecture": "Mofarax", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps},
         "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    if side:
        c["token_side"] = {"dim": side}
    return c


CONFIGS = {
    # layers of unlike shape, odd sizes everywhere: grouped heads, partial rotation, a layer without feed-forward
    "odd": config(200, 301, [layer(6, 2, 48, 50, 500.0, 32, 0.2, 120), layer(4, 4, 32, 33, 1e4, 16, None, None),
                             layer(5, 1, 24, 100, 1e5, 24, 0.25, 72), layer(3, 3, 56, 70, 1e4, 6, 0.13, 250)],
                  loop=(1, 3, 2), side=20, scale=14.1, eps=3e-5),
    # grouped heads at the kernels' own head dim (the matrix-core decode kernel), the loop over all layers
    "gqa128": config(256, 128, [layer(8, 2, 128, 160, ff=192), layer(4, 1, 128, 64, ff=320)], loop=(0, 2, 2), side=64, scale=1.0),
    # head dim above 128, no mask in one layer, neither loop nor side input
    "wide_heads": config(192, 97, [layer(2, 1, 160, None, ff=64), layer(2, 2, 200, 90, dims=100, ff=96)]),
    # one head, chunks shorter than a wave's 32 rows, the loop at the end, a single pass
    "tiny_chunk": config(64, 64, [layer(1, 1, 64, 7, ff=64), layer(2, 1, 64, 40, ff=64)], loop=(1, 2, 1), side=8),
}


def sharp_weights(cfg, seed=0, gain=4.0):
    """Random weights whose queries are scaled up: attention picks few keys, so a wrong key shows."""
    w = M.random_model(cfg, seed)
    for name in w:
        if name.endswith(".mix.q"):
            w[name] = (w[name].float() * gain).bfloat16()
    return w


def write_checkpoint(path, cfg, weights):
    from safetensors.torch import save_file

    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in weights.items()}, str(path / "model.safetensors"))
    return str(path)
