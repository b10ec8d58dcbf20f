"""Plain, slow statement of the Mofarax decoder (TEST INFRASTRUCTURE: the checker, never imported by the product).

One function per mechanism, whole sequences only, no cache, no batching, no fusion; ``dtype`` (float32 or float64) is
what everything is computed in.  Notation: x residual stream, h normed stream, W_* weights stored [out, in].

    x_0   = s_e * E[token]
    layer:  h = rms(x) * (1 + w);   x += attention(h) + mlp(h)          both sublayers read the same h
            g = gelu(W_g x) * e[token];  y = W_p g;   x += rms(y) * w_y       e: the layer's slice of the side table
    loop:   the layers [start, stop) run `times` times over the same weights; ahead of pass t: x += x_0 when t > 0,
            then x += step[t]
    logits = W_head (rms(x) * (1 + w_f))

``attention``: grouped heads, values = the projected keys before rotation, rotation of interleaved pairs of the first
`dims` dimensions, and a key is visible to a query of the same chunk of positions at or behind it."""
from __future__ import annotations

import math

import torch

__all__ = ["gelu_tanh", "rms", "rms_norm", "rotate_interleaved", "chunk_mask", "grouped_attention", "attention_mixer",
           "gated_mlp", "side_input", "layer_schedule", "forward", "random_model", "tensor_shapes"]


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms(x, eps: float):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps: float, offset: float):
    """rms(x) * (offset + w): offset 1 = a weight stored around zero, 0 = a plain weight."""
    return rms(x, eps) * (offset + w)


def rotate_interleaved(x, positions, base: float, dims: int):
    """x [T, heads, D]: the pair (2i, 2i+1), i < dims/2, turned by the angle position * base^(-2i/dims)."""
    out = x.clone()
    for i in range(dims // 2):
        a = positions.to(torch.float64) * (float(base) ** (-2.0 * i / dims))
        c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
        u, v = x[:, :, 2 * i], x[:, :, 2 * i + 1]
        out[:, :, 2 * i] = u * c - v * s
        out[:, :, 2 * i + 1] = v * c + u * s
    return out


def chunk_mask(n: int, size: int | None):
    """[n, n] bool: may query i see key j?  Same chunk of `size` positions (None: one chunk), not ahead."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    ok = j <= i
    if size:
        ok = ok & (i // size == j // size)
    return ok


def grouped_attention(q, k, v, scale: float, mask):
    """q [T, H, D], k / v [T, G, D]; query head h reads key/value head h // (H / G)."""
    heads, groups = q.shape[1], k.shape[1]
    out = torch.empty(q.shape[0], heads, v.shape[2], dtype=q.dtype)
    for h in range(heads):
        g = h // (heads // groups)
        score = (q[:, h] @ k[:, g].T) * scale
        out[:, h] = torch.softmax(score.masked_fill(~mask, -math.inf), dim=-1) @ v[:, g]
    return out


def attention_mixer(h, positions, m: dict, w: dict):
    """m: the mixer's sizes and constants; w: {'q', 'k', 'o'}."""
    t = h.shape[0]
    q = (h @ w["q"].T).view(t, m["heads"], m["dim"])
    k = (h @ w["k"].T).view(t, m["kv_heads"], m["dim"])
    rot = m["rot"]
    qr = rotate_interleaved(q, positions, rot["base"], rot["dims"])
    kr = rotate_interleaved(k, positions, rot["base"], rot["dims"])
    size = (m.get("mask") or {}).get("size")
    o = grouped_attention(qr, kr, k, m["scale"], chunk_mask(t, size))
    return o.reshape(t, -1) @ w["o"].T


def gated_mlp(h, w: dict):
    return (gelu_tanh(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def side_input(x, e, w: dict, eps: float):
    y = (gelu_tanh(x @ w["gate"].T) * e) @ w["proj"].T
    return rms_norm(y, w["norm"], eps, 0.0)


def layer_schedule(n_layers: int, loop: dict | None):
    """[(layer, pass or None when the layer starts no pass)]: the layer runs in order."""
    if not loop:
        return [(i, None) for i in range(n_layers)]
    a, b, n = loop["start"], loop["stop"], loop["times"]
    runs = [(i, None) for i in range(a)]
    for t in range(n):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n_layers)]


def _layer_weights(w: dict, i: int, part: str):
    p = f"l{i}.{part}."
    return {k[len(p):]: v for k, v in w.items() if k.startswith(p)}


def forward(cfg: dict, weights: dict, tokens, dtype=torch.float32, states: list | None = None):
    """Logits [T, vocab] of one sequence; ``states`` (if given) collects the residual stream after every layer run."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    pos = torch.arange(tokens.numel())
    eps = cfg["norm"]["eps"]
    x0 = w["embed"][tokens] * cfg["embedding"]["scale"]
    x = x0.clone()
    side_dim = (cfg.get("token_side") or {}).get("dim")
    for i, start in layer_schedule(len(cfg["layers"]), cfg.get("loop")):
        if start is not None:
            if start > 0:
                x = x + x0
            x = x + w["loop.step"][start]
        layer = cfg["layers"][i]
        h = rms_norm(x, w[f"l{i}.norm1"], eps, 1.0)
        y = attention_mixer(h, pos, layer["mixer"], _layer_weights(w, i, "mix"))
        if layer.get("mlp"):
            y = y + gated_mlp(h, _layer_weights(w, i, "mlp"))
        x = x + y
        if side_dim:
            e = w["side.embed"][tokens][:, i * side_dim:(i + 1) * side_dim]
            x = x + side_input(x, e, _layer_weights(w, i, "side"), eps)
        if states is not None:
            states.append(x.clone())
    return rms_norm(x, w["final.norm"], eps, 1.0) @ w["head"].T


# ---- small random models for the tests --------------------------------------------------------------------------------
def tensor_shapes(cfg: dict) -> dict:
    """name -> shape of every tensor a checkpoint of this configuration holds."""
    v, d = cfg["vocab"], cfg["width"]
    out = {"embed": (v, d), "final.norm": (d,), "head": (v, d)}
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], d)
    s = (cfg.get("token_side") or {}).get("dim")
    if s:
        out["side.embed"] = (v, s * len(cfg["layers"]))
    for i, layer in enumerate(cfg["layers"]):
        m, f = layer["mixer"], layer.get("mlp")
        out[f"l{i}.norm1"] = (d,)
        out[f"l{i}.mix.q"] = (m["heads"] * m["dim"], d)
        out[f"l{i}.mix.k"] = (m["kv_heads"] * m["dim"], d)
        out[f"l{i}.mix.o"] = (d, m["heads"] * m["vdim"])
        if f:
            out[f"l{i}.mlp.gate"] = out[f"l{i}.mlp.up"] = (f["ff"], d)
            out[f"l{i}.mlp.down"] = (d, f["ff"])
        if s:
            out[f"l{i}.side.gate"], out[f"l{i}.side.proj"], out[f"l{i}.side.norm"] = (s, d), (d, s), (d,)
    return out


def random_model(cfg: dict, seed: int = 0) -> dict:
    """bf16-representable random weights of unit-gain scale (norm weights around their neutral value)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(*shape, generator=g)
        if name.endswith("side.norm"):
            t = 1.0 + 0.2 * t
        elif name.endswith("norm1") or name == "final.norm":
            t = 0.2 * t
        elif name == "embed":
            t = t / cfg["embedding"]["scale"]
        elif name == "loop.step":
            t = 0.3 * t
        elif name != "side.embed":
            t = t / math.sqrt(shape[-1])
        out[name] = t.bfloat16()
    return out
