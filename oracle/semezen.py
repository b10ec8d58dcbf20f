"""Plain, slow statement of the Semezen decoder (TEST INFRASTRUCTURE: the checker, never imported by the product).

One function per mechanism, whole sequences only, no cache, no batching, no fusion; ``dtype`` (float32 or float64) is
what everything is computed in.  Notation: X [T, s, width] residual streams, W_* weights stored [out, in].

    X_j   = E[token], every stream j
    sublayer f with (a, B, c) = hc.in, hc.mix, hc.out:   u = sum_j a_j X_j;   X_j <- sum_i B_ij X_i + c_j f(rms(u) w)
    layer: the mixer, whose normed input is first blended with the previous token's (``token_shift``), then the mlp or none
    mixer: windowed attention with keys for values and a gate (``attention_mixer``), or a gated running mean (``mingru_mixer``)
    mlp:   ``dense_mlp`` (gelu), or ``moe`` (clamped gated experts behind a sigmoid router)
    logits = W_head rms(sum_j X_j) w"""
from __future__ import annotations

import math

import torch

from .kugulorn import silu
from .mofarax import rms
from .pununex import sigmoid, window_mask

__all__ = ["scaled_frequencies", "rotate_halves", "attend", "attention_mixer", "gru_scan", "mingru_mixer", "gelu", "dense_mlp", "expert",
           "route", "moe", "token_shift", "read_streams", "write_streams", "forward", "tensor_shapes", "random_model"]


# ---- attention -------------------------------------------------------------------------------------------------------------
def scaled_frequencies(base: float, dims: int, scaling: dict | None, dtype=torch.float64):
    """[dims / 2]: base^(-2i/dims); with ``scaling``, those whose wavelength is long against the original context divided by the
    factor, a linear blend (in original / wavelength) between the two bounds."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            turns = scaling["original"] * f / (2.0 * math.pi)      # original / wavelength
            if turns < scaling["low"]:
                f = f / scaling["factor"]
            elif turns <= scaling["high"]:
                s = (turns - scaling["low"]) / (scaling["high"] - scaling["low"])
                f = (1.0 - s) * f / scaling["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=dtype)


def rotate_halves(x, positions, freq):
    """x [T, H, D]: dim i < len(freq) turns with dim i + len(freq) by positions * freq[i]; the dims behind pass."""
    n = freq.numel()
    angle = positions.to(freq.dtype)[:, None] * freq[None, :]
    c, s = angle.cos()[:, None].to(x.dtype), angle.sin()[:, None].to(x.dtype)
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n:]], -1)


def attend(q, k, v, scale: float, mask):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]."""
    per = q.shape[1] // k.shape[1]
    out = torch.empty(q.shape[0], q.shape[1], v.shape[2], dtype=v.dtype)
    for h in range(q.shape[1]):
        s = ((q[:, h] @ k[:, h // per].T) * scale).masked_fill(~mask, float("-inf"))
        out[:, h] = torch.softmax(s, -1) @ v[:, h // per]
    return out


def attention_mixer(h, m: dict, w: dict, p: str, eps: float):
    t = h.shape[0]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).reshape(t, m["heads"], m["dim"])
    k = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(t, m["kv_heads"], m["dim"])
    v = k
    freq = scaled_frequencies(m["rot"]["base"], m["rot"]["dims"], m["rot"].get("scaling"))
    q, k = (rms(rotate_halves(z, torch.arange(t), freq), eps) for z in (q, k))
    o = attend(q, k, v, m["scale"], window_mask(t, (m.get("mask") or {}).get("size")))
    return (o.reshape(t, -1) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---- gated running mean ------------------------------------------------------------------------------------------------------
def gru_scan(z, u, state=None):
    """z, u [T, width] -> S [T, width], token by token: S <- (1 - z) S + z (u + 1/2 for u >= 0, else sigmoid(u))."""
    s = torch.zeros_like(z[0]) if state is None else state
    cand = torch.where(u >= 0, u + 0.5, sigmoid(u))
    out = torch.empty_like(z)
    for t in range(z.shape[0]):
        s = (1.0 - z[t]) * s + z[t] * cand[t]
        out[t] = s
    return out


def mingru_mixer(h, w: dict, p: str):
    z, u = sigmoid(h @ w[p + "z"].T + w[p + "z.b"]), h @ w[p + "x"].T + w[p + "x.b"]
    return (gru_scan(z, u) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---- feed-forward ------------------------------------------------------------------------------------------------------------
def gelu(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def dense_mlp(h, w: dict, p: str):
    return gelu(h @ w[p + "up"].T) @ w[p + "down"].T


def expert(h, w: dict, p: str, limit: float):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def route(z, top: int):
    """Router logits [T, R] -> (chosen [T, top], their scores [T, top])."""
    s = sigmoid(z)
    chosen = s.topk(top, -1).indices
    return chosen, s.gather(1, chosen)


def moe(h, m: dict, w: dict, p: str):
    """Sum over a token's choices of expert(score * h)."""
    chosen, score = route(h @ w[p + "router"].T, m["router"]["top"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, c in zip(chosen[t].tolist(), score[t]):
            y[t] += expert(c * h[t], w, f"{p}e{e}.", m["expert"]["limit"])
    return y


# ---- the streams -------------------------------------------------------------------------------------------------------------
def token_shift(h, share):
    """Each row moved towards the row before it (zeros ahead of the first) by ``share``, element by element."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (before - h) * share


def read_streams(x, a):
    return (x * a[:, None]).sum(1)


def write_streams(x, mix, out, y):
    """x [T, s, width], mix [from, to]."""
    return torch.einsum("tiw,ij->tjw", x, mix) + out[None, :, None] * y[:, None, :]


def forward(cfg: dict, weights: dict, tokens, dtype=torch.float64, residuals: list | None = None):
    """-> logits [T, vocab]; ``residuals`` receives the sum of the streams after every layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens)][:, None].repeat(1, cfg["streams"], 1)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = rms(read_streams(x, w[p + "hc1.in"]), eps) * w[p + "norm1"]
        h = token_shift(h, w[p + "shift"])
        if layer["type"] == "attention":
            y = attention_mixer(h, layer["mixer"], w, p + "mix.", eps)
        else:
            y = mingru_mixer(h, w, p + "mix.")
        x = write_streams(x, w[p + "hc1.mix"], w[p + "hc1.out"], y)
        if layer.get("mlp"):
            h = rms(read_streams(x, w[p + "hc2.in"]), eps) * w[p + "norm2"]
            y = moe(h, layer["mlp"], w, p + "mlp.") if layer["mlp"]["kind"] == "moe" else dense_mlp(h, w, p + "mlp.")
            x = write_streams(x, w[p + "hc2.mix"], w[p + "hc2.out"], y)
        if residuals is not None:
            residuals.append(x.sum(1))
    return (rms(x.sum(1), eps) * w["final.norm"]) @ w["head"].T


def tensor_shapes(cfg: dict) -> dict:
    d, v, s = cfg["width"], cfg["vocab"], cfg["streams"]
    out = {"embed": (v, d), "final.norm": (d,), "head": (v, d)}
    for i, layer in enumerate(cfg["layers"]):
        m, mlp, p = layer["mixer"], layer.get("mlp"), f"l{i}."
        out[p + "shift"] = (d,)
        for n in ("1", "2") if mlp else ("1",):
            out[f"{p}norm{n}"] = (d,)
            out[f"{p}hc{n}.in"], out[f"{p}hc{n}.out"], out[f"{p}hc{n}.mix"] = (s,), (s,), (s, s)
        if layer["type"] == "attention":
            q, k = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
            out.update({p + "mix.q": (q, d), p + "mix.q.b": (q,), p + "mix.k": (k, d), p + "mix.k.b": (k,), p + "mix.g": (q, d),
                        p + "mix.o": (d, q)})
        else:
            n = m["width"]
            out.update({p + "mix." + k: (n, d) for k in "zxg"})
            out.update({p + "mix.z.b": (n,), p + "mix.x.b": (n,), p + "mix.o": (d, n)})
        if not mlp:
            continue
        if mlp["kind"] == "dense":
            out[p + "mlp.up"], out[p + "mlp.down"] = (mlp["ff"], d), (d, mlp["ff"])
            continue
        out[p + "mlp.router"] = (mlp["router"]["experts"], d)
        for e in range(mlp["router"]["experts"]):
            q, ff = f"{p}mlp.e{e}.", mlp["expert"]["ff"]
            out[q + "gate"] = out[q + "up"] = (ff, d)
            out[q + "down"] = (d, ff)
    return out


def random_model(cfg: dict, seed: int = 0) -> dict:
    """bf16 tensors of every name: unit-gain projections, norm weights spread around 1, shares of the previous token between 0 and
    1 and beyond, streams that are read and written unlike, gates that are open, shut and between."""
    g, out = torch.Generator().manual_seed(seed), {}
    s = cfg["streams"]
    for name, shape in tensor_shapes(cfg).items():
        r = torch.randn(*shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if last.startswith("norm"):
            r = 1.0 + 0.3 * r
        elif last == "shift":
            r = 0.5 + 0.4 * r
        elif last == "in":
            r = 1.0 / s + 0.5 * r
        elif last == "out":
            r = 1.0 + 0.5 * r
        elif last == "mix":
            if name.endswith(".mix"):
                r = torch.eye(s) + 0.3 * r / s
        elif name.endswith(".z.b"):
            r = -1.5 + 1.5 * r
        elif last == "b":
            r = 0.5 * r
        elif last == "router":
            r = 1.5 * r * shape[1] ** -0.5
        elif len(shape) == 2 and name != "embed":
            r = r * shape[1] ** -0.5
        out[name] = r.to(torch.bfloat16)
    return out
