"""Plain, slow statement of the Pununex decoder (TEST INFRASTRUCTURE: the checker, never imported by the product).

One function per mechanism, whole sequences only, no cache, no batching, no fusion; ``dtype`` (float32 or float64) is
what everything is computed in.  Notation: x residual stream (every sublayer reads it as it is), W_* weights stored [out, in].

    x_0   = E[token] + B[row(previous token, token)]
    layer:  x += s1 * ln(mixer(x));   x += s2 * ln(mlp(x))      ln: layer norm with weight and bias, s: a vector per sublayer
    mixer:  a gated delta rule (``delta_mixer``), or windowed attention and a gated delta rule side by side (``parallel_mixer``)
    mlp:    ``gated_mlp`` (relu gate), or ``moe`` (silu experts, identity experts, a shared one), or none
    logits = W_head ln(x)"""
from __future__ import annotations

import torch

from .kugulorn import causal_conv, silu, softplus
from .mofarax import rms

__all__ = ["bigram_rows", "layer_norm", "window_mask", "sink_attention", "attention_mixer", "unit", "delta_scan", "delta_operands",
           "delta_mixer", "parallel_mixer", "gated_mlp", "route", "moe", "forward", "random_model", "tensor_shapes"]


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def bigram_rows(tokens, buckets: int, mul_prev: int, mul_cur: int) -> list[int]:
    return [buckets if i == 0 else (tokens[i - 1] * mul_prev + t * mul_cur) % buckets for i, t in enumerate(tokens)]


def layer_norm(x, weight, bias, eps: float):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * weight + bias


# ---- attention -------------------------------------------------------------------------------------------------------------
def window_mask(n: int, size: int | None, keep_first: int = 0):
    """[n, n] bool: may query i see key j?  Not ahead, and (size given) fewer than `size` positions behind or among the first
    `keep_first`."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    ok = j <= i
    return ok & ((i - j < size) | (j < keep_first)) if size else ok


def sink_attention(q, k, v, scale: float, softcap: float | None, sink, mask):
    """q [T, H, D], k [T, G, D], v [T, G, V], sink [H] -> [T, H, V]: capped scores, a denominator with one more term per head."""
    per = q.shape[1] // k.shape[1]
    out = torch.empty(q.shape[0], q.shape[1], v.shape[2], dtype=v.dtype)
    for h in range(q.shape[1]):
        s = (q[:, h] @ k[:, h // per].T) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        s = s.masked_fill(~mask, float("-inf"))
        top = torch.maximum(s.max(-1, keepdim=True).values, sink[h])
        e = torch.exp(s - top)
        out[:, h] = (e / (e.sum(-1, keepdim=True) + torch.exp(sink[h] - top))) @ v[:, h // per]
    return out


def attention_mixer(h, m: dict, w: dict, p: str, eps: float):
    t, mask = h.shape[0], m.get("mask") or {}
    q = (h @ w[p + "q"].T).reshape(t, m["heads"], m["dim"])
    k = (h @ w[p + "k"].T).reshape(t, m["kv_heads"], m["dim"])
    v = (h @ w[p + "v"].T).reshape(t, m["kv_heads"], m["vdim"])
    q, k = rms(q, eps) * w[p + "q.norm"], rms(k, eps) * w[p + "k.norm"]
    o = sink_attention(q, k, v, m["scale"], m.get("softcap"), w[p + "sink"],
                       window_mask(t, mask.get("size"), mask.get("keep_first", 0)))
    return o.reshape(t, -1) @ w[p + "o"].T


# ---- gated delta rule --------------------------------------------------------------------------------------------------------
def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_scan(q, k, v, beta, decay, state=None):
    """q / k [T, H, D], v [T, H, V], beta [T, H], decay [T, H, D] (a factor per key channel) -> o [T, H, V], token by token:
    S' = decay S_old,  u = beta (v - k S'),  S_new = S' + (k outer u),  o = q S_new, vectors as rows."""
    s = torch.zeros(k.shape[1], k.shape[2], v.shape[2], dtype=v.dtype) if state is None else state.clone()
    o = torch.empty_like(v)
    for i in range(v.shape[0]):
        s = decay[i][:, :, None] * s
        u = beta[i][:, None] * (v[i] - (s * k[i][:, :, None]).sum(1))
        s = s + k[i][:, :, None] * u[:, None, :]
        o[i] = (s * q[i][:, :, None]).sum(1)
    return o


def delta_operands(q, k, heads: int):
    """Convolved q / k [T, G, D] -> unit vectors per head, q scaled, one copy per head that reads them."""
    per = heads // k.shape[1]
    return (unit(q) * q.shape[2] ** -0.5).repeat_interleave(per, 1), unit(k).repeat_interleave(per, 1)


def delta_mixer(h, m: dict, w: dict, p: str, eps: float, channel_decay: bool):
    """``channel_decay``: a decay per key channel and a sigmoid gate, both of low rank; else a decay per head and a silu gate."""
    t, heads, kv, dim, vdim = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    zero = torch.zeros((), dtype=h.dtype)
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"], zero.expand(w[p + n].shape[0]))) for n in "qkv")
    q, k = delta_operands(q.reshape(t, kv, dim), k.reshape(t, kv, dim), heads)
    beta = sigmoid(h @ w[p + "b"].T)
    rate = torch.exp(w[p + "A_log"])
    if channel_decay:
        a = ((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]).reshape(t, heads, dim)
        gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T)
    else:
        a = (h @ w[p + "a"].T + w[p + "dt_bias"])[:, :, None].expand(t, heads, dim)
        gate = silu(h @ w[p + "g"].T)
    o = delta_scan(q, k, v.reshape(t, heads, vdim), beta, torch.exp(-rate[:, None] * softplus(a)))
    o = rms(o, eps) * w[p + "norm"] * gate.reshape(t, heads, vdim)
    return o.reshape(t, -1) @ w[p + "o"].T


def parallel_mixer(h, m: dict, w: dict, p: str, eps: float):
    return (m["left_scale"] * attention_mixer(h, m["left"], w, p + "left.", eps)
            + m["right_scale"] * delta_mixer(h, m["right"], w, p + "right.", eps, True))


# ---- feed-forward ------------------------------------------------------------------------------------------------------------
def gated_mlp(h, w: dict, p: str, act):
    return (act(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(z, correction, top: int, groups: int, keep: int, scale: float):
    """Router logits [T, R] -> (chosen [T, top], weights [T, top])."""
    s = torch.softmax(z, -1)
    choice = (s + correction).reshape(z.shape[0], groups, -1)
    best = choice.max(-1).values.topk(keep, -1).indices
    allowed = torch.zeros(z.shape[0], groups, dtype=torch.bool).scatter(1, best, True)
    choice = choice.masked_fill(~allowed[:, :, None], float("-inf")).reshape(z.shape)
    chosen = choice.topk(top, -1).indices
    weight = s.gather(1, chosen)
    return chosen, weight / (weight.sum(-1, keepdim=True) + 1e-20) * scale


def moe(h, m: dict, w: dict, p: str):
    r = m["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    chosen, weight = route(h @ w[p + "router"].T, w[p + "correction"], r["top"], groups["count"], groups["keep"], r["scale"])
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, c in zip(chosen[t].tolist(), weight[t]):
            y[t] += c * (gated_mlp(h[t], w, f"{p}e{e}.", silu) if e < r["experts"] else h[t])
    return y + gated_mlp(h, w, p + "shared.", silu) if m.get("shared") else y


# ---- the model -----------------------------------------------------------------------------------------------------------------
def forward(cfg: dict, weights: dict, tokens, dtype=torch.float64, residuals: list | None = None):
    """-> logits [T, vocab]; ``residuals`` receives the stream after every layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, big = cfg["norm"]["eps"], cfg["embedding"].get("bigram")
    tokens = torch.as_tensor(tokens).tolist()
    x = w["embed"][tokens]
    if big:
        x = x + w["bigram"][bigram_rows(tokens, big["buckets"], big["mul_prev"], big["mul_cur"])]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        if layer["type"] == "parallel":
            y = parallel_mixer(x, layer["mixer"], w, p + "mix.", eps)
        else:
            y = delta_mixer(x, layer["mixer"], w, p + "mix.", eps, False)
        x = x + w[p + "ls1"] * layer_norm(y, w[p + "norm1"], w[p + "norm1.b"], eps)
        if layer.get("mlp"):
            moe_kind = layer["mlp"]["kind"] == "moe"
            y = moe(x, layer["mlp"], w, p + "mlp.") if moe_kind else gated_mlp(x, w, p + "mlp.", torch.relu)
            x = x + w[p + "ls2"] * layer_norm(y, w[p + "norm2"], w[p + "norm2.b"], eps)
        if residuals is not None:
            residuals.append(x.clone())
    return layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["head"].T


def delta_shapes(m: dict, d: int, ranks: tuple[int, int] | None) -> dict:
    """``ranks``: of the decay's and the gate's projections (a decay per key channel), None = a decay per head."""
    h, g, dim, vdim, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
    out = {"q": (g * dim, d), "k": (g * dim, d), "v": (h * vdim, d), "q.conv": (g * dim, taps), "k.conv": (g * dim, taps),
           "v.conv": (h * vdim, taps), "b": (h, d), "A_log": (h,), "norm": (vdim,), "o": (d, h * vdim)}
    if ranks:
        out.update(a1=(ranks[0], d), a2=(h * dim, ranks[0]), dt_bias=(h * dim,), g1=(ranks[1], d), g2=(h * vdim, ranks[1]))
    else:
        out.update(a=(h, d), dt_bias=(h,), g=(h * vdim, d))
    return out


def tensor_shapes(cfg: dict, ranks: tuple[int, int] = (24, 24)) -> dict:
    d, v = cfg["width"], cfg["vocab"]
    out = {"embed": (v, d), "final.norm": (d,), "final.norm.b": (d,), "head": (v, d)}
    if cfg["embedding"].get("bigram"):
        out["bigram"] = (cfg["embedding"]["bigram"]["buckets"] + 1, d)
    for i, layer in enumerate(cfg["layers"]):
        m, mlp, p = layer["mixer"], layer.get("mlp"), f"l{i}."
        for n in ("1", "2") if mlp else ("1",):
            out[f"{p}norm{n}"] = out[f"{p}norm{n}.b"] = out[f"{p}ls{n}"] = (d,)
        if layer["type"] == "parallel":
            a, q = m["left"], p + "mix.left."
            out[q + "q"], out[q + "k"] = (a["heads"] * a["dim"], d), (a["kv_heads"] * a["dim"], d)
            out[q + "v"], out[q + "o"] = (a["kv_heads"] * a["vdim"], d), (d, a["heads"] * a["vdim"])
            out[q + "q.norm"] = out[q + "k.norm"] = (a["dim"],)
            out[q + "sink"] = (a["heads"],)
            out.update({f"{p}mix.right.{k}": s for k, s in delta_shapes(m["right"], d, ranks).items()})
        else:
            out.update({f"{p}mix.{k}": s for k, s in delta_shapes(m, d, None).items()})
        if not mlp:
            continue
        parts = {"": mlp["ff"]} if mlp["kind"] == "dense" else {f"e{j}.": mlp["expert"]["ff"] for j in range(mlp["router"]["experts"])}
        if mlp["kind"] == "moe":
            n = mlp["router"]["experts"] + mlp["router"].get("identity", 0)
            out[p + "mlp.router"], out[p + "mlp.correction"] = (n, d), (n,)
            if mlp.get("shared"):
                parts["shared."] = mlp["shared"]["ff"]
        for name, ff in parts.items():
            out[f"{p}mlp.{name}gate"] = out[f"{p}mlp.{name}up"] = (ff, d)
            out[f"{p}mlp.{name}down"] = (d, ff)
    return out


def random_model(cfg: dict, seed: int = 0, ranks: tuple[int, int] = (24, 24)) -> dict:
    """bf16 tensors of every name: unit-gain projections, norm weights and layer scales spread around 1, sinks and corrections that
    matter, decays from slow to fast."""
    g, out = torch.Generator().manual_seed(seed), {}
    for name, shape in tensor_shapes(cfg, ranks).items():
        r = torch.randn(*shape, generator=g)
        last = name.rsplit(".", 1)[-1]
        if last.startswith("norm"):
            r = 1.0 + 0.3 * r
        elif last in ("ls1", "ls2"):
            r = 1.0 + 0.5 * r
        elif last == "dt_bias":
            r = -2.5 + 1.5 * r
        elif last == "A_log":
            r = -1.0 + 1.5 * r
        elif last == "conv":
            r = r * shape[1] ** -0.5
        elif name.endswith(("norm.b", "norm1.b", "norm2.b")):
            r = 0.3 * r
        elif last == "correction":
            r = 0.1 * r
        elif last == "router":
            r = 2.0 * r * shape[1] ** -0.5
        elif len(shape) == 2 and name not in ("embed", "bigram"):
            r = r * shape[1] ** -0.5
        out[name] = r.to(torch.bfloat16)
    return out
