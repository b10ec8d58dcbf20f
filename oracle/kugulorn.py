"""Plain, slow statement of the Kugulorn decoder (TEST INFRASTRUCTURE: the checker, never imported by the product).

One function per mechanism, whole sequences only, no cache, no batching, no fusion; ``dtype`` (float32 or float64) is
what everything is computed in.  Notation: x residual stream, h normed stream, W_* weights stored [out, in].

    x_0   = E[token]
    layer:  x += m * s1 * (rms(mixer(rms(x) * w1)) * w1b);   x += m * s2 * (rms(mlp(rms(x) * w2)) * w2b)
            m: one number of the model, s1 / s2: a vector per sublayer; a layer may have no mlp
    mixer:  latent attention (``latent_attention_mixer``) or a selective state space (``mamba2_mixer``)
    mlp:    ``clamped_glu``
    logits = W_head (rms(x) * w_f)"""
from __future__ import annotations

import torch

from .mofarax import rms, rotate_interleaved

__all__ = ["window_mask", "latents", "latent_attention", "latent_attention_mixer", "causal_conv", "ssm_scan", "gated_group_norm",
           "mamba2_mixer", "clamped_glu", "forward", "random_model", "tensor_shapes"]


def silu(z):
    return z / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.where(z > 0, z, torch.zeros_like(z)) + torch.log1p(torch.exp(-z.abs()))


# ---- latent attention ------------------------------------------------------------------------------------------------------
def window_mask(n: int, size: int | None):
    """[n, n] bool: may query i see key j?  Not ahead, and (size given) fewer than `size` positions behind."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    ok = j <= i
    if size:
        ok = ok & (i - j < size)
    return ok


def latents(h, w_dkv, w_norm, rank: int, base: float, eps: float):
    """What a layer caches: c = rms(first `rank` rows of W_dkv h) * w, and the remaining rows rotated (one part, all heads)."""
    z = h @ w_dkv.T
    pos = torch.arange(h.shape[0])
    c = rms(z[:, :rank], eps) * w_norm
    rot = z[:, rank:]
    return c, rotate_interleaved(rot[:, None, :], pos, base, rot.shape[1])[:, 0]


def latent_attention(q_plain, q_rot, k_plain, k_rot, v, scale: float, mask):
    """q_plain / k_plain [T, H, D], q_rot [T, H, R], k_rot [T, R], v [T, H, V] -> [T, H, V]."""
    out = torch.empty(q_plain.shape[0], q_plain.shape[1], v.shape[2], dtype=v.dtype)
    for head in range(q_plain.shape[1]):
        s = (q_plain[:, head] @ k_plain[:, head].T + q_rot[:, head] @ k_rot.T) * scale
        p = torch.softmax(s.masked_fill(~mask, float("-inf")), -1)
        out[:, head] = p @ v[:, head]
    return out


def latent_attention_mixer(h, m: dict, w: dict, p: str, shared: dict, index: int, eps: float):
    """``shared``: layer index -> (c, rotated part) of the layers that have a W_dkv."""
    t, heads, dim, rot, vdim = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    base = m["rot"]["base"]
    if m.get("kv_from") is None:
        shared[index] = latents(h, w[p + "dkv"], w[p + "dkv.norm"], m["kv_rank"], base, eps)
    c, k_rot = shared[index if m.get("kv_from") is None else m["kv_from"]]
    c_q = rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
    q = (c_q @ w[p + "uq"].T).reshape(t, heads, dim + rot)
    q_rot = rotate_interleaved(q[:, :, dim:], torch.arange(t), base, rot)
    k = (c @ w[p + "uk"].T).reshape(t, heads, dim)
    v = (c @ w[p + "uv"].T).reshape(t, heads, vdim)
    o = latent_attention(q[:, :, :dim], q_rot, k, k_rot, v, m["scale"], window_mask(t, (m.get("mask") or {}).get("size")))
    return o.reshape(t, heads * vdim) @ w[p + "o"].T


# ---- selective state space ---------------------------------------------------------------------------------------------------
def causal_conv(x, weight, bias):
    """x [T, C], weight [C, taps] (its last column belongs to the current token), zeros ahead of the first token."""
    taps, y = weight.shape[1], bias.expand(x.shape).clone()
    for back in range(taps):
        shifted = torch.cat([torch.zeros(min(back, x.shape[0]), x.shape[1], dtype=x.dtype), x[:max(x.shape[0] - back, 0)]])
        y = y + shifted * weight[:, taps - 1 - back]
    return y


def ssm_scan(x, b, c, dt, a_log, d):
    """x [T, H, P], b / c [T, G, N], dt [T, H] (positive), a_log / d [H] -> y [T, H, P], token by token:
    S <- exp(-exp(a_log) dt) S + dt b x^T,  y = S^T c + d x; head h reads group h // (H / G)."""
    t, heads, p = x.shape
    per = heads // b.shape[1]
    s, y = torch.zeros(heads, b.shape[2], p, dtype=x.dtype), torch.empty_like(x)
    b, c = b.repeat_interleave(per, 1), c.repeat_interleave(per, 1)
    decay = torch.exp(-torch.exp(a_log) * dt)
    for i in range(t):
        s = decay[i][:, None, None] * s + dt[i][:, None, None] * b[i][:, :, None] * x[i][:, None, :]
        y[i] = (s * c[i][:, :, None]).sum(1) + d[:, None] * x[i]
    return y


def gated_group_norm(y, z, weight, groups: int, eps: float):
    """rms of (y * silu(z)) in `groups` equal parts, then the weight."""
    g = (y * silu(z)).reshape(y.shape[0], groups, -1)
    return rms(g, eps).reshape(y.shape) * weight


def mamba2_mixer(h, m: dict, w: dict, p: str, eps: float):
    t, heads, vdim, n, groups = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = heads * vdim
    z, xbc, dt = (h @ w[p + "in"].T).split([inner, inner + 2 * groups * n, heads], 1)
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, b, c = xbc.split([inner, groups * n, groups * n], 1)
    y = ssm_scan(x.reshape(t, heads, vdim), b.reshape(t, groups, n), c.reshape(t, groups, n), softplus(dt + w[p + "dt_bias"]),
                 w[p + "A_log"], w[p + "D"]).reshape(t, inner)
    return gated_group_norm(y, z, w[p + "norm"], m["norm_groups"], eps) @ w[p + "o"].T


# ---- feed-forward ------------------------------------------------------------------------------------------------------------
def clamped_glu(gate, up, limit: float):
    g = torch.minimum(gate, torch.tensor(limit, dtype=gate.dtype))
    u = up.clamp(-limit, limit)
    return g / (1.0 + torch.exp(-1.702 * g)) * (u + 1.0)


# ---- the model -----------------------------------------------------------------------------------------------------------------
def forward(cfg: dict, weights: dict, tokens, dtype=torch.float64, residuals: list | None = None):
    """-> logits [T, vocab]; ``residuals`` receives the stream after every layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x, shared = w["embed"][torch.as_tensor(tokens)], {}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = rms(x, eps) * w[p + "norm1"]
        if layer["type"] == "mamba2":
            y = mamba2_mixer(h, layer["mixer"], w, p + "mix.", eps)
        else:
            y = latent_attention_mixer(h, layer["mixer"], w, p + "mix.", shared, i, eps)
        x = x + mult * w[p + "ls1"] * (rms(y, eps) * w[p + "norm1b"])
        if layer["mlp"] is not None:
            h = rms(x, eps) * w[p + "norm2"]
            y = clamped_glu(h @ w[p + "mlp.gate"].T, h @ w[p + "mlp.up"].T, layer["mlp"]["limit"]) @ w[p + "mlp.down"].T
            x = x + mult * w[p + "ls2"] * (rms(y, eps) * w[p + "norm2b"])
        if residuals is not None:
            residuals.append(x.clone())
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T


def tensor_shapes(cfg: dict) -> dict:
    d, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],), "head": (cfg["vocab"], cfg["width"])}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}."
        for name in ("norm1", "norm1b", "ls1") + (("norm2", "norm2b", "ls2") if layer["mlp"] else ()):
            out[p + name] = (d,)
        q = p + "mix."
        if layer["type"] == "mamba2":
            inner, bc = m["heads"] * m["vdim"], 2 * m["groups"] * m["state"]
            out[q + "in"], out[q + "o"] = (2 * inner + bc + m["heads"], d), (d, inner)
            out[q + "conv"], out[q + "conv.b"] = (inner + bc, m["conv"]), (inner + bc,)
            out[q + "dt_bias"] = out[q + "A_log"] = out[q + "D"] = (m["heads"],)
            out[q + "norm"] = (inner,)
        else:
            h = m["heads"]
            out[q + "dq"], out[q + "dq.norm"] = (m["q_rank"], d), (m["q_rank"],)
            out[q + "uq"], out[q + "o"] = (h * (m["dim"] + m["rot_dim"]), m["q_rank"]), (d, h * m["vdim"])
            out[q + "uk"], out[q + "uv"] = (h * m["dim"], m["kv_rank"]), (h * m["vdim"], m["kv_rank"])
            if m.get("kv_from") is None:
                out[q + "dkv"], out[q + "dkv.norm"] = (m["kv_rank"] + m["rot_dim"], d), (m["kv_rank"],)
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            out[p + "mlp.gate"] = out[p + "mlp.up"] = (ff, d)
            out[p + "mlp.down"] = (d, ff)
    return out


def random_model(cfg: dict, seed: int = 0) -> dict:
    """bf16 tensors of every name: unit-gain projections, norm weights and layer scales spread around 1 (some negative scales),
    decays from slow to fast."""
    g, out = torch.Generator().manual_seed(seed), {}
    for name, shape in tensor_shapes(cfg).items():
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
        elif last == "b":
            r = 0.3 * r
        elif len(shape) == 2 and name != "embed":
            r = r * shape[1] ** -0.5
        out[name] = r.to(torch.bfloat16)
    return out
