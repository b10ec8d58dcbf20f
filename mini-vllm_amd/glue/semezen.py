"""Semezen decoder glue: several fp32 residual streams, one launch between two sublayers.

    X_j = E[token], every stream j; h = rms(read X) w, blended with the token before's                  (one launch)
    attention:  [q | k | gate] GEMM with biases
      rotation, unit length + K/V store + attention + gate (decode: ONE launch) -> output GEMM
    gated running mean:  [z | x | gate] GEMM with biases -> recurrence (layers/mingru.py) -> output GEMM
    -> streams mixed and written, what the next sublayer reads normed (and blended)                      (one launch)
    up GEMM with gelu -> down GEMM, or experts (layers/moe.py)
    -> the same launch
Values are the projected keys: the K plane of the cache holds rotated keys of unit length, the V plane the projected ones.  A head's
rotated pairs lie side by side in the stored weights (layers/rotary_embedding.py: halves_as_pairs).  Head dims between the
kernels' sizes, and widths that are no multiple of 64, are zero-padded in the weights at load time."""
from __future__ import annotations

import os

import torch
from torch import nn

from .. import hip_ops
from ..layers import (Attention, ExpertMLP, HyperConnection, MinGRU, ParallelLMHead, ResidualStreams, Segment, SegmentedLinear, TokenShift,
                      get_rope, halves_as_pairs, padded_parameter)
from ..layers.linear import gelu_linear, pad_to
from ..parallel_state import get_tensor_parallel_world_size
from ..utils.context import get_context
from ..utils.loader import load_weight
from .mofarax import kernel_head_dim

__all__ = ["SemezenLayer", "SemezenForCausalLM"]

# rows up to which a decode step folds rotation + K/V store into the attention launch (see glue/qwen.py)
ROPE_FOLD_MAX_ROWS = int(os.environ.get("MV_ROPE_FOLD_MAX", "128"))


class KeyValueAttention(nn.Module):
    """Windowed attention over keys that are the values as well, its output gated."""

    def __init__(self, width: int, spec, eps: float, max_positions: int) -> None:
        super().__init__()
        d, order = kernel_head_dim(spec.dim), halves_as_pairs(spec.dim, spec.rot_dims)
        self.heads, self.kv_heads, self.dim, self.head_dim, self.eps = spec.heads, spec.kv_heads, spec.dim, d, eps
        rows = lambda name, heads: Segment(name, heads, spec.dim, d, order=order)
        self.in_proj = SegmentedLinear(width, [rows("q", spec.heads), rows("k", spec.kv_heads), rows("g", spec.heads)], split="out", bias=True)
        self.o = SegmentedLinear(width, [rows("o", spec.heads)], split="in")
        scaling = spec.scaling and {"type": "wavelength", "factor": spec.scaling.factor, "low": spec.scaling.low,
                                    "high": spec.scaling.high, "original": spec.scaling.original}
        self.rotary = get_rope(d, spec.rot_dims, max_positions, spec.rot_base, scaling, interleaved=True)
        self.attn = Attention(spec.heads, d, spec.scale, spec.kv_heads, mask=hip_ops.AttnMask(window=spec.window))

    def forward(self, h, positions):
        ctx, t, d, at, attn = get_context(), h.shape[0], self.head_dim, self.in_proj.offsets, self.attn
        z, cols = self.in_proj(h), self.heads * d
        q, k = (z[:, at[n]:at[n] + heads * d].view(t, heads, d) for n, heads in (("q", self.heads), ("k", self.kv_heads)))
        gate = z[:, at["g"]:at["g"] + cols]
        wide = self.o.weight.shape[1]
        mixed = (torch.empty if wide == cols else torch.zeros)((t, wide), dtype=h.dtype, device=h.device)
        out = mixed[:, :cols].view(t, self.heads, d)
        has_cache = attn.k_cache.numel() > 0
        cos, sin = self.rotary._tables(h.device)
        how = {"interleaved_pairs": self.rotary.interleaved_pairs, "norm_dim": self.dim, "unit_norm": True}
        turn = (positions, cos, sin, None, None, self.eps)
        o = None
        if (t <= ROPE_FOLD_MAX_ROWS and has_cache and not ctx.is_prefill and ctx.slot_mapping is not None
                and ctx.block_tables is not None and ctx.context_lens is not None):
            o = hip_ops.rope_paged_decode(q, k, k, *turn, ctx.slot_mapping, attn.k_cache, attn.v_cache, ctx.block_tables,
                                          ctx.context_lens, attn.scale, out=out, mask=attn.gated(gate), **how)
        if o is None:
            want_k = ctx.is_prefill and not (ctx.prefix_cached and has_cache)
            q, k_rot = hip_ops.rope_qk_store(q, k, k, *turn, k_cache=attn.k_cache if has_cache else None,
                                             v_cache=attn.v_cache if has_cache else None,
                                             slot_mapping=ctx.slot_mapping if has_cache else None, want_k_out=want_k, **how)
            attn(q, k_rot, k, kv_stored=True, out=out, gate=gate)
        return self.o(mixed, partial_ok=True)


class GeluMLP(nn.Module):
    def __init__(self, width: int, ff: int) -> None:
        super().__init__()
        self.up = SegmentedLinear(width, [Segment("up", ff)], split="out")
        self.down = SegmentedLinear(width, [Segment("down", ff)], split="in")

    def forward(self, h):
        return self.down(gelu_linear(h, self.up), partial_ok=True), None


class SemezenLayer(nn.Module):
    def __init__(self, config, index: int) -> None:
        super().__init__()
        spec, width = config.layers[index], config.hidden_size
        w, m = pad_to(width), spec.mlp
        self.mix = (KeyValueAttention(width, spec.mixer, config.norm_eps, config.max_position_embeddings or 4096)
                    if spec.type == "attention" else MinGRU(width, spec.mixer.width))
        self.hc1, self.norm1, self.shift = HyperConnection(config.streams), padded_parameter(w), TokenShift(w)
        self.mlp = None
        if m is not None:
            self.mlp = (GeluMLP(width, m.ff) if not hasattr(m, "experts") else
                        ExpertMLP(width, m.experts, 0, m.top, 1, 1, 1.0, m.ff, act=hip_ops.clamped_glu(m.limit), sigmoid=True,
                                  corrected=False, raw_weights=True, weigh_inputs=True))
            self.hc2, self.norm2 = HyperConnection(config.streams), padded_parameter(w)


class SemezenForCausalLM(nn.Module):
    def __init__(self, config) -> None:
        super().__init__()
        if get_tensor_parallel_world_size() > 1:
            raise ValueError("Semezen runs on one GPU: its experts and recurrences are not sharded")
        self.config = config
        w = pad_to(config.hidden_size)
        self.embed = padded_parameter(config.vocab_size, w)
        self.stack = []
        for i in range(len(config.layers)):
            layer = SemezenLayer(config, i)
            self.add_module(f"l{i}", layer)
            self.stack.append(layer)
        self.final_norm = padded_parameter(w)
        self.head = ParallelLMHead(config.vocab_size, config.hidden_size, storage_dim=w)

    def forward(self, input_ids, positions):
        ids, positions, c = input_ids.contiguous(), positions.contiguous(), self.config
        x = ResidualStreams(c.streams, ids, self.embed, c.norm_eps, c.hidden_size)
        mixer_input = lambda layer: {"norm_w": layer.norm1, "read": layer.hc1.read, "shift": layer.shift.rows(positions)}
        h = x.start(**mixer_input(self.stack[0]))
        for layer, after in zip(self.stack, self.stack[1:] + [None]):
            last = after is None
            then = {"norm_w": self.final_norm, "last": True} if last else mixer_input(after)
            y = layer.mix(h, positions)
            if layer.mlp is None:
                h = x.add(y, layer.hc1, **then)
                continue
            h = x.add(y, layer.hc1, layer.norm2, layer.hc2.read)
            y, experts = layer.mlp(h)
            h = x.add(y, layer.hc2, experts=experts, **then)
        return h

    def compute_logits(self, hidden_states, gather: bool = True):
        return self.head(hidden_states, gather=gather)

    # ---- weights ------------------------------------------------------------------------------------------------------
    @property
    def packed_modules_mapping(self) -> dict:
        """Checkpoint name fragment -> (parameter, segment); the first fragment that a name contains wins."""
        out = {"final.norm": ("final_norm", None), ".shift": (".shift.share", None)}
        for q in "12":
            out.update({f".hc{q}.in": (f".hc{q}.read", None), f".hc{q}.out": (f".hc{q}.write", None)})
        out.update({f".mix.{n}.b": (".mix.in_proj.bias", n) for n in "qkzx"})
        out.update({f".mix.{n}": (".mix.in_proj.weight", n) for n in "qkgzx"})
        out.update({".mix.o": (".mix.o.weight", "o"), ".mlp.up": (".mlp.up.weight", "up"), ".mlp.down": (".mlp.down.weight", "down")})
        for e in range(max((getattr(s.mlp, "experts", 0) for s in self.config.layers), default=0)):
            out.update({f".mlp.e{e}.{n}": (".mlp.down" if n == "down" else ".mlp.gate_up", (e, n)) for n in ("gate", "up", "down")})
        out["head"] = ("head.weight", None)
        return out

    def check_loaded(self, names) -> None:
        """Every tensor of the configuration, and no other, must have found its place."""
        want = set(self.config.weight_shapes())
        if set(names) != want:
            raise ValueError(f"checkpoint does not fit the configuration: missing or unusable {sorted(want - set(names))[:8]}, "
                             f"unexpected {sorted(set(names) - want)[:8]}")

    def load_weights(self, weights) -> None:
        mapping = self.packed_modules_mapping
        self.check_loaded([n for n, t in weights.items() if load_weight(self, n, t, mapping)])

    def dummy_weights(self, gen) -> dict:
        """Random checkpoint tensors of unit gain (norm weights neutral, streams read evenly and kept apart, gates of all speeds)."""
        out, dev, n = {}, self.embed.device, self.config.streams
        for name, shape in self.config.weight_shapes().items():
            last = name.rsplit(".", 1)[-1]
            t = torch.empty(shape, device=dev, dtype=torch.float32).normal_(0.0, 1.0, generator=gen)
            if last.startswith("norm") or last == "out":
                t.fill_(1.0)
            elif last == "in":
                t.fill_(1.0 / n)
            elif name.endswith((".hc1.mix", ".hc2.mix")):
                t.copy_(torch.eye(n))
            elif last == "shift":
                t.mul_(0.2).add_(0.5)
            elif last == "b":
                t.sub_(2.0) if name.endswith(".z.b") else t.zero_()
            elif len(shape) == 2 and name != "embed":
                t /= shape[-1] ** 0.5
            out[name] = t.to(self.embed.dtype)
        return out
