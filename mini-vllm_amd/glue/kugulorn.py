"""Kugulorn decoder glue: an fp32 residual stream through layers of one or two sublayers, each normed on both sides and scaled.

    mixer (latent attention or state space)  ->  x += mult * scale1 * rms(y) w1b;  h = rms(x) w2        (one launch)
    [gate | up] GEMM with the clamped gate (decode: ONE launch) -> down GEMM
                                             ->  x += mult * scale2 * rms(y) w2b;  h = next layer's norm (one launch)"""
from __future__ import annotations

import torch
from torch import nn

from .. import hip_ops
from ..layers import LatentAttention, Mamba2, ParallelLMHead, Segment, SegmentedLinear, padded_parameter
from ..layers.linear import gated_linear, pad_to
from ..utils.loader import load_weight

__all__ = ["KugulornLayer", "KugulornForCausalLM"]


class ClampedMLP(nn.Module):
    def __init__(self, width: int, ff: int, limit: float) -> None:
        super().__init__()
        self.gate_up = SegmentedLinear(width, [Segment("gate", ff), Segment("up", ff)], split="out")
        self.down = SegmentedLinear(width, [Segment("down", ff)], split="in")
        self.act = hip_ops.clamped_glu(limit)

    def forward(self, h):
        return self.down(gated_linear(h, self.gate_up, self.act), partial_ok=True)


class KugulornLayer(nn.Module):
    def __init__(self, config, index: int, before: list) -> None:
        super().__init__()
        spec, width, eps = config.layers[index], config.hidden_size, config.norm_eps
        m, w = spec.mixer, pad_to(width)
        self.recurrent = spec.type == "mamba2"
        if self.recurrent:
            self.mix = Mamba2(width, m.heads, m.vdim, m.state, m.groups, m.taps, m.norm_groups, eps)
        else:
            self.mix = LatentAttention(width, m.heads, m.dim, m.rot_dim, m.vdim, m.q_rank, m.kv_rank, m.rot_base, m.scale,
                                       m.window, eps, config.max_position_embeddings or 4096,
                                       None if m.kv_from is None else before[m.kv_from].mix)
        self.norm1, self.norm1b, self.ls1 = (padded_parameter(w) for _ in range(3))
        self.mlp = None
        if spec.mlp is not None:
            self.mlp = ClampedMLP(width, spec.mlp.ff, spec.mlp.limit)
            self.norm2, self.norm2b, self.ls2 = (padded_parameter(w) for _ in range(3))


class KugulornForCausalLM(nn.Module):
    # checkpoint name fragment -> (parameter, segment(s)); the first fragment that a name contains wins
    packed_modules_mapping = {
        ".mix.dq.norm": (".mix.q_norm", None), ".mix.dkv.norm": (".mix.kv_norm", None), ".mix.dq": (".mix.down.weight", "dq"),
        ".mix.dkv": (".mix.down.weight", ("latent", "rot")), ".mix.uq": (".mix.uq.weight", "uq"),
        ".mix.uk": (".mix.ukv.weight", "uk"), ".mix.uv": (".mix.ukv.weight", "uv"), ".mix.o": (".mix.o.weight", "o"),
        ".mix.in": (".mix.in_proj.weight", ("z", "x", "b", "c", "dt")), ".mix.conv.b": (".mix.conv_b", None),
        ".mlp.gate": (".mlp.gate_up.weight", "gate"), ".mlp.up": (".mlp.gate_up.weight", "up"),
        ".mlp.down": (".mlp.down.weight", "down"), "final.norm": ("final_norm", None), "head": ("head.weight", None)}

    def __init__(self, config) -> None:
        super().__init__()
        self.config = config
        w = pad_to(config.hidden_size)
        self.embed = padded_parameter(config.vocab_size, w)
        self.stack = []
        for i in range(len(config.layers)):
            layer = KugulornLayer(config, i, self.stack)
            self.add_module(f"l{i}", layer)
            self.stack.append(layer)
        self.final_norm = padded_parameter(w)
        self.head = ParallelLMHead(config.vocab_size, config.hidden_size, storage_dim=w)

    def _add(self, x, y, norm_b, scale, next_norm):
        c = self.config
        return hip_ops.residual_update(x, y=getattr(y, "data", y), y_norm_w=norm_b, y_scale=scale, y_mult=c.residual_mult,
                                       norm_w=next_norm, eps=c.norm_eps, cols_true=c.hidden_size)

    def forward(self, input_ids, positions):
        c, ids = self.config, input_ids.contiguous()
        x = torch.empty((ids.shape[0], self.embed.shape[1]), dtype=torch.float32, device=ids.device)
        h = hip_ops.residual_update(x, embed=self.embed, ids=ids, start=True, norm_w=self.stack[0].norm1, eps=c.norm_eps,
                                    cols_true=c.hidden_size)
        for i, layer in enumerate(self.stack):
            after = self.stack[i + 1].norm1 if i + 1 < len(self.stack) else self.final_norm
            y = layer.mix(h) if layer.recurrent else layer.mix(h, positions)
            h = self._add(x, y, layer.norm1b, layer.ls1, after if layer.mlp is None else layer.norm2)
            if layer.mlp is not None:
                h = self._add(x, layer.mlp(h), layer.norm2b, layer.ls2, after)
        for layer in self.stack:
            if not layer.recurrent and layer.mix.owner is layer.mix:
                layer.mix._rows = None      # the step's rows
        return h

    def compute_logits(self, hidden_states, gather: bool = True):
        return self.head(hidden_states, gather=gather)

    # ---- weights ------------------------------------------------------------------------------------------------------
    def check_loaded(self, names) -> None:
        """Every tensor of the configuration, and no other, must have found its place."""
        want = set(self.config.weight_shapes())
        if set(names) != want:
            raise ValueError(f"checkpoint does not fit the configuration: missing or unusable {sorted(want - set(names))[:8]}, "
                             f"unexpected {sorted(set(names) - want)[:8]}")

    def load_weights(self, weights) -> None:
        self.check_loaded([n for n, t in weights.items() if load_weight(self, n, t, self.packed_modules_mapping)])

    def dummy_weights(self, gen) -> dict:
        """Random checkpoint tensors of unit gain (norm weights and scales neutral, decays of all speeds)."""
        out, dev = {}, self.embed.device
        for name, shape in self.config.weight_shapes().items():
            last = name.rsplit(".", 1)[-1]
            t = torch.empty(shape, device=dev, dtype=torch.float32).normal_(0.0, 1.0, generator=gen)
            if last.startswith("norm") or last in ("ls1", "ls2", "D"):
                t.fill_(1.0)
            elif last == "dt_bias":
                t.sub_(3.0)
            elif last == "b":
                t.zero_()
            elif len(shape) == 2 and name != "embed":
                t /= shape[-1] ** 0.5
            out[name] = t.to(self.embed.dtype)
        return out
