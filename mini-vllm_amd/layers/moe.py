"""Mixture of experts on the gfx950 kernels of csrc/moe.hip.

    router: fp32 logits, scores, choice by groups with a correction, weights           (one launch)
    pairs (token, choice) sorted by expert                                             (one launch)
    per expert [gate | up] with the activation, then down                              (one launch each)
The weighted sum over a token's choices (identity experts: the token's own input) is left to the residual update behind the layer;
where the weight multiplies the expert's input instead, it multiplies the sums of [gate | up], ahead of the activation.
Expert weights are kept in ONE form: as the checkpoint has them in fp32, fragment-ordered in 16 bits (``finish_weights``)."""
from __future__ import annotations

import torch
from torch import nn

from .. import hip_ops
from ..utils.loader import materialize
from .latent_attention import padded_parameter
from .linear import Segment, SegmentedLinear, gated_linear, pad_to

__all__ = ["ExpertMLP"]

# pairs per expert up to which a launch works on tiles of that many rows
TILES = ((8, 16), (40, 32), (96, 64), (768, 128))


class ExpertMLP(nn.Module):
    def __init__(self, width: int, experts: int, identity: int, top: int, groups: int, keep: int, scale: float, ff: int,
                 shared_ff: int = 0, act: hip_ops.GateAct | None = None, sigmoid: bool = False, corrected: bool = True,
                 raw_weights: bool = False, weigh_inputs: bool = False) -> None:
        """``sigmoid``: scores are sigmoids of the logits, not a softmax; ``corrected``: a number per output joins the scores in the
        choice; ``raw_weights``: the weights are the chosen scores, not divided by their sum; ``weigh_inputs``: they multiply the
        experts' inputs, not their outputs."""
        super().__init__()
        if weigh_inputs and identity:
            raise ValueError("identity experts have no product that could weigh its input")
        self.sigmoid, self.raw_weights, self.weigh_inputs = sigmoid, raw_weights, weigh_inputs
        self.experts, self.top, self.groups, self.keep, self.scale = experts, top, groups, keep, float(scale)
        self.act = act or hip_ops.GateAct(0, 0.0, 0.0)     # silu
        w, f = pad_to(width), pad_to(ff)
        self.w, self.f, self.width, self.ff = w, f, width, ff
        self.router = padded_parameter(experts + identity, w)
        self.correction = padded_parameter(experts + identity) if corrected else None
        self.gate_up, self.down = nn.Parameter(torch.zeros(experts, 2, f, w)), nn.Parameter(torch.zeros(experts, w, f))
        self.gate_up.weight_loader = self.down.weight_loader = self._load
        self.packed = False
        self.shared_gate_up = self.shared_down = None
        if shared_ff:
            self.shared_gate_up = SegmentedLinear(width, [Segment("gate", shared_ff), Segment("up", shared_ff)], split="out")
            self.shared_down = SegmentedLinear(width, [Segment("down", shared_ff)], split="in")

    def extra_repr(self) -> str:
        return f"experts={self.experts}, outputs={self.router.shape[0]}, top={self.top}, groups={self.keep} of {self.groups}, ff={self.ff}"

    def _load(self, param, tensor, shard=None, *args, **kwargs):
        """shard: (expert, "gate" | "up" | "down")."""
        e, what = shard
        t, want = materialize(tensor), (self.width, self.ff) if what == "down" else (self.ff, self.width)
        if tuple(t.shape) != want:
            raise ValueError(f"expert {e} {what}: expected {want}, got {tuple(t.shape)}")
        dst = param.data[e] if what == "down" else param.data[e, int(what == "up")]
        dst[:want[0], :want[1]].copy_(t)

    def finish_weights(self) -> None:
        """The form that the kernels read, in place of the loaded one."""
        if self.router.dtype != torch.float32 and not self.packed:
            for p in (self.gate_up, self.down):
                p.data = hip_ops.pack_weight(p.data.view(-1, p.shape[-1]))
            self.packed = True

    def tile_rows(self, tokens: int) -> int:
        if self.router.dtype == torch.float32:
            return 16
        per = tokens * self.top / self.experts
        return next((rows for most, rows in TILES if per <= most), 256)

    def route(self, h):
        """-> (weights [T, top], the pairs sorted by expert)."""
        ids, weights = hip_ops.moe_route(h, self.router, self.correction, self.top, self.groups, self.keep, self.scale, self.sigmoid,
                                         self.raw_weights)
        return weights, hip_ops.moe_group(ids, self.experts, self.tile_rows(h.shape[0]), weights if self.weigh_inputs else None)

    def forward(self, h):
        """-> (shared expert's output or None, the routed experts' part for ``hip_ops.residual_update``)."""
        weights, g = self.route(h)
        z = hip_ops.moe_linear(h, self.gate_up, self.f, g, self.act, gather=True, experts=self.experts, in_scale=g.weights)
        y = hip_ops.moe_linear(z, self.down, self.w, g, experts=self.experts)
        shared = None
        if self.shared_gate_up is not None:
            shared = self.shared_down(gated_linear(h, self.shared_gate_up, "silu"), partial_ok=True)
        return shared, (y, g.place, None if self.weigh_inputs else weights)
