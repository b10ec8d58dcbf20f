"""Gated delta rule on the gfx950 kernels of csrc/delta*.hip: per head a state S of key channels x columns,
    S' = g S_old,   u = beta (v - k S'),   S_new = S' + (k outer u),   o = q S_new     (rows; k and q of length 1; fp32 throughout)
then o's RMS norm per head, a weight shared by the heads, and a gate.

    prompts: causal convolution + silu of [v | k | q], the recurrence in chunks, norm and gate
    decode:  all of it in one launch per step, the fp32 state streamed through once
The module owns what lies between the projections; the layer around it merges ``segments`` into its input projection (they read the
same input as whatever stands beside the rule) and projects the output.  A sequence's state (S, last inputs of the convolution) lives
in a slot of its own (engine/state_slots.py).  Column and key sizes between the kernels' are zero-padded."""
from __future__ import annotations

import torch
from torch import nn

from .. import hip_ops
from ..utils.context import get_context
from ..utils.loader import materialize
from .latent_attention import padded_parameter
from .linear import BlockLinear, Segment, pad_to

__all__ = ["GatedDeltaRule"]


class GatedDeltaRule(nn.Module):
    def __init__(self, heads: int, kv_heads: int, dim: int, vdim: int, taps: int, eps: float, gate: str = "silu",
                 ranks: tuple[int, int] | None = None, out_scale: float = 1.0, prefix: str = "", unit_eps: float = 1e-6) -> None:
        """``ranks``: of the projections of a decay per key channel and of the gate; None: a decay per head, a full gate."""
        super().__init__()
        self.heads, self.taps, self.gate, self.out_scale, self.prefix, self.ranks = heads, taps, gate, float(out_scale), prefix, ranks
        p, n = pad_to(vdim, 16), pad_to(dim, 32)
        self.segments = [Segment(prefix + "v", heads, vdim, p), Segment(prefix + "k", kv_heads, dim, n),
                         Segment(prefix + "q", kv_heads, dim, n), Segment(prefix + "b", heads)]
        if ranks:
            self.segments += [Segment(prefix + "a1", ranks[0]), Segment(prefix + "g1", ranks[1])]
            self.lift = BlockLinear([(ranks[0], Segment("a2", heads, dim, n)), (ranks[1], Segment("g2", heads, vdim, p))])
        else:
            self.segments += [Segment(prefix + "a", heads), Segment(prefix + "g", heads, vdim, p)]
            self.lift = None
        at, off = {}, 0
        for s in self.segments:
            at[s.name[len(prefix):]], off = off, off + s.local(1)
        self.at, self.columns = at, off
        self.shape = hip_ops.DeltaShape(heads, kv_heads, p, n, at["k"], at["q"], vdim, dim ** -0.5, ranks is not None, float(eps),
                                        float(unit_eps))
        self.conv = nn.Parameter(torch.zeros(taps, self.shape.channels))     # the checkpoint's three, transposed
        self._places = {"v": (heads, vdim, p), "k": (kv_heads, dim, n), "q": (kv_heads, dim, n)}
        self.conv.weight_loader = self._load_conv
        self.A_log = padded_parameter(heads)
        self.dt_bias = nn.Parameter(torch.zeros(heads * n if ranks else heads))
        self.dt_bias.weight_loader = lambda param, t, *a, **k: self._spread(param.data, t, heads, dim if ranks else 1, n if ranks else 1)
        self.norm = padded_parameter(p)
        self.conv_state: torch.Tensor = torch.tensor([])     # [2, slots, taps - 1, channels], assigned by the executor
        self.state: torch.Tensor = torch.tensor([])          # fp32 [2, slots, heads, n, p]

    @staticmethod
    def _spread(dst, tensor, units: int, unit: int, stored: int) -> None:
        """tensor [units * unit] -> the leading ``unit`` of every ``stored`` elements of dst's last dim."""
        t = materialize(tensor)
        if tuple(t.shape) != tuple(dst.shape[:-1]) + (units * unit,):
            raise ValueError(f"expected {units * unit} elements, got {tuple(t.shape)}")
        dst.unflatten(-1, (units, stored))[..., :unit].copy_(t.unflatten(-1, (units, unit)))

    def _load_conv(self, param, tensor, which: str | None = None, *args, **kwargs):
        units, unit, stored = self._places[which]
        t = materialize(tensor)
        if tuple(t.shape) != (units * unit, self.taps):
            raise ValueError(f"convolution of {which}: expected {(units * unit, self.taps)}, got {tuple(t.shape)}")
        off = self.at[which]
        self._spread(param.data[:, off:off + units * stored], t.t(), units, unit, stored)

    def state_shapes(self, dtype) -> dict:
        """Attribute -> (shape of one slot, dtype); the executor assigns [2, slots, *shape] tensors."""
        s = self.shape
        return {"conv_state": ((self.taps - 1, s.channels), dtype), "state": ((s.heads, s.n, s.p), torch.float32)}

    def extra_repr(self) -> str:
        s = self.shape
        return f"heads={s.heads}, kv_heads={s.groups}, state={s.n}x{s.p}, taps={self.taps}, channel_decay={s.channel_decay}, gate={self.gate}"

    def forward(self, z, out) -> None:
        """z [T, columns]: the segments' outputs, in order; out [T, heads * p] (rows may be strided)."""
        ctx, t, s, at = get_context(), z.shape[0], self.shape, self.at
        x, beta = z[:, :s.channels], z[:, at["b"]:at["b"] + s.heads]
        if self.lift is not None:
            lifted = self.lift(z[:, at["a1"]:at["a1"] + self.lift.input_size])
            a = lifted[:, :s.heads * s.n]
            gate = lifted[:, self.lift.offsets["g2"]:self.lift.offsets["g2"] + s.heads * s.p]
        else:
            a, gate = z[:, at["a"]:at["a"] + s.heads], z[:, at["g"]:at["g"] + s.heads * s.p]
        slots = ctx.state_slots
        nd = ctx.decode_rows if ctx.is_prefill else t
        if nd:
            hip_ops.delta_step(s, x[:nd], beta[:nd], a[:nd], self.dt_bias, self.A_log, self.conv, self.conv_state, self.state, slots[:nd],
                               ctx.context_lens[:nd], gate[:nd], self.norm, self.gate, self.out_scale, out=out[:nd])
        if nd < t:
            cu_q, cu_k, max_q = ((ctx.rest_cum_seqlens_q, ctx.rest_cum_seqlens_k, ctx.rest_max_seqlen_q) if nd else
                                 (ctx.cum_seqlens_q, ctx.cum_seqlens_k, ctx.max_seqlen_q))
            xc = hip_ops.causal_conv(x[nd:], self.conv, None, s.conv, self.conv_state, slots[nd:], cu_q, cu_k, max_q)
            y = hip_ops.delta_prefill(s, xc, beta[nd:], a[nd:], self.dt_bias, self.A_log, self.state, slots[nd:], cu_q, cu_k, max_q)
            hip_ops.head_norm_gate(y, gate[nd:], self.norm, s.heads, s.p, s.p_true, s.eps, self.gate, self.out_scale, out=out[nd:])
