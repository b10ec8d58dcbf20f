"""Selective state space layer (Mamba-2) on the gfx950 kernels of csrc/ssm*.hip.

    input projection [gate z | x | b | c | step size]
    prompts: causal convolution + silu of [x | b | c], then the recurrence in chunks
    decode:  both in one launch per step, the fp32 state streamed through once
    gate, norm in equal parts, output projection
A sequence's state (recurrent fp32 state, last inputs of the convolution) lives in a slot of its own (engine/state_slots.py);
the pools are allocated by the executor from ``state_shapes``.  Column and state sizes between the kernels' are zero-padded."""
from __future__ import annotations

import torch
from torch import nn

from .. import hip_ops
from ..parallel_state import divide, get_tensor_parallel_world_size
from ..utils.context import get_context
from ..utils.loader import materialize
from .linear import Segment, SegmentedLinear, pad_to

__all__ = ["Mamba2"]


class Mamba2(nn.Module):
    def __init__(self, width: int, heads: int, vdim: int, state: int, groups: int, taps: int, norm_groups: int,
                 eps: float = 1e-6) -> None:
        super().__init__()
        tp = get_tensor_parallel_world_size()
        self.heads, self.groups, self.norm_groups = divide(heads, tp), divide(groups, tp), divide(norm_groups, tp)
        self.vdim, self.taps, self.eps = vdim, taps, float(eps)
        self.p, self.n = pad_to(vdim, 16), pad_to(state, 32)
        self.in_proj = SegmentedLinear(width, [
            Segment("z", heads, vdim, self.p), Segment("x", heads, vdim, self.p), Segment("b", groups, state, self.n),
            Segment("c", groups, state, self.n), Segment("dt", heads)], "out")
        at = self.in_proj.offsets
        self.x_off, self.dt_off = at["x"], at["dt"]
        b_off, c_off = at["b"] - at["x"], at["c"] - at["x"]
        self.channels = c_off + self.groups * self.n
        self.shape = (self.heads, self.groups, self.p, self.n, b_off, c_off)
        # (checkpoint channels, units, unit, stored, offset) of the convolved channels
        conv = [(heads, vdim, self.p, 0), (groups, state, self.n, b_off), (groups, state, self.n, c_off)]
        self.conv = self._vector((taps, self.channels), conv, taps)      # [taps, channels]: the checkpoint's, transposed
        self.conv_b = self._vector((self.channels,), conv)
        self.dt_bias, self.A_log, self.D = (self._vector((self.heads,), [(heads, 1, 1, 0)]) for _ in range(3))
        self.norm = self._vector((self.heads * self.p,), [(heads, vdim, self.p, 0)])
        self.o = SegmentedLinear(width, [Segment("o", heads, vdim, self.p)], split="in")
        self.conv_state: torch.Tensor = torch.tensor([])    # [2, slots, taps - 1, channels], assigned by the executor
        self.ssm_state: torch.Tensor = torch.tensor([])     # fp32 [2, slots, heads, n, p]

    def _vector(self, shape, runs, taps: int = 0) -> nn.Parameter:
        """Zeros; a checkpoint tensor [sum of units * unit (, taps)] goes to its runs (units, unit, stored, offset) along the
        last dim, a rank's units only."""
        p, tp = nn.Parameter(torch.zeros(*shape)), get_tensor_parallel_world_size()
        rank = self._rank()

        def load(param, tensor, *args, **kwargs):
            t = materialize(tensor)
            want = (sum(u * n for u, n, _, _ in runs),) + ((taps,) if taps else ())
            if tuple(t.shape) != want:
                raise ValueError(f"expected {want}, got {tuple(t.shape)}")
            at = 0
            for units, unit, stored, off in runs:
                mine = units // tp
                piece = t[at + rank * mine * unit:at + (rank + 1) * mine * unit]
                piece = piece.t().unflatten(1, (mine, unit)) if taps else piece.unflatten(0, (mine, unit))
                dst = param.data[..., off:off + mine * stored].unflatten(-1, (mine, stored))
                dst[..., :unit].copy_(piece)
                at += units * unit

        p.weight_loader = load
        return p

    @staticmethod
    def _rank() -> int:
        from ..parallel_state import get_tensor_parallel_rank

        return get_tensor_parallel_rank() if get_tensor_parallel_world_size() > 1 else 0

    def state_shapes(self, dtype) -> dict:
        """Attribute -> (shape of one slot, dtype); the executor assigns [2, slots, *shape] tensors."""
        return {"conv_state": ((self.taps - 1, self.channels), dtype), "ssm_state": ((self.heads, self.n, self.p), torch.float32)}

    def extra_repr(self) -> str:
        return f"heads={self.heads}, vdim={self.vdim}, state={self.n}, groups={self.groups}, taps={self.taps}"

    def forward(self, h):
        ctx, t = get_context(), h.shape[0]
        z = self.in_proj(h)
        x, dt = z[:, self.x_off:self.x_off + self.channels], z[:, self.dt_off:self.dt_off + self.heads]
        y = torch.empty((t, self.heads * self.p), dtype=h.dtype, device=h.device)
        slots = ctx.state_slots
        nd = ctx.decode_rows if ctx.is_prefill else t
        if nd:
            hip_ops.ssm_step(x[:nd], dt[:nd], self.conv, self.conv_b, self.dt_bias, self.A_log, self.D, self.shape,
                             self.conv_state, self.ssm_state, slots[:nd], ctx.context_lens[:nd], out=y[:nd])
        if nd < t:
            cu_q, cu_k, max_q = ((ctx.rest_cum_seqlens_q, ctx.rest_cum_seqlens_k, ctx.rest_max_seqlen_q) if nd else
                                 (ctx.cum_seqlens_q, ctx.cum_seqlens_k, ctx.max_seqlen_q))
            xc = hip_ops.causal_conv(x[nd:], self.conv, self.conv_b, self.shape, self.conv_state, slots[nd:], cu_q, cu_k, max_q)
            hip_ops.ssm_prefill(xc, dt[nd:], self.dt_bias, self.A_log, self.D, self.shape, self.ssm_state, slots[nd:], cu_q, cu_k,
                                max_q, out=y[nd:])
        g = hip_ops.gated_group_norm(y, z, self.norm, self.heads, self.p, self.vdim, self.norm_groups, self.eps,
                                     self.o.weight.shape[1])
        return self.o(g, partial_ok=True)
