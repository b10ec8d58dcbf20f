"""Gated running mean (minGRU) on the gfx950 kernels of csrc/gru.hip: element by element S <- (1 - z) S + z c(u), read out as
S silu(g); z, u and g are projections of the current token only, everything behind them is fp32.

    prompts: chunks of the sequence beside each other, then one walk over every chunk
    decode:  one launch per step
A sequence's state lives in a slot of its own (engine/state_slots.py)."""
from __future__ import annotations

import torch
from torch import nn

from .. import hip_ops
from ..utils.context import get_context
from .linear import Segment, SegmentedLinear, pad_to

__all__ = ["MinGRU"]


class MinGRU(nn.Module):
    def __init__(self, width: int, state_width: int) -> None:
        super().__init__()
        self.n = pad_to(state_width)
        self.in_proj = SegmentedLinear(width, [Segment(s, state_width) for s in "zxg"], split="out", bias=True)
        self.o = SegmentedLinear(width, [Segment("o", state_width)], split="in")
        self.state: torch.Tensor = torch.tensor([])          # fp32 [2, slots, n], assigned by the executor

    def state_shapes(self, dtype) -> dict:
        """Attribute -> (shape of one slot, dtype); the executor assigns [2, slots, *shape] tensors."""
        return {"state": ((self.n,), torch.float32)}

    def forward(self, h, positions=None):
        ctx, t, n = get_context(), h.shape[0], self.n
        y, at = self.in_proj(h), self.in_proj.offsets
        z, u, g = (y[:, at[s]:at[s] + n] for s in "zxg")
        out = torch.empty((t, n), dtype=h.dtype, device=h.device)
        slots = ctx.state_slots
        nd = ctx.decode_rows if ctx.is_prefill else t
        if nd:
            hip_ops.gru_step(z[:nd], u[:nd], g[:nd], self.state, slots[:nd], ctx.context_lens[:nd], out[:nd])
        if nd < t:
            cu_q, cu_k, max_q = ((ctx.rest_cum_seqlens_q, ctx.rest_cum_seqlens_k, ctx.rest_max_seqlen_q) if nd else
                                 (ctx.cum_seqlens_q, ctx.cum_seqlens_k, ctx.max_seqlen_q))
            hip_ops.gru_prefill(z[nd:], u[nd:], g[nd:], self.state, slots[nd:], cu_q, cu_k, max_q, out[nd:])
        return self.o(out, partial_ok=True)
