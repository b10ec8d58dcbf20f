"""A table row per (previous token, token), added to the token embedding where the residual stream starts (csrc/residual.hip).  The
token before a step's first lives in the sequence's state slot (engine/state_slots.py)."""
from __future__ import annotations

import torch
from torch import nn

from .. import hip_ops
from ..utils.context import get_context
from .latent_attention import padded_parameter

__all__ = ["PairEmbedding"]


class PairEmbedding(nn.Module):
    def __init__(self, buckets: int, mul_prev: int, mul_cur: int, storage_dim: int) -> None:
        super().__init__()
        self.muls = (mul_prev, mul_cur)
        self.weight = padded_parameter(buckets + 1, storage_dim)
        self.prev_tokens: torch.Tensor = torch.tensor([])     # int32 [2, slots], assigned by the executor

    def state_shapes(self, dtype) -> dict:
        """Attribute -> (shape of one slot, dtype); the executor assigns [2, slots, *shape] tensors."""
        return {"prev_tokens": ((), torch.int32)}

    def rows(self, positions) -> hip_ops.PairTable:
        """This step's argument of ``hip_ops.residual_update``."""
        ctx = get_context()
        return hip_ops.PairTable(self.weight.data, *self.muls, positions, self.prev_tokens, ctx.state_slots,
                                 ctx.cum_seqlens_q if ctx.is_prefill else None)
