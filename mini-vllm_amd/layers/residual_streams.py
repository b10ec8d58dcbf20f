"""Several residual streams with learned reads, writes and mixes (hyper-connections), and the blend of a normed row with the one of the
token before (token shift); both on csrc/streams.hip, where one launch does all that lies between two sublayers."""
from __future__ import annotations

import torch
from torch import nn

from .. import hip_ops
from ..utils.context import get_context
from .latent_attention import padded_parameter

__all__ = ["HyperConnection", "ResidualStreams", "TokenShift"]


class HyperConnection(nn.Module):
    """How a sublayer reads the streams (a weight each) and writes them (mix [from, to], a weight each for its output)."""

    def __init__(self, streams: int) -> None:
        super().__init__()
        self.read, self.write = padded_parameter(streams), padded_parameter(streams)
        self.mix = padded_parameter(streams, streams)


class TokenShift(nn.Module):
    """h + (h of the token before - h) * share; the last h of a sequence is kept in its slot (engine/state_slots.py), in fp32."""

    def __init__(self, cols: int) -> None:
        super().__init__()
        self.share = padded_parameter(cols)
        self.prev: torch.Tensor = torch.tensor([])           # fp32 [2, slots, cols], assigned by the executor

    def state_shapes(self, dtype) -> dict:
        """Attribute -> (shape of one slot, dtype); the executor assigns [2, slots, *shape] tensors."""
        return {"prev": ((self.share.numel(),), torch.float32)}

    def rows(self, positions) -> hip_ops.StreamShift:
        """This step's argument of ``hip_ops.stream_update``."""
        ctx = get_context()
        return hip_ops.StreamShift(self.share.data, self.prev, positions, ctx.state_slots, ctx.cum_seqlens_q if ctx.is_prefill else None)


class ResidualStreams:
    """The streams of one step, in two buffers that take turns."""

    def __init__(self, streams: int, ids, embed, eps: float, cols_true: int) -> None:
        self.streams, self.eps, self.cols_true = streams, eps, cols_true
        shape = (ids.shape[0], streams, embed.shape[1])
        self.now, self.spare = (torch.empty(shape, dtype=torch.float32, device=ids.device) for _ in range(2))
        self.ids, self.embed = ids, embed

    def start(self, norm_w, read=None, shift=None):
        """Every stream starts from the embedding; -> what the first sublayer reads."""
        return hip_ops.stream_update(self.streams, norm_w, self.eps, embed=self.embed, ids=self.ids, x_out=self.now, in_w=read,
                                     shift=shift, cols_true=self.cols_true)

    def add(self, y, written: HyperConnection, norm_w, read=None, shift=None, experts=None, last: bool = False):
        """A sublayer's output goes through its connection; -> what the next one reads (``read`` None: the sum of the streams)."""
        h = hip_ops.stream_update(self.streams, norm_w, self.eps, x=self.now, x_out=None if last else self.spare, y=getattr(y, "data", y),
                                  mix=written.mix, out_w=written.write, in_w=read, experts=experts, shift=shift, cols_true=self.cols_true)
        if not last:
            self.now, self.spare = self.spare, self.now
        return h
