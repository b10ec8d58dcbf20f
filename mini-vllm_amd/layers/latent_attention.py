"""Latent attention over the paged cache: a token's keys and values are one cached row [latent | rotated part] that every head
reads through up-projections of its own (csrc/latent*.hip).

    down projection [query latent | latent | rotated part] -> norms, rotation, cache store      (one launch)
    query up projection -> per head [plain | part to rotate]
    decode rows: plain part through W_uk^T into the latent's coordinates, attention over the cached rows themselves (their
                 latents are the values), per head W_uv behind it
    prompts:     keys and values expanded from the rows ([W_uk ; W_uv], one product), attention per head
A layer may read another layer's rows (``source``): it then has no latent of its own and owns no cache plane.

Sizes between the kernels' are zero-padded in the weights at load time."""
from __future__ import annotations

import torch
import torch.nn.functional as F
from torch import nn

from .. import hip_ops
from ..parallel_state import divide, get_tensor_parallel_world_size
from ..utils.context import get_context
from ..utils.loader import materialize
from .linear import Segment, SegmentedLinear, pad_to
from .rotary_embedding import get_rope

__all__ = ["LatentAttention", "padded_parameter"]

KERNEL_DIMS = (64, 128, 192, 256)   # head dims of the prefill kernel


def _kernel_dim(n: int) -> int:
    return next((d for d in KERNEL_DIMS if n <= d), pad_to(n, 64))


def padded_parameter(*shape: int) -> nn.Parameter:
    """Zeros; a checkpoint tensor of the same rank fills the leading corner."""
    p = nn.Parameter(torch.zeros(*shape))

    def load(param, tensor, *args, **kwargs):
        t = materialize(tensor)
        if t.dim() != param.dim() or any(a > b for a, b in zip(t.shape, param.shape)):
            raise ValueError(f"cannot place {tuple(t.shape)} in {tuple(param.shape)}")
        param.data[tuple(slice(0, n) for n in t.shape)].copy_(t)

    p.weight_loader = load
    return p


class LatentAttention(nn.Module):
    def __init__(self, width: int, heads: int, dim: int, rot_dim: int, vdim: int, q_rank: int, kv_rank: int, rot_base: float,
                 scale: float, window: int = 0, eps: float = 1e-6, max_positions: int = 4096,
                 source: "LatentAttention | None" = None) -> None:
        super().__init__()
        self.heads = divide(heads, get_tensor_parallel_world_size())
        self.scale, self.window, self.eps = float(scale), int(window), float(eps)
        self.q_rank, self.kv_rank, self.rot_dim = q_rank, kv_rank, rot_dim
        self.plain, self.rot_cols, self.kv_cols = pad_to(dim, 32), pad_to(rot_dim, 32), pad_to(kv_rank)
        self.dq, self.dv = _kernel_dim(self.plain + self.rot_cols), _kernel_dim(vdim)
        self._source = (source,)        # (a tuple: the other layer's parameters are not this layer's)
        rows = [Segment("dq", q_rank)]
        if source is None:
            rows += [Segment("latent", kv_rank), Segment("rot", rot_dim)]
            self.kv_norm = padded_parameter(self.kv_cols)
            self.latent_cache: torch.Tensor = torch.tensor([])    # [blocks, block_size, row_cols], assigned by the executor
            # how far back the layers that read this cache look (0: to the start): the span of keys that a portion of a
            # prompt gathers
            self.span_window = self.window
            self._rows = None           # this step's rows: whole prompts' own, or gathered
        else:
            if (source.kv_rank, source.rot_dim) != (kv_rank, rot_dim):
                raise ValueError("a layer that reads another layer's latents must have its latent and rotated sizes")
            source.span_window = 0 if 0 in (source.span_window, self.window) else max(source.span_window, self.window)
        self.down = SegmentedLinear(width, rows, split="none")
        self.q_norm = padded_parameter(pad_to(q_rank))
        self.uq = SegmentedLinear(q_rank, [Segment("uq", heads, dim + rot_dim, self.dq, ((dim, 0), (rot_dim, self.plain)))], "out")
        self.ukv = SegmentedLinear(kv_rank, [Segment("uk", heads, dim, self.plain), Segment("uv", heads, vdim, self.dv)], "out")
        self.o = SegmentedLinear(width, [Segment("o", heads, vdim, self.dv)], split="in")
        self.rotary = get_rope(rot_dim, rot_dim, max_positions, rot_base, interleaved=True)
        self.uk_t = self.uv = None

    @property
    def owner(self) -> "LatentAttention":
        return self._source[0] if self._source[0] is not None else self

    @property
    def row_cols(self) -> int:
        return self.kv_cols + self.rot_cols

    def extra_repr(self) -> str:
        return (f"heads={self.heads}, row={self.kv_rank}+{self.rot_dim}, scale={self.scale}, window={self.window}, "
                f"shares={self._source[0] is not None}")

    def finish_weights(self) -> None:
        """Per-head forms of the up-projections for decode steps: W_uk transposed, W_uv as it lies."""
        h, w, at = self.heads, self.ukv.weight.data, self.ukv.offsets["uv"]
        self.uk_t = w[:h * self.plain].view(h, self.plain, self.kv_cols).transpose(1, 2).contiguous()
        self.uv = w[at:at + h * self.dv].view(h, self.dv, self.kv_cols)

    def _keys(self, ctx):
        """(rows, cumulative lengths, longest) of the keys of this step's prompts, from the cache of the owner."""
        own = self.owner
        cu, start, total, longest = ctx.key_spans[own.span_window]
        if own._rows is None:
            own._rows = hip_ops.latent_gather(own.latent_cache, ctx.block_tables[ctx.decode_rows:], cu, start, total, longest)
        return own._rows, cu, longest

    def forward(self, h, positions):
        ctx, own, t = get_context(), self.owner, h.shape[0]
        has_cache = own.latent_cache.numel() > 0
        if not ctx.is_prefill and (not has_cache or ctx.context_lens is None or ctx.block_tables is None):
            raise RuntimeError("decode step without a latent cache, context lengths or block tables")
        cos, sin = self.rotary._tables(h.device)
        gathered = ctx.is_prefill and ctx.prefix_cached and has_cache and ctx.block_tables is not None
        z = self.down(h)
        kv = None
        if own is self:
            self._rows = None
            kv = (self.kv_norm, self.down.offsets["latent"], self.kv_rank, self.down.offsets["rot"], self.rot_dim, self.rot_cols)
        c_q, rows = hip_ops.latent_prep(z, self.q_norm, 0, self.q_rank, self.eps, kv, positions, cos, sin,
                                        own.latent_cache if has_cache else None, ctx.slot_mapping,
                                        want_rows=ctx.is_prefill and not gathered)
        if rows is not None:
            own._rows = rows
        q = self.uq(c_q)[:, :self.heads * self.dq].view(t, self.heads, self.dq)
        out = torch.empty((t, self.heads, self.dv), dtype=h.dtype, device=h.device)
        nd = (ctx.decode_rows if gathered else 0) if ctx.is_prefill else t
        if nd:
            qa = torch.empty((nd, self.heads, self.row_cols), dtype=h.dtype, device=h.device)
            hip_ops.head_linear(q[:nd], self.uk_t, qa, (self.rot_dim, self.rot_cols, positions[:nd], cos, sin))
            lat = hip_ops.latent_decode(qa, own.latent_cache, ctx.block_tables[:nd], ctx.context_lens[:nd], self.kv_cols,
                                        self.scale, self.window)
            hip_ops.head_linear(lat, self.uv, out[:nd])
        if nd < t:
            if gathered:
                rows, cu_k, max_k = self._keys(ctx)
                cu_q, max_q = ((ctx.rest_cum_seqlens_q, ctx.rest_max_seqlen_q) if ctx.decode_rows else
                               (ctx.cum_seqlens_q, ctx.max_seqlen_q))
            else:
                rows, cu_q, max_q = own._rows, ctx.cum_seqlens_q, ctx.max_seqlen_q
                cu_k, max_k = cu_q, max_q
            at = self.ukv.offsets["uv"]
            kvx = F.linear(rows[:, :self.kv_cols], self.ukv.weight)
            hip_ops.latent_prefill(q[nd:], kvx[:, :self.heads * self.plain].unflatten(1, (self.heads, self.plain)),
                                   kvx[:, at:at + self.heads * self.dv].unflatten(1, (self.heads, self.dv)),
                                   rows[:, self.kv_cols:], cu_q, cu_k, max_q, max_k, positions[nd:], cos, sin, self.rot_dim,
                                   self.scale, self.window, out=out[nd:])
        return self.o(out.view(t, self.heads * self.dv), partial_ok=True)
