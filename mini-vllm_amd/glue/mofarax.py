"""Mofarax decoder glue.

Attention and feed-forward of a layer read ONE norm and are summed, and the residual stream is fp32, so a layer is
    [q | k] GEMM
    -> rotation + K/V store + attention (decode: ONE launch)           into the left columns of `mixed`
    [gate | up] GEMM with gelu(gate) * up                              into its right columns (decode: ONE launch)
    -> [o | down] GEMM over `mixed`                                    both sublayers summed in the accumulators
    -> residual += that; cast                                          (mv_residual_update)
    -> side gate GEMM -> gelu * token table -> side projection         (decode: the last two in ONE launch)
    -> residual += rms(.) * w [+ embedding + pass vector]; next layer's norm    (mv_residual_update)
Layers of the loop run several times over the same weights; each pass has attention modules (K/V planes) of its own.
Values are the projected keys before rotation: the K plane of the cache holds rotated keys, the V plane the raw ones.
Head dims between the kernels' sizes, and widths that are no multiple of 64, are zero-padded in the weights at load time."""
from __future__ import annotations

import os

import torch
from torch import nn

from .. import hip_ops
from ..layers import Attention, ParallelLMHead, Segment, SegmentedLinear, get_rope, padded_parameter
from ..layers.linear import MID_M_MAX, divide, gated_linear, pad_to
from ..parallel_state import get_tensor_parallel_world_size
from ..utils.context import get_context
from ..utils.loader import load_weight

__all__ = ["MofaraxLayer", "MofaraxForCausalLM", "kernel_head_dim"]

# rows up to which a decode step folds rotation + K/V store into the attention launch (see glue/qwen.py)
ROPE_FOLD_MAX_ROWS = int(os.environ.get("MV_ROPE_FOLD_MAX", "128"))


def kernel_head_dim(dim: int) -> int:
    """Head dim the attention kernels store `dim` at (zero-padded)."""
    for d in (64, 128, 256):
        if dim <= d:
            return d
    raise ValueError(f"head dims above 256 are not supported, got {dim}")


class SideInput(nn.Module):
    """gelu(W_gate x) * e[token], projected back to the stream's width (its RMS norm rides in the residual update)."""

    def __init__(self, width: int, dim: int, offset: int) -> None:
        super().__init__()
        self.dim, self.offset = dim, offset
        self.gate = SegmentedLinear(width, [Segment("gate", dim)], split="none")
        self.proj = SegmentedLinear(dim, [Segment("proj", width)], split="none")
        self.norm = padded_parameter(pad_to(width))

    def forward(self, x, ids, table):
        packed, n = self.proj.weight_packed, self.proj.weight.shape[0]
        # (prefill: the library product and a launch of its own for the lookup were as fast or faster)
        if packed is not None and x.shape[0] <= MID_M_MAX and self.proj.weight.shape[1] <= hip_ops.GATED_LOOKUP_LINEAR_MAX_K:
            return hip_ops.gated_lookup_linear(self.gate(x), table, self.offset, self.dim, ids, packed, n)
        return self.proj(hip_ops.gated_lookup(self.gate(x), table, self.offset, self.dim, ids))


class MofaraxLayer(nn.Module):
    def __init__(self, config, index: int, passes: int) -> None:
        super().__init__()
        spec, tp = config.layers[index], get_tensor_parallel_world_size()
        a, width = spec.attention, config.hidden_size
        self.heads, self.kv_heads, self.ff = divide(a.heads, tp), divide(a.kv_heads, tp), spec.ff
        self.head_dim = d = kernel_head_dim(a.dim)
        self.norm1 = padded_parameter(pad_to(width))
        rows = [Segment("o", a.heads, a.dim, d)]
        self.qk = SegmentedLinear(width, [Segment("q", a.heads, a.dim, d), Segment("k", a.kv_heads, a.dim, d)], split="out")
        if spec.ff:
            self.gate_up = SegmentedLinear(width, [Segment("gate", spec.ff), Segment("up", spec.ff)], split="out")
            rows += [Segment("down", spec.ff)]
        self.proj_out = SegmentedLinear(width, rows, split="in")
        self.rotary = get_rope(d, a.rot_dims, config.max_position_embeddings or 4096, a.rot_base, interleaved=True)
        # one per pass of the loop: the weights are shared, the K/V planes are not
        self.attn = nn.ModuleList(Attention(self.heads, d, a.scale, self.kv_heads, chunk=a.chunk) for _ in range(passes))
        self.side = SideInput(width, config.side_dim, index * config.side_dim) if config.side_dim else None

    def _attend(self, attn: Attention, q, k, positions, out) -> None:
        ctx = get_context()
        has_cache = attn.k_cache.numel() > 0
        cos, sin = self.rotary._tables(q.device)
        pairs = self.rotary.interleaved_pairs
        if (q.shape[0] <= ROPE_FOLD_MAX_ROWS and has_cache and not ctx.is_prefill and ctx.slot_mapping is not None
                and ctx.block_tables is not None and ctx.context_lens is not None):
            o = hip_ops.rope_paged_decode(q, k, k, positions, cos, sin, None, None, 0.0, ctx.slot_mapping, attn.k_cache,
                                          attn.v_cache, ctx.block_tables, ctx.context_lens, attn.scale,
                                          interleaved_pairs=pairs, chunk=attn.chunk, out=out)
            if o is not None:
                return
        want_k = ctx.is_prefill and not (ctx.prefix_cached and has_cache)
        q_rot, k_rot = hip_ops.rope_qk_store(q, k, k, positions, cos, sin,
                                             k_cache=attn.k_cache if has_cache else None,
                                             v_cache=attn.v_cache if has_cache else None,
                                             slot_mapping=ctx.slot_mapping if has_cache else None, want_k_out=want_k,
                                             interleaved_pairs=pairs)
        attn(q_rot, k_rot, k, kv_stored=True, out=out)

    def forward(self, h, positions, run: int):
        """attention(h) + mlp(h) of pass ``run``: [T, width] (or its K-split partial sums)."""
        t, d = h.shape[0], self.head_dim
        z, k_at = self.qk(h), self.qk.offsets["k"]
        q = z[:, :self.heads * d].view(t, self.heads, d)
        k = z[:, k_at:k_at + self.kv_heads * d].view(t, self.kv_heads, d)
        mixed = torch.empty((t, self.proj_out.weight.shape[1]), dtype=h.dtype, device=h.device)
        self._attend(self.attn[run], q, k, positions, mixed[:, :self.heads * d].view(t, self.heads, d))
        if self.ff:
            gated_linear(h, self.gate_up, "gelu_tanh", out=mixed[:, self.proj_out.offsets["down"]:])
        return self.proj_out(mixed, partial_ok=True)


class MofaraxForCausalLM(nn.Module):
    # checkpoint name fragment -> (parameter, segment); a trailing fragment wins over nothing, so the order is free
    packed_modules_mapping = {".mix.q": (".qk.weight", "q"), ".mix.k": (".qk.weight", "k"),
                              ".mlp.gate": (".gate_up.weight", "gate"), ".mlp.up": (".gate_up.weight", "up"),
                              ".mix.o": (".proj_out.weight", "o"), ".mlp.down": (".proj_out.weight", "down"),
                              ".side.gate": (".side.gate.weight", "gate"), ".side.proj": (".side.proj.weight", "proj"),
                              "side.embed": ("side_embed", None), "final.norm": ("final_norm", None),
                              "loop.step": ("loop_step", None), "head": ("head.weight", None)}

    def __init__(self, config) -> None:
        super().__init__()
        self.config = config
        w = pad_to(config.hidden_size)
        self.runs = config.layer_runs()
        self.embed = padded_parameter(config.vocab_size, w)
        self.loop_step = padded_parameter(config.loop[2], w) if config.loop else None
        self.side_embed = padded_parameter(config.vocab_size, config.side_dim * len(config.layers)) if config.side_dim else None
        self.stack = []
        for i in range(len(config.layers)):
            layer = MofaraxLayer(config, i, 1 + max(t for j, t, _ in self.runs if j == i))
            self.add_module(f"l{i}", layer)
            self.stack.append(layer)
        self.final_norm = padded_parameter(w)
        self.head = ParallelLMHead(config.vocab_size, config.hidden_size, storage_dim=w)

    # ---- the residual stream between two layer runs -------------------------------------------------------------------
    def _edge(self, x, r: int, ids, dtype, y=None, y_norm_w=None):
        """Add ``y`` (none: start the stream from the embedding) and what comes ahead of layer run ``r``; -> the input of
        that run (or of the head): the stream under its norm."""
        c = self.config
        vec, again = None, False
        if r < len(self.runs):
            i, t, starts = self.runs[r]
            norm = self.stack[i].norm1
            if starts:
                vec, again = self.loop_step[t], t > 0
        else:
            norm = self.final_norm
        return hip_ops.residual_update(
            x, y=y, y_norm_w=y_norm_w, embed=self.embed if y is None or again else None, ids=ids,
            embed_scale=c.embedding_scale, start=y is None, vec=vec, norm_w=norm, norm_offset=1.0, eps=c.norm_eps,
            cols_true=c.hidden_size, dtype=dtype)

    def forward(self, input_ids, positions):
        c, ids, dtype = self.config, input_ids.contiguous(), self.embed.dtype
        x = torch.empty((ids.shape[0], self.embed.shape[1]), dtype=torch.float32, device=ids.device)
        h = self._edge(x, 0, ids, dtype)
        for r, (i, t, _) in enumerate(self.runs):
            layer = self.stack[i]
            y = layer(h, positions, t)
            y = getattr(y, "data", y)           # K-split partial sums are added up by the residual update
            if layer.side is None:
                h = self._edge(x, r + 1, ids, dtype, y)
                continue
            xs = hip_ops.residual_update(x, y=y, dtype=dtype, want_out=dtype != torch.float32)
            y = layer.side(x if xs is None else xs, ids, self.side_embed)
            h = self._edge(x, r + 1, ids, dtype, y, layer.side.norm)
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
        """Random checkpoint tensors of unit gain (norm weights neutral)."""
        out, dev = {}, self.embed.device
        for name, shape in self.config.weight_shapes().items():
            if name.endswith("side.norm"):
                t = torch.ones(shape, device=dev)
            elif name.endswith("norm1") or name == "final.norm":
                t = torch.zeros(shape, device=dev)
            else:
                t = torch.empty(shape, device=dev, dtype=self.embed.dtype).normal_(0.0, 1.0, generator=gen)
                if name == "embed":
                    t /= self.config.embedding_scale
                elif name not in ("side.embed", "loop.step"):
                    t /= shape[-1] ** 0.5
            out[name] = t
        return out
