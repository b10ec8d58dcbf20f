"""Pununex decoder glue: an fp32 residual stream that the sublayers read as it is; their outputs are layer-normed, scaled and added.

    x = E[token] + B[previous token, token]                                            (one launch)
    [every input of the layer's mixers] GEMM
      gated delta rule (layers/delta_rule.py), beside it in some layers attention: head norms + K/V store + attention (decode: ONE
      launch), both into `mixed`
    -> [o | o] GEMM over `mixed`, the two mixers summed in the accumulators, their scales already in it
    -> x += scale * ln(y);  cast                                                       (one launch)
    dense or expert feed-forward
    -> x += scale * ln(y) (y: the shared expert + the weighted choices);  cast         (one launch)
Head dims between the kernels' sizes, and widths that are no multiple of 64, are zero-padded in the weights at load time."""
from __future__ import annotations

import os

import torch
from torch import nn

from .. import hip_ops
from ..layers import Attention, ExpertMLP, GatedDeltaRule, PairEmbedding, ParallelLMHead, Segment, SegmentedLinear, padded_parameter
from ..layers.linear import gated_linear, pad_to
from ..parallel_state import get_tensor_parallel_world_size
from ..utils.context import get_context
from ..utils.loader import load_weight
from .mofarax import kernel_head_dim

__all__ = ["PununexLayer", "PununexForCausalLM"]

# rows up to which a decode step folds head norms + K/V store into the attention launch (see glue/qwen.py)
NORM_FOLD_MAX_ROWS = int(os.environ.get("MV_ROPE_FOLD_MAX", "128"))


def _mixed(rows: int, linear, used: int, like):
    """Input rows of an output projection; columns that nothing writes must be zero."""
    cols = linear.weight.shape[1]
    make = torch.empty if used == cols else torch.zeros
    return make((rows, cols), dtype=like.dtype, device=like.device)


class DeltaMixer(nn.Module):
    def __init__(self, width: int, spec, eps: float) -> None:
        super().__init__()
        self.rule = GatedDeltaRule(spec.heads, spec.kv_heads, spec.dim, spec.vdim, spec.taps, eps)
        self.in_proj = SegmentedLinear(width, self.rule.segments, split="out")
        self.used = spec.heads * self.rule.shape.p
        self.o = SegmentedLinear(width, [Segment("o", spec.heads, spec.vdim, self.rule.shape.p)], split="in")

    def forward(self, h, positions):
        mixed = _mixed(h.shape[0], self.o, self.used, h)
        self.rule(self.in_proj(h), mixed[:, :self.used])
        return self.o(mixed, partial_ok=True)


class ParallelMixer(nn.Module):
    """Attention (left) and a gated delta rule (right) on the same input: one input and one output projection."""

    def __init__(self, width: int, spec, eps: float) -> None:
        super().__init__()
        a, r = spec.left, spec.right
        d = self.head_dim = kernel_head_dim(max(a.dim, a.vdim))
        self.heads, self.kv_heads, self.dim, self.eps = a.heads, a.kv_heads, a.dim, eps
        self.rule = GatedDeltaRule(r.heads, r.kv_heads, r.dim, r.vdim, r.taps, eps, "sigmoid", (r.decay_rank, r.gate_rank),
                                   spec.right_scale, "right.")
        self.in_proj = SegmentedLinear(width, [Segment("left.q", a.heads, a.dim, d), Segment("left.k", a.kv_heads, a.dim, d),
                                               Segment("left.v", a.kv_heads, a.vdim, d), *self.rule.segments], split="out")
        self.q_norm, self.k_norm, self.sink = padded_parameter(d), padded_parameter(d), padded_parameter(a.heads)
        self.attn = Attention(a.heads, d, a.scale, a.kv_heads,
                              mask=hip_ops.AttnMask(a.window, a.keep_first, a.softcap, spec.left_scale))
        self.o = SegmentedLinear(width, [Segment("left.o", a.heads, a.vdim, d),
                                         Segment("right.o", r.heads, r.vdim, self.rule.shape.p)], split="in")
        self.right_cols = r.heads * self.rule.shape.p
        self.used = self.o.offsets["right.o"] + self.right_cols

    def finish_weights(self) -> None:
        self.attn.with_sink(self.sink.data)

    def _attend(self, z, positions, out) -> None:
        ctx, t, d, at, attn = get_context(), z.shape[0], self.head_dim, self.in_proj.offsets, self.attn
        q, k, v = (z[:, at[n]:at[n] + h * d].view(t, h, d)
                   for n, h in (("left.q", self.heads), ("left.k", self.kv_heads), ("left.v", self.kv_heads)))
        has_cache = attn.k_cache.numel() > 0
        norms = (positions, None, None, self.q_norm, self.k_norm, self.eps)      # nothing is rotated
        if (t <= NORM_FOLD_MAX_ROWS and has_cache and not ctx.is_prefill and ctx.slot_mapping is not None
                and ctx.block_tables is not None and ctx.context_lens is not None):
            o = hip_ops.rope_paged_decode(q, k, v, *norms, ctx.slot_mapping, attn.k_cache, attn.v_cache, ctx.block_tables,
                                          ctx.context_lens, attn.scale, interleaved_pairs=0, out=out, mask=attn.mask,
                                          norm_dim=self.dim)
            if o is not None:
                return
        want_k = ctx.is_prefill and not (ctx.prefix_cached and has_cache)
        q, k = hip_ops.rope_qk_store(q, k, v, *norms, k_cache=attn.k_cache if has_cache else None,
                                     v_cache=attn.v_cache if has_cache else None,
                                     slot_mapping=ctx.slot_mapping if has_cache else None, want_k_out=want_k, interleaved_pairs=0,
                                     norm_dim=self.dim)
        attn(q, k, v, kv_stored=True, out=out)

    def forward(self, h, positions):
        z, t = self.in_proj(h), h.shape[0]
        mixed = _mixed(t, self.o, self.used, h)
        self._attend(z, positions, mixed[:, :self.heads * self.head_dim].view(t, self.heads, self.head_dim))
        start, right = self.in_proj.offsets["right.v"], self.o.offsets["right.o"]
        self.rule(z[:, start:start + self.rule.columns], mixed[:, right:right + self.right_cols])
        return self.o(mixed, partial_ok=True)


class ReluMLP(nn.Module):
    def __init__(self, width: int, ff: int) -> None:
        super().__init__()
        self.gate_up = SegmentedLinear(width, [Segment("gate", ff), Segment("up", ff)], split="out")
        self.down = SegmentedLinear(width, [Segment("down", ff)], split="in")

    def forward(self, h):
        return self.down(gated_linear(h, self.gate_up, hip_ops.RELU_GLU), partial_ok=True), None


class PununexLayer(nn.Module):
    def __init__(self, config, index: int) -> None:
        super().__init__()
        spec, width = config.layers[index], config.hidden_size
        w, m = pad_to(width), spec.mlp
        self.mix = (ParallelMixer if spec.type == "parallel" else DeltaMixer)(width, spec.mixer, config.norm_eps)
        self.norm1, self.norm1_b, self.ls1 = (padded_parameter(w) for _ in range(3))
        self.mlp = None
        if m is not None:
            self.mlp = (ReluMLP(width, m.ff) if not hasattr(m, "experts") else
                        ExpertMLP(width, m.experts, m.identity, m.top, m.groups, m.keep, m.scale, m.ff, m.shared_ff))
            self.norm2, self.norm2_b, self.ls2 = (padded_parameter(w) for _ in range(3))


class PununexForCausalLM(nn.Module):
    def __init__(self, config) -> None:
        super().__init__()
        if get_tensor_parallel_world_size() > 1:
            raise ValueError("Pununex runs on one GPU: its experts and low-rank projections are not sharded")
        self.config = config
        w = pad_to(config.hidden_size)
        self.embed = padded_parameter(config.vocab_size, w)
        self.bigram = PairEmbedding(config.pair_buckets, *config.pair_muls, w) if config.pair_buckets else None
        self.stack = []
        for i in range(len(config.layers)):
            layer = PununexLayer(config, i)
            self.add_module(f"l{i}", layer)
            self.stack.append(layer)
        self.final_norm, self.final_norm_b = padded_parameter(w), padded_parameter(w)
        self.head = ParallelLMHead(config.vocab_size, config.hidden_size, storage_dim=w)

    def _add(self, x, y, layer, which: str, last: bool, experts=None):
        """Add a sublayer's output to the stream; -> what the next one (``last``: the head) reads."""
        cast = last or x.dtype != self.embed.dtype       # (fp32: the stream itself)
        norm, bias, scale = (getattr(layer, n + which + b) for n, b in (("norm", ""), ("norm", "_b"), ("ls", "")))
        h = hip_ops.residual_update(x, y=getattr(y, "data", y), y_norm_w=norm, y_norm_b=bias, y_scale=scale, layer_norm=True,
                                    eps=self.config.norm_eps, cols_true=self.config.hidden_size, dtype=self.embed.dtype,
                                    experts=experts, norm_w=self.final_norm if last else None,
                                    norm_b=self.final_norm_b if last else None, want_out=cast)
        return h if cast else x

    def forward(self, input_ids, positions):
        ids = input_ids.contiguous()
        x = torch.empty((ids.shape[0], self.embed.shape[1]), dtype=torch.float32, device=ids.device)
        cast = self.embed.dtype != torch.float32
        h = hip_ops.residual_update(x, embed=self.embed, ids=ids, start=True, cols_true=self.config.hidden_size, want_out=cast,
                                    pairs=self.bigram.rows(positions.contiguous()) if self.bigram is not None else None)
        h = h if cast else x
        for i, layer in enumerate(self.stack):
            last = i + 1 == len(self.stack)
            h = self._add(x, layer.mix(h, positions), layer, "1", last and layer.mlp is None)
            if layer.mlp is not None:
                y, experts = layer.mlp(h)
                h = self._add(x, y, layer, "2", last, experts)
        return h

    def compute_logits(self, hidden_states, gather: bool = True):
        return self.head(hidden_states, gather=gather)

    # ---- weights ------------------------------------------------------------------------------------------------------
    @property
    def packed_modules_mapping(self) -> dict:
        """Checkpoint name fragment -> (parameter, segment); the first fragment that a name contains wins."""
        out = {"final.norm.b": ("final_norm_b", None), "final.norm": ("final_norm", None), "norm1.b": ("norm1_b", None),
               "norm2.b": ("norm2_b", None), ".mix.left.q.norm": (".mix.q_norm", None), ".mix.left.k.norm": (".mix.k_norm", None),
               ".mix.left.sink": (".mix.sink", None)}
        for side in ("", "right."):
            at = ".mix." + side
            out.update({f"{at}{n}.conv": (".mix.rule.conv", n) for n in "qkv"})
            out.update({at + n: (".mix.rule." + n, None) for n in ("A_log", "dt_bias", "norm")})
        out.update({".mix.right.a2": (".mix.rule.lift.weight", "a2"), ".mix.right.g2": (".mix.rule.lift.weight", "g2")})
        for side, names in (("left.", ("q", "k", "v")), ("right.", ("q", "k", "v", "b", "a1", "g1")), ("", ("q", "k", "v", "b", "a", "g"))):
            out.update({f".mix.{side}{n}": (".mix.in_proj.weight", side + n) for n in names})
            out[f".mix.{side}o"] = (".mix.o.weight", side + "o")
        out.update({".mlp.shared.gate": (".mlp.shared_gate_up.weight", "gate"), ".mlp.shared.up": (".mlp.shared_gate_up.weight", "up"),
                    ".mlp.shared.down": (".mlp.shared_down.weight", "down")})
        for e in range(max((getattr(s.mlp, "experts", 0) for s in self.config.layers), default=0)):
            out.update({f".mlp.e{e}.{n}": (".mlp.down" if n == "down" else ".mlp.gate_up", (e, n)) for n in ("gate", "up", "down")})
        out.update({".mlp.gate": (".mlp.gate_up.weight", "gate"), ".mlp.up": (".mlp.gate_up.weight", "up"),
                    ".mlp.down": (".mlp.down.weight", "down"), "bigram": ("bigram.weight", None), "head": ("head.weight", None)})
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
        """Random checkpoint tensors of unit gain (norm weights and scales neutral, decays of all speeds)."""
        out, dev = {}, self.embed.device
        for name, shape in self.config.weight_shapes().items():
            last = name.rsplit(".", 1)[-1]
            t = torch.empty(shape, device=dev, dtype=torch.float32).normal_(0.0, 1.0, generator=gen)
            if last.startswith("norm") or last in ("ls1", "ls2"):
                t.fill_(1.0)
            elif last == "dt_bias":
                t.sub_(3.0)
            elif name.endswith(("norm.b", "norm1.b", "norm2.b")) or last == "correction":
                t.zero_()
            elif len(shape) == 2 and name not in ("embed", "bigram"):
                t /= shape[-1] ** 0.5
            out[name] = t.to(self.embed.dtype)
        return out
