"""Configurations of architectures that are described by this framework's own config.json layout (a top-level
``"architecture"`` key) instead of a transformers config class."""
from __future__ import annotations

import json
import math
import struct
from dataclasses import dataclass, replace
from pathlib import Path

__all__ = ["AttentionSpec", "LayerSpec", "MofaraxConfig", "LatentAttentionSpec", "Mamba2Spec", "ClampedMlpSpec", "MixerLayerSpec",
           "KugulornConfig", "DeltaRuleSpec", "SinkAttentionSpec", "ParallelMixerSpec", "ReluMlpSpec", "MoeSpec", "DeltaLayerSpec",
           "PununexConfig", "WavelengthScaling", "KeyValueAttentionSpec", "MinGruSpec", "GeluMlpSpec", "SigmoidMoeSpec", "StreamLayerSpec",
           "SemezenConfig", "NATIVE_CONFIGS", "checkpoint_shapes", "load_native_config"]


def _need(d: dict, key: str, where: str):
    if not isinstance(d, dict) or key not in d:
        raise ValueError(f"{where}: missing {key!r}")
    return d[key]


def _size(v, what: str) -> int:
    if isinstance(v, bool) or not isinstance(v, int) or v <= 0:
        raise ValueError(f"{what} must be a positive integer, got {v!r}")
    return v


def _count(v, what: str) -> int:
    if isinstance(v, bool) or not isinstance(v, int) or v < 0:
        raise ValueError(f"{what} must be a non-negative integer, got {v!r}")
    return v


def _real(v, what: str) -> float:
    if isinstance(v, bool) or not isinstance(v, (int, float)) or not math.isfinite(v):
        raise ValueError(f"{what} must be a finite number, got {v!r}")
    return float(v)


@dataclass(frozen=True)
class AttentionSpec:
    """Grouped-head attention with interleaved rotation and an optional chunk mask; the values are the projected keys."""
    heads: int
    kv_heads: int
    dim: int
    rot_base: float
    rot_dims: int
    scale: float
    chunk: int          # 0: no mask besides causality

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "AttentionSpec":
        heads, kv = _size(_need(m, "heads", where), f"{where}.heads"), _size(_need(m, "kv_heads", where), f"{where}.kv_heads")
        dim = _size(_need(m, "dim", where), f"{where}.dim")
        if heads % kv:
            raise ValueError(f"{where}: {heads} query heads do not divide over {kv} key/value heads")
        if _size(m.get("vdim", dim), f"{where}.vdim") != dim:
            raise ValueError(f"{where}: the values are the keys, so vdim ({m['vdim']}) must equal dim ({dim})")
        rot = _need(m, "rot", where)
        rot_dims = _size(_need(rot, "dims", f"{where}.rot"), f"{where}.rot.dims")
        if rot_dims % 2 or rot_dims > dim:
            raise ValueError(f"{where}.rot.dims must be even and at most dim ({dim}), got {rot_dims!r}")
        base = _real(_need(rot, "base", f"{where}.rot"), f"{where}.rot.base")
        mask = m.get("mask") or {}
        chunk = _size(mask["size"], f"{where}.mask.size") if mask.get("size") is not None else 0
        scale = _real(_need(m, "scale", where), f"{where}.scale")
        if scale <= 0 or base <= 0:
            raise ValueError(f"{where}: scale and rot.base must be positive, got {scale} and {base}")
        return cls(heads, kv, dim, base, rot_dims, scale, chunk)


@dataclass(frozen=True)
class LayerSpec:
    attention: AttentionSpec
    ff: int             # 0: no feed-forward

    @classmethod
    def from_dict(cls, d: dict, where: str) -> "LayerSpec":
        kind = _need(d, "type", where)
        if kind != "attention":
            raise ValueError(f"{where}: unsupported layer type {kind!r}")
        mlp, ff = d.get("mlp"), 0
        if mlp is not None:
            if mlp.get("kind", "dense") != "dense":
                raise ValueError(f"{where}: unsupported feed-forward {mlp.get('kind')!r}")
            ff = _size(_need(mlp, "ff", f"{where}.mlp"), f"{where}.mlp.ff")
        return cls(AttentionSpec.from_dict(_need(d, "mixer", where), f"{where}.mixer"), ff)


class MofaraxConfig:
    """Parallel attention / feed-forward layers over a 32-bit residual stream, a per-layer token table, and a run of
    layers that is passed several times over the same weights."""
    model_type = "mofarax"

    def __init__(self, raw: dict) -> None:
        self.architectures = ["Mofarax"]
        self.vocab_size = _size(_need(raw, "vocab", "config"), "vocab")
        self.hidden_size = _size(_need(raw, "width", "config"), "width")
        self.embedding_scale = _real((raw.get("embedding") or {}).get("scale", 1.0), "embedding.scale")
        self.norm_eps = _real(_need(_need(raw, "norm", "config"), "eps", "norm"), "norm.eps")
        side = raw.get("token_side")
        self.side_dim = _size(_need(side, "dim", "token_side"), "token_side.dim") if side else 0
        layers = _need(raw, "layers", "config")
        if not isinstance(layers, list) or not layers:
            raise ValueError("config: 'layers' must be a non-empty list")
        self.layers = [LayerSpec.from_dict(d, f"layers[{i}]") for i, d in enumerate(layers)]
        loop = raw.get("loop")
        self.loop = None
        if loop:
            start, stop = _need(loop, "start", "loop"), _need(loop, "stop", "loop")
            times = _size(_need(loop, "times", "loop"), "loop.times")
            if not 0 <= start < stop <= len(layers):
                raise ValueError(f"loop: [{start}, {stop}) is not a run of the {len(layers)} layers")
            self.loop = (start, stop, times)
        # what the engine asks of any configuration
        a = [s.attention for s in self.layers]
        self.num_hidden_layers = len(self.layer_runs())
        self.num_attention_heads = max(s.heads for s in a)
        self.num_key_value_heads = max(s.kv_heads for s in a)
        self.head_dim = max(s.dim for s in a)
        self.intermediate_size = max(s.ff for s in self.layers)
        self.max_position_embeddings: int | None = None    # none of its own; the engine's Config fills it in
        self.torch_dtype = raw.get("dtype", "bfloat16")
        self.eos_token_id = None
        self.tie_word_embeddings = False

    def layer_runs(self) -> list[tuple[int, int, bool]]:
        """The layer runs in order: (layer, pass, does a pass of the loop start here?)."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, 0, False) for i in range(n)]
        start, stop, times = self.loop
        runs = [(i, 0, False) for i in range(start)]
        for t in range(times):
            runs += [(i, t, i == start) for i in range(start, stop)]
        return runs + [(i, 0, False) for i in range(stop, n)]

    def weight_shapes(self) -> dict[str, tuple[int, ...]]:
        """Name -> shape of every tensor of a checkpoint."""
        v, d, s = self.vocab_size, self.hidden_size, self.side_dim
        out: dict[str, tuple[int, ...]] = {"embed": (v, d), "final.norm": (d,), "head": (v, d)}
        if self.loop:
            out["loop.step"] = (self.loop[2], d)
        if s:
            out["side.embed"] = (v, s * len(self.layers))
        for i, layer in enumerate(self.layers):
            a, p = layer.attention, f"l{i}."
            out[p + "norm1"] = (d,)
            out[p + "mix.q"], out[p + "mix.k"] = (a.heads * a.dim, d), (a.kv_heads * a.dim, d)
            out[p + "mix.o"] = (d, a.heads * a.dim)
            if layer.ff:
                out[p + "mlp.gate"] = out[p + "mlp.up"] = (layer.ff, d)
                out[p + "mlp.down"] = (d, layer.ff)
            if s:
                out[p + "side.gate"], out[p + "side.proj"], out[p + "side.norm"] = (s, d), (d, s), (d,)
        return out


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Attention whose keys and values are one cached latent per token; see layers/latent_attention.py."""
    heads: int
    dim: int            # unrotated query / key dims of a head
    rot_dim: int        # rotated ones, one key part for all heads
    vdim: int
    q_rank: int
    kv_rank: int
    rot_base: float
    scale: float
    window: int         # 0: every key up to the query
    kv_from: int | None  # layer whose latents this one reads instead of its own

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "LatentAttentionSpec":
        sizes = {k: _size(_need(m, k, where), f"{where}.{k}") for k in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")}
        rot = _need(m, "rot", where)
        dims = _size(rot.get("dims", sizes["rot_dim"]), f"{where}.rot.dims")
        if sizes["rot_dim"] % 2 or dims != sizes["rot_dim"]:
            raise ValueError(f"{where}: rot_dim must be even and all of it rotated, got {sizes['rot_dim']} and rot.dims {dims}")
        base, scale = _real(_need(rot, "base", f"{where}.rot"), f"{where}.rot.base"), _real(_need(m, "scale", where), f"{where}.scale")
        if scale <= 0 or base <= 0:
            raise ValueError(f"{where}: scale and rot.base must be positive, got {scale} and {base}")
        mask = m.get("mask") or {}
        window = _size(mask["size"], f"{where}.mask.size") if mask.get("size") is not None else 0
        source = m.get("kv_from")
        if source is not None and (isinstance(source, bool) or not isinstance(source, int) or source < 0):
            raise ValueError(f"{where}.kv_from must be a layer's index, got {source!r}")
        return cls(**sizes, rot_base=base, scale=scale, window=window, kv_from=source)

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        h, out = self.heads, {"dq": (self.q_rank, width), "dq.norm": (self.q_rank,)}
        out["uq"], out["o"] = (h * (self.dim + self.rot_dim), self.q_rank), (width, h * self.vdim)
        out["uk"], out["uv"] = (h * self.dim, self.kv_rank), (h * self.vdim, self.kv_rank)
        if self.kv_from is None:
            out["dkv"], out["dkv.norm"] = (self.kv_rank + self.rot_dim, width), (self.kv_rank,)
        return out


@dataclass(frozen=True)
class Mamba2Spec:
    """Selective state space mixer; see layers/mamba2.py."""
    heads: int
    vdim: int
    state: int
    groups: int
    taps: int           # of the causal convolution
    norm_groups: int

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "Mamba2Spec":
        s = {k: _size(_need(m, k, where), f"{where}.{k}") for k in ("heads", "vdim", "state", "groups", "conv", "norm_groups")}
        s["taps"] = s.pop("conv")
        if s["heads"] % s["groups"]:
            raise ValueError(f"{where}: {s['heads']} heads do not divide over {s['groups']} groups")
        if s["heads"] * s["vdim"] % s["norm_groups"]:
            raise ValueError(f"{where}: {s['heads'] * s['vdim']} columns do not divide into {s['norm_groups']} norm groups")
        return cls(**s)

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        inner, bc = self.heads * self.vdim, 2 * self.groups * self.state
        out = {"in": (2 * inner + bc + self.heads, width), "conv": (inner + bc, self.taps), "conv.b": (inner + bc,)}
        out["dt_bias"] = out["A_log"] = out["D"] = (self.heads,)
        out["norm"], out["o"] = (inner,), (width, inner)
        return out


@dataclass(frozen=True)
class ClampedMlpSpec:
    ff: int
    limit: float

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "ClampedMlpSpec":
        if m.get("kind", "dense") != "dense":
            raise ValueError(f"{where}: unsupported feed-forward {m.get('kind')!r}")
        limit = _real(_need(m, "limit", where), f"{where}.limit")
        if limit <= 0:
            raise ValueError(f"{where}.limit must be positive, got {limit}")
        return cls(_size(_need(m, "ff", where), f"{where}.ff"), limit)


@dataclass(frozen=True)
class MixerLayerSpec:
    """A mixer of one of several kinds and an optional feed-forward."""
    type: str
    mixer: LatentAttentionSpec | Mamba2Spec
    mlp: ClampedMlpSpec | None
    KINDS = {"latent_attention": LatentAttentionSpec, "mamba2": Mamba2Spec}

    @classmethod
    def from_dict(cls, d: dict, where: str) -> "MixerLayerSpec":
        kind = _need(d, "type", where)
        if kind not in cls.KINDS:
            raise ValueError(f"{where}: unsupported layer type {kind!r}; known: {sorted(cls.KINDS)}")
        mlp = d.get("mlp")
        return cls(kind, cls.KINDS[kind].from_dict(_need(d, "mixer", where), f"{where}.mixer"),
                   None if mlp is None else ClampedMlpSpec.from_dict(mlp, f"{where}.mlp"))


class KugulornConfig:
    """Latent attention and state space layers, some sharing one layer's latents, over a 32-bit residual stream."""
    model_type = "kugulorn"

    def __init__(self, raw: dict) -> None:
        self.architectures = ["Kugulorn"]
        self.vocab_size = _size(_need(raw, "vocab", "config"), "vocab")
        self.hidden_size = _size(_need(raw, "width", "config"), "width")
        self.norm_eps = _real(_need(_need(raw, "norm", "config"), "eps", "norm"), "norm.eps")
        self.residual_mult = _real(raw.get("residual_mult", 1.0), "residual_mult")
        layers = _need(raw, "layers", "config")
        if not isinstance(layers, list) or not layers:
            raise ValueError("config: 'layers' must be a non-empty list")
        self.layers = [MixerLayerSpec.from_dict(d, f"layers[{i}]") for i, d in enumerate(layers)]
        for i, s in enumerate(self.layers):
            j = getattr(s.mixer, "kv_from", None)
            if j is None:
                continue
            src = self.layers[j] if j < i else None
            if src is None or src.type != s.type or src.mixer.kv_from is not None:
                raise ValueError(f"layers[{i}].mixer.kv_from: {j} is not an earlier layer with latents of its own")
            a, b = src.mixer, s.mixer
            if (a.kv_rank, a.rot_dim, a.rot_base) != (b.kv_rank, b.rot_dim, b.rot_base):
                raise ValueError(f"layers[{i}].mixer: kv_rank, rot_dim and rot.base must equal those of layer {j}")
        # what the engine asks of any configuration
        self.num_hidden_layers = len(self.layers)
        self.num_attention_heads = max(s.mixer.heads for s in self.layers)
        self.num_key_value_heads = 1
        self.head_dim = max((s.mixer.kv_rank + s.mixer.rot_dim for s in self.layers if s.type != "mamba2"), default=1)
        self.intermediate_size = max((s.mlp.ff for s in self.layers if s.mlp), default=0)
        self.recurrent_state = any(s.type == "mamba2" for s in self.layers)
        self.max_position_embeddings: int | None = None    # none of its own; the engine's Config fills it in
        self.torch_dtype = raw.get("dtype", "bfloat16")
        self.eos_token_id = None
        self.tie_word_embeddings = False

    def weight_shapes(self) -> dict[str, tuple[int, ...]]:
        """Name -> shape of every tensor of a checkpoint."""
        v, d = self.vocab_size, self.hidden_size
        out: dict[str, tuple[int, ...]] = {"embed": (v, d), "final.norm": (d,), "head": (v, d)}
        for i, s in enumerate(self.layers):
            p = f"l{i}."
            out[p + "norm1"] = out[p + "norm1b"] = out[p + "ls1"] = (d,)
            out.update({f"{p}mix.{k}": v for k, v in s.mixer.weight_shapes(d).items()})
            if s.mlp:
                out[p + "norm2"] = out[p + "norm2b"] = out[p + "ls2"] = (d,)
                out[p + "mlp.gate"] = out[p + "mlp.up"] = (s.mlp.ff, d)
                out[p + "mlp.down"] = (d, s.mlp.ff)
        return out


@dataclass(frozen=True)
class SinkAttentionSpec:
    """Grouped-head attention without positions: normed queries and keys, a window that keeps the first tokens, capped scores, a
    sink per head in the softmax denominator."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float      # 0: none
    window: int         # 0: every key up to the query
    keep_first: int

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "SinkAttentionSpec":
        s = {k: _size(_need(m, k, where), f"{where}.{k}") for k in ("heads", "kv_heads", "dim", "vdim")}
        if s["heads"] % s["kv_heads"]:
            raise ValueError(f"{where}: {s['heads']} query heads do not divide over {s['kv_heads']} key/value heads")
        scale, cap = _real(_need(m, "scale", where), f"{where}.scale"), m.get("softcap")
        cap = 0.0 if cap is None else _real(cap, f"{where}.softcap")
        if scale <= 0 or cap < 0:
            raise ValueError(f"{where}: scale must be positive and softcap not negative, got {scale} and {cap}")
        mask = m.get("mask") or {}
        window = _size(mask["size"], f"{where}.mask.size") if mask.get("size") is not None else 0
        return cls(**s, scale=scale, softcap=cap, window=window,
                   keep_first=_count(mask.get("keep_first") or 0, f"{where}.mask.keep_first"))

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        return {"q": (self.heads * self.dim, width), "k": (self.kv_heads * self.dim, width), "v": (self.kv_heads * self.vdim, width),
                "q.norm": (self.dim,), "k.norm": (self.dim,), "sink": (self.heads,), "o": (width, self.heads * self.vdim)}


@dataclass(frozen=True)
class DeltaRuleSpec:
    """Gated delta rule; see layers/delta_rule.py.  ``channel_decay``: a decay per key channel and a sigmoid gate, each through a
    projection of low rank; else a decay per head and a silu gate."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int           # of the causal convolutions
    channel_decay: bool = False
    decay_rank: int = 0  # of the low-rank projections; a checkpoint's tensors give them (0: not known yet)
    gate_rank: int = 0

    @classmethod
    def from_dict(cls, m: dict, where: str, channel_decay: bool = False) -> "DeltaRuleSpec":
        s = {k: _size(_need(m, k, where), f"{where}.{k}") for k in ("heads", "kv_heads", "dim", "vdim", "conv")}
        s["taps"] = s.pop("conv")
        if s["heads"] % s["kv_heads"]:
            raise ValueError(f"{where}: {s['heads']} heads do not divide over {s['kv_heads']} key heads")
        rank = _count(m.get("rank") or 0, f"{where}.rank")
        return cls(**s, channel_decay=channel_decay, decay_rank=rank, gate_rank=rank)

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        h, k, v = self.heads, self.kv_heads * self.dim, self.heads * self.vdim
        out = {"q": (k, width), "k": (k, width), "v": (v, width), "q.conv": (k, self.taps), "k.conv": (k, self.taps),
               "v.conv": (v, self.taps), "b": (h, width), "A_log": (h,), "norm": (self.vdim,), "o": (width, v)}
        if self.channel_decay:
            if not self.decay_rank or not self.gate_rank:
                raise ValueError("the ranks of the decay's and the gate's projections are not known: they come from the "
                                 "checkpoint's tensors a1 and g1 (or 'rank' in the configuration)")
            out.update(a1=(self.decay_rank, width), a2=(h * self.dim, self.decay_rank), dt_bias=(h * self.dim,),
                       g1=(self.gate_rank, width), g2=(v, self.gate_rank))
        else:
            out.update(a=(h, width), dt_bias=(h,), g=(v, width))
        return out


@dataclass(frozen=True)
class ParallelMixerSpec:
    """Attention and a gated delta rule side by side on the same input, summed with a scale each."""
    left: SinkAttentionSpec
    right: DeltaRuleSpec
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "ParallelMixerSpec":
        return cls(SinkAttentionSpec.from_dict(_need(m, "left", where), f"{where}.left"),
                   DeltaRuleSpec.from_dict(_need(m, "right", where), f"{where}.right", channel_decay=True),
                   _real(m.get("left_scale", 1.0), f"{where}.left_scale"), _real(m.get("right_scale", 1.0), f"{where}.right_scale"))

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        return {f"{side}.{k}": s for side in ("left", "right") for k, s in getattr(self, side).weight_shapes(width).items()}


@dataclass(frozen=True)
class ReluMlpSpec:
    ff: int

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "ReluMlpSpec":
        return cls(_size(_need(m, "ff", where), f"{where}.ff"))

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        return {"gate": (self.ff, width), "up": (self.ff, width), "down": (width, self.ff)}


@dataclass(frozen=True)
class MoeSpec:
    """Experts behind a router with groups, a correction of the choice and identity experts; see layers/moe.py."""
    experts: int
    identity: int       # router outputs behind the experts whose output is the input itself
    top: int
    groups: int
    keep: int           # groups that a token chooses from
    scale: float
    ff: int
    shared_ff: int      # 0: no shared expert

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "MoeSpec":
        r, at = _need(m, "router", where), f"{where}.router"
        experts, top = _size(_need(r, "experts", at), f"{at}.experts"), _size(_need(r, "top", at), f"{at}.top")
        identity, groups = _count(r.get("identity") or 0, f"{at}.identity"), r.get("groups") or {}
        count, keep = _size(groups.get("count", 1), f"{at}.groups.count"), _size(groups.get("keep", 1), f"{at}.groups.keep")
        outputs = experts + identity
        if outputs % count or keep > count or top > outputs // count * keep:
            raise ValueError(f"{at}: {outputs} outputs in {count} groups, of which {keep} count, cannot give {top} choices")
        shared, ff = m.get("shared"), _need(_need(m, "expert", where), "ff", f"{where}.expert")
        return cls(experts, identity, top, count, keep, _real(r.get("scale", 1.0), f"{at}.scale"), _size(ff, f"{where}.expert.ff"),
                   _size(_need(shared, "ff", f"{where}.shared"), f"{where}.shared.ff") if shared else 0)

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        n = self.experts + self.identity
        out: dict[str, tuple[int, ...]] = {"router": (n, width), "correction": (n,)}
        for name, ff in [(f"e{i}", self.ff) for i in range(self.experts)] + ([("shared", self.shared_ff)] if self.shared_ff else []):
            out[name + ".gate"] = out[name + ".up"] = (ff, width)
            out[name + ".down"] = (width, ff)
        return out


@dataclass(frozen=True)
class DeltaLayerSpec:
    """A mixer of one of several kinds and an optional feed-forward of one of several kinds."""
    type: str
    mixer: DeltaRuleSpec | ParallelMixerSpec
    mlp: ReluMlpSpec | MoeSpec | None
    MIXERS = {"delta": DeltaRuleSpec, "parallel": ParallelMixerSpec}
    MLPS = {"dense": ReluMlpSpec, "moe": MoeSpec}

    @classmethod
    def from_dict(cls, d: dict, where: str) -> "DeltaLayerSpec":
        kind, mlp = _need(d, "type", where), d.get("mlp")
        if kind not in cls.MIXERS:
            raise ValueError(f"{where}: unsupported layer type {kind!r}; known: {sorted(cls.MIXERS)}")
        if mlp is not None and _need(mlp, "kind", f"{where}.mlp") not in cls.MLPS:
            raise ValueError(f"{where}.mlp: unsupported feed-forward {mlp['kind']!r}; known: {sorted(cls.MLPS)}")
        return cls(kind, cls.MIXERS[kind].from_dict(_need(d, "mixer", where), f"{where}.mixer"),
                   None if mlp is None else cls.MLPS[mlp["kind"]].from_dict(mlp, f"{where}.mlp"))


class PununexConfig:
    """Gated delta rule layers, some beside windowed attention, dense or expert feed-forwards, and a table of token pairs."""
    model_type = "pununex"
    recurrent_state = True     # the token before, and the delta rules' states

    def __init__(self, raw: dict) -> None:
        self.architectures = ["Pununex"]
        self.vocab_size = _size(_need(raw, "vocab", "config"), "vocab")
        self.hidden_size = _size(_need(raw, "width", "config"), "width")
        self.norm_eps = _real(_need(_need(raw, "norm", "config"), "eps", "norm"), "norm.eps")
        pairs = (raw.get("embedding") or {}).get("bigram")
        self.pair_buckets, self.pair_muls = 0, (0, 0)
        if pairs:
            at = "embedding.bigram"
            self.pair_buckets = _size(_need(pairs, "buckets", at), f"{at}.buckets")
            self.pair_muls = tuple(_count(_need(pairs, k, at), f"{at}.{k}") for k in ("mul_prev", "mul_cur"))
        layers = _need(raw, "layers", "config")
        if not isinstance(layers, list) or not layers:
            raise ValueError("config: 'layers' must be a non-empty list")
        self.layers = [DeltaLayerSpec.from_dict(d, f"layers[{i}]") for i, d in enumerate(layers)]
        # what the engine asks of any configuration
        attention = [s.mixer.left for s in self.layers if s.type == "parallel"]
        self.num_hidden_layers = len(self.layers)
        self.num_attention_heads = max([a.heads for a in attention], default=1)
        self.num_key_value_heads = max([a.kv_heads for a in attention], default=1)
        self.head_dim = max([max(a.dim, a.vdim) for a in attention], default=1)
        self.intermediate_size = max((s.mlp.ff for s in self.layers if s.mlp), default=0)
        self.max_position_embeddings: int | None = None    # none of its own; the engine's Config fills it in
        self.torch_dtype = raw.get("dtype", "bfloat16")
        self.eos_token_id = None
        self.tie_word_embeddings = False

    def take_shapes(self, shapes: dict[str, tuple[int, ...]]) -> None:
        """Sizes that only a checkpoint's tensors give: the ranks of the low-rank projections."""
        for i, s in enumerate(self.layers):
            a1, g1 = (shapes.get(f"l{i}.mix.right.{k}") for k in ("a1", "g1"))
            if s.type == "parallel" and a1 and g1:
                self.layers[i] = replace(s, mixer=replace(s.mixer, right=replace(s.mixer.right, decay_rank=a1[0], gate_rank=g1[0])))

    def weight_shapes(self) -> dict[str, tuple[int, ...]]:
        """Name -> shape of every tensor of a checkpoint."""
        v, d = self.vocab_size, self.hidden_size
        out: dict[str, tuple[int, ...]] = {"embed": (v, d), "final.norm": (d,), "final.norm.b": (d,), "head": (v, d)}
        if self.pair_buckets:
            out["bigram"] = (self.pair_buckets + 1, d)
        for i, s in enumerate(self.layers):
            p = f"l{i}."
            out.update({f"{p}mix.{k}": v for k, v in s.mixer.weight_shapes(d).items()})
            out[p + "norm1"] = out[p + "norm1.b"] = out[p + "ls1"] = (d,)
            if s.mlp:
                out[p + "norm2"] = out[p + "norm2.b"] = out[p + "ls2"] = (d,)
                out.update({f"{p}mlp.{k}": v for k, v in s.mlp.weight_shapes(d).items()})
        return out


@dataclass(frozen=True)
class WavelengthScaling:
    """Rotary frequencies divided by a factor where their wavelength is long; see layers/rotary_embedding.py."""
    factor: float
    low: float
    high: float
    original: float

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "WavelengthScaling":
        s = {k: _real(_need(m, k, where), f"{where}.{k}") for k in ("factor", "low", "high", "original")}
        if min(s.values()) <= 0 or s["high"] < s["low"]:
            raise ValueError(f"{where}: positive numbers required, high at least low, got {s}")
        return cls(**s)


@dataclass(frozen=True)
class KeyValueAttentionSpec:
    """Grouped-head attention in a window whose values are the projected keys, with a gate on its output; queries and keys have a
    length of one (times the root of their size) behind the rotation."""
    heads: int
    kv_heads: int
    dim: int
    rot_base: float
    rot_dims: int
    scaling: WavelengthScaling | None
    scale: float
    window: int         # 0: every key up to the query

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "KeyValueAttentionSpec":
        a = AttentionSpec.from_dict(m, where)      # (sizes, rotation and scale; its mask's size is a window here)
        scaling = m["rot"].get("scaling")
        return cls(a.heads, a.kv_heads, a.dim, a.rot_base, a.rot_dims,
                   WavelengthScaling.from_dict(scaling, f"{where}.rot.scaling") if scaling else None, a.scale, a.chunk)

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        q, k = self.heads * self.dim, self.kv_heads * self.dim
        return {"q": (q, width), "q.b": (q,), "k": (k, width), "k.b": (k,), "g": (q, width), "o": (width, q)}


@dataclass(frozen=True)
class MinGruSpec:
    """Gated running mean; see layers/mingru.py."""
    width: int

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "MinGruSpec":
        return cls(_size(_need(m, "width", where), f"{where}.width"))

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        n = self.width
        return {"z": (n, width), "z.b": (n,), "x": (n, width), "x.b": (n,), "g": (n, width), "o": (width, n)}


@dataclass(frozen=True)
class GeluMlpSpec:
    ff: int

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "GeluMlpSpec":
        return cls(_size(_need(m, "ff", where), f"{where}.ff"))

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        return {"up": (self.ff, width), "down": (width, self.ff)}


@dataclass(frozen=True)
class SigmoidMoeSpec:
    """Experts with a clamped gate behind sigmoid scores that multiply their inputs; see layers/moe.py."""
    experts: int
    top: int
    ff: int
    limit: float

    @classmethod
    def from_dict(cls, m: dict, where: str) -> "SigmoidMoeSpec":
        r, e = _need(m, "router", where), _need(m, "expert", where)
        experts, top = _size(_need(r, "experts", f"{where}.router"), f"{where}.router.experts"), _size(_need(r, "top", f"{where}.router"), f"{where}.router.top")
        if top > experts:
            raise ValueError(f"{where}.router: {experts} experts cannot give {top} choices")
        mlp = ClampedMlpSpec.from_dict(dict(e, kind="dense"), f"{where}.expert")
        return cls(experts, top, mlp.ff, mlp.limit)

    def weight_shapes(self, width: int) -> dict[str, tuple[int, ...]]:
        out: dict[str, tuple[int, ...]] = {"router": (self.experts, width)}
        for i in range(self.experts):
            out[f"e{i}.gate"] = out[f"e{i}.up"] = (self.ff, width)
            out[f"e{i}.down"] = (width, self.ff)
        return out


@dataclass(frozen=True)
class StreamLayerSpec:
    type: str
    mixer: KeyValueAttentionSpec | MinGruSpec
    mlp: GeluMlpSpec | SigmoidMoeSpec | None
    MIXERS = {"attention": KeyValueAttentionSpec, "mingru": MinGruSpec}
    MLPS = {"dense": GeluMlpSpec, "moe": SigmoidMoeSpec}

    @classmethod
    def from_dict(cls, d: dict, where: str) -> "StreamLayerSpec":
        kind, mlp = _need(d, "type", where), d.get("mlp")
        if kind not in cls.MIXERS:
            raise ValueError(f"{where}: unsupported layer type {kind!r}; known: {sorted(cls.MIXERS)}")
        if mlp is not None and _need(mlp, "kind", f"{where}.mlp") not in cls.MLPS:
            raise ValueError(f"{where}.mlp: unsupported feed-forward {mlp['kind']!r}; known: {sorted(cls.MLPS)}")
        return cls(kind, cls.MIXERS[kind].from_dict(_need(d, "mixer", where), f"{where}.mixer"),
                   None if mlp is None else cls.MLPS[mlp["kind"]].from_dict(mlp, f"{where}.mlp"))


class SemezenConfig:
    """Windowed attention and gated running means over several residual streams, each mixer reading a blend of two tokens."""
    model_type = "semezen"
    recurrent_state = True     # the normed row of the token before, in every layer
    MAX_STREAMS = 8            # of the kernel

    def __init__(self, raw: dict) -> None:
        self.architectures = ["Semezen"]
        self.vocab_size = _size(_need(raw, "vocab", "config"), "vocab")
        self.hidden_size = _size(_need(raw, "width", "config"), "width")
        self.norm_eps = _real(_need(_need(raw, "norm", "config"), "eps", "norm"), "norm.eps")
        self.streams = _size(_need(raw, "streams", "config"), "streams")
        if self.streams > self.MAX_STREAMS:
            raise ValueError(f"streams: at most {self.MAX_STREAMS} are supported, got {self.streams}")
        layers = _need(raw, "layers", "config")
        if not isinstance(layers, list) or not layers:
            raise ValueError("config: 'layers' must be a non-empty list")
        self.layers = [StreamLayerSpec.from_dict(d, f"layers[{i}]") for i, d in enumerate(layers)]
        # what the engine asks of any configuration
        attention = [s.mixer for s in self.layers if s.type == "attention"]
        self.num_hidden_layers = len(self.layers)
        self.num_attention_heads = max([a.heads for a in attention], default=1)
        self.num_key_value_heads = max([a.kv_heads for a in attention], default=1)
        self.head_dim = max([a.dim for a in attention], default=1)
        self.intermediate_size = max((s.mlp.ff for s in self.layers if s.mlp), default=0)
        self.max_position_embeddings: int | None = None    # none of its own; the engine's Config fills it in
        self.torch_dtype = raw.get("dtype", "bfloat16")
        self.eos_token_id = None
        self.tie_word_embeddings = False

    def weight_shapes(self) -> dict[str, tuple[int, ...]]:
        """Name -> shape of every tensor of a checkpoint."""
        v, d, n = self.vocab_size, self.hidden_size, self.streams
        out: dict[str, tuple[int, ...]] = {"embed": (v, d), "final.norm": (d,), "head": (v, d)}
        for i, s in enumerate(self.layers):
            p = f"l{i}."
            out[p + "shift"] = (d,)
            out.update({f"{p}mix.{k}": v for k, v in s.mixer.weight_shapes(d).items()})
            if s.mlp:
                out.update({f"{p}mlp.{k}": v for k, v in s.mlp.weight_shapes(d).items()})
            for q in ("1", "2") if s.mlp else ("1",):
                out[f"{p}norm{q}"] = (d,)
                out[f"{p}hc{q}.in"], out[f"{p}hc{q}.out"], out[f"{p}hc{q}.mix"] = (n,), (n,), (n, n)
        return out


NATIVE_CONFIGS = {"Mofarax": MofaraxConfig, "Kugulorn": KugulornConfig, "Pununex": PununexConfig, "Semezen": SemezenConfig}


def checkpoint_shapes(model_dir) -> dict[str, tuple[int, ...]]:
    """Tensor name -> shape of a directory's safetensors files, from their headers (an 8-byte length, then JSON)."""
    out: dict[str, tuple[int, ...]] = {}
    for path in sorted(Path(model_dir).glob("*.safetensors")):
        with open(path, "rb") as f:
            (n,) = struct.unpack("<Q", f.read(8))
            header = json.loads(f.read(n))
        out.update({k: tuple(v["shape"]) for k, v in header.items() if k != "__metadata__"})
    return out


def load_native_config(model_dir: str):
    """The configuration of a directory whose config.json names one of these architectures, else None."""
    path = Path(model_dir) / "config.json"
    if not path.is_file():
        return None
    raw = json.loads(path.read_text())
    name = raw.get("architecture") if isinstance(raw, dict) else None
    if name is None:
        return None
    if name not in NATIVE_CONFIGS:
        raise ValueError(f"unsupported architecture {name!r} in {path}; known: {sorted(NATIVE_CONFIGS)}")
    config = NATIVE_CONFIGS[name](raw)
    if hasattr(config, "take_shapes"):
        config.take_shapes(checkpoint_shapes(model_dir))
    return config
