"""Typed configuration of the Lifesun decoder, read from ``config.json``.

The file lists the model's layers one by one: ``{"architecture": "Lifesun", "vocab": V, "width": D, "norm": {"eps": e},
"logit_scale": s, "loop": {"start", "stop", "times"}, "layers": [{"type": ..., "mixer": {...}, "mlp": {...} | null},
...]}``.  Every size and constant that can differ between two models of the design is a key of the file; ``loop``, a
mixer's ``mask`` and ``mlp`` may be absent (the model then has no such thing), ``kv_heads`` and ``vdim`` default to
``heads`` and ``dim``, and a key this reader does not know is an error.

A layer's ``type`` names its mixer, two mixers side by side with a weight each (``left``, ``right``, ``left_scale``,
``right_scale``).  ``parallel``: on the left an attention within chunks (``heads``, ``kv_heads``, ``dim``, ``vdim``,
``scale``, ``mask = {"size"}``), on the right a real-gated linear recurrent unit (``width``, ``blocks`` of its gates'
matrices, ``conv`` taps).  ``parallel_2``: on the left an attention over a sliding window with capped scores (the same
keys, ``softcap`` and ``rot = {"base", "dims"}``), on the right a retention (``heads``, ``dim``, ``vdim``, ``rot``,
``decay``, one number a head).  Feed-forward ``dense``: ``ff`` (its width).
"""
from __future__ import annotations

import dataclasses
from typing import Any, Mapping, Optional

from .llama4 import ConfigError
from .rovidra import DenseFeedForwardConfig, _need, _only
from .specs import LayerSpec, ModelPlan, OrderEntry, part
from .tiradra import LoopConfig, looped_order

# fixed by the design
DECAY_RATE = 8.0  # the recurrent unit's decay is exp(-DECAY_RATE * gate * softplus(lam))


@dataclasses.dataclass(frozen=True)
class HalfRotationConfig:
    base: float
    dims: int

    @classmethod
    def from_dict(cls, m: Mapping[str, Any], where: str, limit: int) -> "HalfRotationConfig":
        _only(m, ("base", "dims"), where)
        c = cls(float(_need(m, "base", where)), int(_need(m, "dims", where)))
        if c.dims % 2 or not 0 < c.dims <= limit or c.base <= 0:
            raise ConfigError(f"config.json: {where}: an even dims of at most {limit} and a positive base are needed")
        return c

    def to_dict(self) -> dict:
        return dataclasses.asdict(self)

    def spec(self):
        return part("rope_half", theta=self.base, rotary_dim=self.dims)


def _attention_sizes(m: Mapping[str, Any], where: str) -> dict:
    heads, dim = int(_need(m, "heads", where)), int(_need(m, "dim", where))
    kv = int(m["kv_heads"]) if m.get("kv_heads") is not None else heads
    vdim = int(m["vdim"]) if m.get("vdim") is not None else dim
    size = None
    if m.get("mask") is not None:
        _only(m["mask"], ("size",), where + ".mask")
        size = int(_need(m["mask"], "size", where + ".mask"))
    if min(heads, kv, dim, vdim) < 1 or heads % kv or (size is not None and size < 1):
        raise ConfigError(f"config.json: {where}: positive sizes and heads a multiple of kv_heads are needed")
    return dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=float(_need(m, "scale", where)), size=size)


@dataclasses.dataclass(frozen=True)
class ChunkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    size: Optional[int]  # tokens of a chunk; None: one chunk holds everything

    @classmethod
    def from_dict(cls, m: Mapping[str, Any], where: str) -> "ChunkAttentionConfig":
        _only(m, ("heads", "kv_heads", "dim", "vdim", "scale", "mask"), where)
        return cls(**_attention_sizes(m, where))

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.size is not None:
            d["mask"] = {"size": self.size}
        return d

    def spec(self, D: int, eps: float):
        return part("attention", hidden_size=D, num_heads=self.heads, num_kv_heads=self.kv_heads, head_dim=self.dim,
                    value_dim=self.vdim, softmax_scale=self.scale,
                    retention=("all",) if self.size is None else ("chunk", self.size), position=part("none"),
                    qk_norm=part("rmsnorm", eps=eps, weighted=False), sink="zero", output_gate="head")


@dataclasses.dataclass(frozen=True)
class CappedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    size: Optional[int]  # tokens a query sees; None: every earlier one
    softcap: float
    rot: HalfRotationConfig

    @classmethod
    def from_dict(cls, m: Mapping[str, Any], where: str) -> "CappedAttentionConfig":
        _only(m, ("heads", "kv_heads", "dim", "vdim", "scale", "mask", "softcap", "rot"), where)
        c = cls(**_attention_sizes(m, where), softcap=float(_need(m, "softcap", where)),
                rot=HalfRotationConfig.from_dict(_need(m, "rot", where), where + ".rot", int(m["dim"])))
        if c.softcap <= 0:
            raise ConfigError(f"config.json: {where}.softcap must be positive")
        return c

    def to_dict(self) -> dict:
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
             "softcap": self.softcap, "rot": self.rot.to_dict()}
        if self.size is not None:
            d["mask"] = {"size": self.size}
        return d

    def spec(self, D: int, eps: float):
        return part("attention", hidden_size=D, num_heads=self.heads, num_kv_heads=self.kv_heads, head_dim=self.dim,
                    value_dim=self.vdim, softmax_scale=self.scale,
                    retention=("all",) if self.size is None else ("window", self.size), position=self.rot.spec(),
                    qk_norm=part("rmsnorm", eps=eps, weighted=True, before_rotation=True, span="projection"),
                    score_cap=self.softcap)


@dataclasses.dataclass(frozen=True)
class GatedUnitConfig:
    width: int
    blocks: int
    conv: int

    @classmethod
    def from_dict(cls, m: Mapping[str, Any], where: str) -> "GatedUnitConfig":
        _only(m, ("width", "blocks", "conv"), where)
        c = cls(*(int(_need(m, k, where)) for k in ("width", "blocks", "conv")))
        if min(c.width, c.blocks, c.conv) < 1 or c.width % c.blocks:
            raise ConfigError(f"config.json: {where}: positive sizes and a width of equal blocks are needed")
        return c

    def to_dict(self) -> dict:
        return dataclasses.asdict(self)

    def spec(self, D: int, eps: float):
        return part("gated_unit", hidden_size=D, width=self.width, blocks=self.blocks, conv_taps=self.conv,
                    decay_rate=DECAY_RATE)


@dataclasses.dataclass(frozen=True)
class RetentionConfig:
    heads: int
    dim: int
    vdim: int
    rot: HalfRotationConfig
    decay: tuple

    @classmethod
    def from_dict(cls, m: Mapping[str, Any], where: str) -> "RetentionConfig":
        _only(m, ("heads", "dim", "vdim", "rot", "decay"), where)
        heads, dim = int(_need(m, "heads", where)), int(_need(m, "dim", where))
        c = cls(heads, dim, int(m["vdim"]) if m.get("vdim") is not None else dim,
                HalfRotationConfig.from_dict(_need(m, "rot", where), where + ".rot", dim),
                tuple(float(g) for g in _need(m, "decay", where)))
        if min(c.heads, c.dim, c.vdim) < 1 or len(c.decay) != c.heads or not all(0.0 <= g <= 1.0 for g in c.decay):
            raise ConfigError(f"config.json: {where}: positive sizes and a decay between 0 and 1 for every head are needed")
        return c

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "rot": self.rot.to_dict(),
                "decay": list(self.decay)}

    def spec(self, D: int, eps: float):
        return part("retention", hidden_size=D, num_heads=self.heads, head_dim=self.dim, value_dim=self.vdim,
                    position=self.rot.spec(), decay=self.decay, norm_eps=eps)


@dataclasses.dataclass(frozen=True)
class PairConfig:
    left: Any
    right: Any
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, kinds, m: Mapping[str, Any], where: str) -> "PairConfig":
        _only(m, ("left", "right", "left_scale", "right_scale"), where)
        left, right = kinds
        return cls(left.from_dict(_need(m, "left", where), where + ".left"),
                   right.from_dict(_need(m, "right", where), where + ".right"),
                   float(_need(m, "left_scale", where)), float(_need(m, "right_scale", where)))

    def to_dict(self) -> dict:
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}

    def spec(self, D: int, eps: float):
        return part("side_by_side", hidden_size=D, left=self.left.spec(D, eps), right=self.right.spec(D, eps),
                    left_scale=self.left_scale, right_scale=self.right_scale)


_PAIRS = {"parallel": (ChunkAttentionConfig, GatedUnitConfig), "parallel_2": (CappedAttentionConfig, RetentionConfig)}


@dataclasses.dataclass(frozen=True)
class LifesunLayerConfig:
    type: str
    mixer: PairConfig
    mlp: Optional[DenseFeedForwardConfig]


@dataclasses.dataclass(frozen=True)
class LifesunConfig:
    vocab: int
    width: int
    norm_eps: float
    logit_scale: float
    loop: Optional[LoopConfig]
    layers: tuple

    @classmethod
    def from_dict(cls, top: Mapping[str, Any]) -> "LifesunConfig":
        _only(top, ("architecture", "architectures", "model_type", "vocab", "width", "norm", "logit_scale", "loop",
                    "layers"), "the top level")
        layers = []
        for i, entry in enumerate(_need(top, "layers", "the top level")):
            where = f"layers[{i}]"
            _only(entry, ("type", "mixer", "mlp"), where)
            kind = _need(entry, "type", where)
            if kind not in _PAIRS:
                raise ConfigError(f"config.json: {where}.type {kind!r} is not known ({', '.join(sorted(_PAIRS))})")
            mlp = entry.get("mlp")
            layers.append(LifesunLayerConfig(
                kind, PairConfig.from_dict(_PAIRS[kind], _need(entry, "mixer", where), where + ".mixer"),
                None if mlp is None else DenseFeedForwardConfig.from_dict(mlp, where + ".mlp")))
        if not layers:
            raise ConfigError("config.json: no layers")
        norm = _need(top, "norm", "the top level")
        _only(norm, ("eps",), "norm")
        loop = top.get("loop")
        if loop is not None:
            loop = LoopConfig.from_dict(loop, len(layers))
            if loop.start == loop.stop:
                raise ConfigError(f"config.json: loop {top['loop']} holds no layer")
        scale = top.get("logit_scale")
        return cls(vocab=int(_need(top, "vocab", "the top level")), width=int(_need(top, "width", "the top level")),
                   norm_eps=float(_need(norm, "eps", "norm")), logit_scale=1.0 if scale is None else float(scale),
                   loop=loop, layers=tuple(layers))

    def to_dict(self, architecture: str = "Lifesun") -> dict:
        d = {"architecture": architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
             "logit_scale": self.logit_scale,
             "layers": [{"type": lc.type, "mixer": lc.mixer.to_dict(),
                         "mlp": None if lc.mlp is None else lc.mlp.to_dict()} for lc in self.layers]}
        if self.loop is not None:
            d["loop"] = dataclasses.asdict(self.loop)
        return d

    def plan(self) -> ModelPlan:
        D, eps = self.width, self.norm_eps
        norm = part("layernorm", eps=eps, size=D)
        layers = tuple(
            LayerSpec(mixer=lc.mixer.spec(D, eps), mixer_norm=norm, feed_forward_norm=norm,
                      feed_forward=None if lc.mlp is None else part("dense_swiglu", hidden_size=D,
                                                                    intermediate_size=lc.mlp.ff, activation="gelu_tanh"),
                      arrangement="parallel_one_norm")
            for lc in self.layers)
        # every run of a layer has a cache and state of its own
        order = tuple(OrderEntry(layer=i, cache=k, enters_pass=t)
                      for k, (i, t) in enumerate(looped_order(len(layers), self.loop)))
        return ModelPlan(vocab_size=self.vocab, hidden_size=D, layers=layers, order=order, final_norm=norm,
                         tie_word_embeddings=False,
                         embedding=part("token_embedding", vocab_size=self.vocab, hidden_size=D),
                         loop=None if self.loop is None else part("pass_projection", hidden_size=D, times=self.loop.times),
                         head=part("linear_head", vocab_size=self.vocab, hidden_size=D, scale=self.logit_scale))
