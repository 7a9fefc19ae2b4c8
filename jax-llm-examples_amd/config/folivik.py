"""Typed configuration of the Folivik decoder, read from ``config.json``.

The file lists the model's layers one by one: ``{"architecture": "Folivik", "vocab": V, "width": D, "norm": {"eps":
e}, "layers": [{"type": ..., "mixer": {...}, "mlp": {...} | null}, ...]}``.  A layer's ``type`` names its mixer.
Every size and constant that can differ between two models of the design is a key of the file; a key this reader
does not know is an error.

Mixer ``latent_attention``: ``heads``, ``dim`` and ``rot_dim`` (unrotated and rotated query/key elements a head),
``vdim``, ``kv_rank``, ``q_rank`` (the latents of keys and values and of queries), ``scale``, ``rot = {"base",
"dims"}`` (``dims`` equal to ``rot_dim``).
Mixer ``attention`` (a window with a distance penalty): ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``mask =
{"size"}``.
Mixer ``mamba2``: ``heads``, ``vdim``, ``state``, ``groups``, ``conv`` (taps), ``norm_groups``.
Feed-forward ``moe``: ``router = {"experts", "top", "groups": {"count", "keep"}, "identity", "scale"}`` (``groups``,
``identity`` and ``scale`` may be absent), ``expert = {"ff"}``, ``shared = {"ff"}`` (may be absent).
"""
from __future__ import annotations

import dataclasses
from typing import Any, Mapping, Optional

from .llama4 import ConfigError
from .rovidra import _need, _only
from .specs import LayerSpec, ModelPlan, OrderEntry, part

# fixed by the design
GROUP_SCORE_TERMS = 1  # a group of experts is scored by its largest choice score
WEIGHT_FLOOR = 1e-20  # added to the sum that the chosen experts' scores are divided by


def _positive(where: str, **sizes) -> None:
    for name, value in sizes.items():
        if value < 1:
            raise ConfigError(f"config.json: {where}.{name} must be positive, got {value}")


@dataclasses.dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    q_rank: int
    scale: float
    rot_base: float

    @classmethod
    def from_dict(cls, m: Mapping[str, Any], where: str) -> "LatentAttentionConfig":
        _only(m, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank", "scale", "rot"), where)
        rot = _need(m, "rot", where)
        _only(rot, ("base", "dims"), where + ".rot")
        sizes = {k: int(_need(m, k, where)) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank")}
        _positive(where, **sizes)
        c = cls(**sizes, scale=float(_need(m, "scale", where)), rot_base=float(_need(rot, "base", where + ".rot")))
        if int(_need(rot, "dims", where + ".rot")) != c.rot_dim or c.rot_dim % 2:
            raise ConfigError(f"config.json: {where}.rot.dims must be rot_dim ({c.rot_dim}), and even")
        return c

    def to_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim,
                "kv_rank": self.kv_rank, "q_rank": self.q_rank, "scale": self.scale,
                "rot": {"base": self.rot_base, "dims": self.rot_dim}}

    def spec(self, D: int, eps: float):
        return part("latent_attention", hidden_size=D, num_heads=self.heads, nope_dim=self.dim, rope_dim=self.rot_dim,
                    value_dim=self.vdim, kv_rank=self.kv_rank, query_rank=self.q_rank, query_norm_eps=eps,
                    softmax_scale=self.scale, latent_norm_eps=eps, head_gate=True,
                    position=part("rope_yarn", theta=self.rot_base, rotary_dim=self.rot_dim, pairing="adjacent"))


@dataclasses.dataclass(frozen=True)
class WindowAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int

    @classmethod
    def from_dict(cls, m: Mapping[str, Any], where: str) -> "WindowAttentionConfig":
        _only(m, ("heads", "kv_heads", "dim", "vdim", "scale", "mask"), where)
        mask = _need(m, "mask", where)
        _only(mask, ("size",), where + ".mask")
        heads = int(_need(m, "heads", where))
        dim = int(_need(m, "dim", where))
        c = cls(heads=heads, kv_heads=int(m.get("kv_heads") or heads), dim=dim, vdim=int(m.get("vdim") or dim),
                scale=float(_need(m, "scale", where)), window=int(_need(mask, "size", where + ".mask")))
        _positive(where, heads=c.heads, kv_heads=c.kv_heads, dim=c.dim, vdim=c.vdim)
        _positive(where + ".mask", size=c.window)
        if c.heads % c.kv_heads:
            raise ConfigError(f"config.json: {where}: heads must be a multiple of kv_heads")
        return c

    def to_dict(self) -> dict:
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim,
                "scale": self.scale, "mask": {"size": self.window}}

    def spec(self, D: int, eps: float):
        return part("attention", hidden_size=D, num_heads=self.heads, num_kv_heads=self.kv_heads, head_dim=self.dim,
                    value_dim=self.vdim, softmax_scale=self.scale, retention=("window", self.window),
                    position=part("none"), qk_norm=part("rmsnorm", eps=eps, weighted=True, before_rotation=True),
                    distance_bias=part("log_distance"), head_temperature=True)


@dataclasses.dataclass(frozen=True)
class Mamba2Config:
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    @classmethod
    def from_dict(cls, m: Mapping[str, Any], where: str) -> "Mamba2Config":
        keys = ("heads", "vdim", "state", "groups", "conv", "norm_groups")
        _only(m, keys, where)
        c = cls(**{k: int(_need(m, k, where)) for k in keys})
        _positive(where, **dataclasses.asdict(c))
        if c.heads % c.groups or (c.heads * c.vdim) % c.norm_groups:
            raise ConfigError(f"config.json: {where}: heads must be a multiple of groups, and heads * vdim of norm_groups")
        return c

    def to_dict(self) -> dict:
        return dataclasses.asdict(self)

    @property
    def inner(self) -> int:
        return self.heads * self.vdim

    @property
    def channels(self) -> int:
        return self.inner + 2 * self.groups * self.state

    def spec(self, D: int, eps: float):
        return part("mamba2", hidden_size=D, num_heads=self.heads, value_dim=self.vdim, state_dim=self.state,
                    num_groups=self.groups, conv_taps=self.conv, norm_groups=self.norm_groups, norm_eps=eps)


@dataclasses.dataclass(frozen=True)
class RoutedExpertsConfig:
    experts: int
    top: int
    ff: int
    groups: Optional[int]  # None: every expert can be chosen
    keep: Optional[int]
    identity: int
    scale: float
    shared_ff: Optional[int]  # None: no shared expert

    @classmethod
    def from_dict(cls, m: Mapping[str, Any], where: str) -> "RoutedExpertsConfig":
        _only(m, ("kind", "router", "expert", "shared"), where)
        if m.get("kind", "moe") != "moe":
            raise ConfigError(f"config.json: {where}.kind {m['kind']!r} is not known (moe)")
        router, expert, at = _need(m, "router", where), _need(m, "expert", where), where + ".router"
        _only(router, ("experts", "top", "groups", "identity", "scale"), at)
        _only(expert, ("ff",), where + ".expert")
        groups, shared = router.get("groups"), m.get("shared")
        if groups is not None:
            _only(groups, ("count", "keep"), at + ".groups")
        if shared is not None:
            _only(shared, ("ff",), where + ".shared")
        scale = router.get("scale")
        c = cls(experts=int(_need(router, "experts", at)), top=int(_need(router, "top", at)),
                ff=int(_need(expert, "ff", where + ".expert")),
                groups=None if groups is None else int(_need(groups, "count", at + ".groups")),
                keep=None if groups is None else int(_need(groups, "keep", at + ".groups")),
                identity=int(router.get("identity") or 0), scale=1.0 if scale is None else float(scale),
                shared_ff=None if shared is None else int(_need(shared, "ff", where + ".shared")))
        if not 1 <= c.top <= c.outputs or c.ff < 1 or c.experts < 1 or c.identity < 0 or (c.shared_ff or 1) < 1:
            raise ConfigError(f"config.json: {where}: experts, 1 <= top <= experts + identity and positive widths are needed")
        if c.groups is not None:
            if c.groups < 1 or c.outputs % c.groups or not 1 <= c.keep <= c.groups:
                raise ConfigError(f"config.json: {at}.groups: equal groups and 1 <= keep <= count are needed")
            if c.keep * (c.outputs // c.groups) < c.top:
                raise ConfigError(f"config.json: {at}: the kept groups hold fewer than top experts")
        return c

    @property
    def outputs(self) -> int:
        """The router's rows: the experts and, behind them, the identity experts."""
        return self.experts + self.identity

    def to_dict(self) -> dict:
        router = {"experts": self.experts, "top": self.top, "scale": self.scale}
        if self.identity:
            router["identity"] = self.identity
        if self.groups is not None:
            router["groups"] = {"count": self.groups, "keep": self.keep}
        d = {"kind": "moe", "router": router, "expert": {"ff": self.ff}}
        if self.shared_ff is not None:
            d["shared"] = {"ff": self.shared_ff}
        return d

    def spec(self, D: int):
        return part("moe_scored", hidden_size=D, num_experts=self.experts, top_k=self.top, intermediate_size=self.ff,
                    activation="swiglu", scores="softmax", correction=True, groups=self.groups, keep_groups=self.keep,
                    group_score_terms=GROUP_SCORE_TERMS, identity_experts=self.identity, normalize=WEIGHT_FLOOR,
                    weight_scale=self.scale, shared_intermediate_size=self.shared_ff)


@dataclasses.dataclass(frozen=True)
class FolivikLayerConfig:
    type: str
    mixer: Any
    mlp: Optional[RoutedExpertsConfig]


_MIXERS = {"latent_attention": LatentAttentionConfig, "attention": WindowAttentionConfig, "mamba2": Mamba2Config}


@dataclasses.dataclass(frozen=True)
class FolivikConfig:
    vocab: int
    width: int
    norm_eps: float
    layers: tuple

    @classmethod
    def from_dict(cls, top: Mapping[str, Any]) -> "FolivikConfig":
        _only(top, ("architecture", "architectures", "model_type", "vocab", "width", "norm", "layers"), "the top level")
        layers = []
        for i, entry in enumerate(_need(top, "layers", "the top level")):
            where = f"layers[{i}]"
            _only(entry, ("type", "mixer", "mlp"), where)
            kind = _need(entry, "type", where)
            if kind not in _MIXERS:
                raise ConfigError(f"config.json: {where}.type {kind!r} is not known ({', '.join(sorted(_MIXERS))})")
            mlp = entry.get("mlp")
            layers.append(FolivikLayerConfig(
                kind, _MIXERS[kind].from_dict(_need(entry, "mixer", where), where + ".mixer"),
                None if mlp is None else RoutedExpertsConfig.from_dict(mlp, where + ".mlp")))
        if not layers:
            raise ConfigError("config.json: no layers")
        norm = _need(top, "norm", "the top level")
        _only(norm, ("eps",), "norm")
        return cls(vocab=int(_need(top, "vocab", "the top level")), width=int(_need(top, "width", "the top level")),
                   norm_eps=float(_need(norm, "eps", "norm")), layers=tuple(layers))

    def to_dict(self, architecture: str = "Folivik") -> dict:
        return {"architecture": architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "layers": [{"type": lc.type, "mixer": lc.mixer.to_dict(),
                            "mlp": None if lc.mlp is None else lc.mlp.to_dict()} for lc in self.layers]}

    def plan(self) -> ModelPlan:
        D, eps = self.width, self.norm_eps
        norm = part("rmsnorm", eps=eps, size=D, one_number=True)
        layers = tuple(
            LayerSpec(mixer=lc.mixer.spec(D, eps), feed_forward=None if lc.mlp is None else lc.mlp.spec(D),
                      mixer_norm=norm, feed_forward_norm=norm, arrangement="pre_norm") for lc in self.layers)
        return ModelPlan(vocab_size=self.vocab, hidden_size=D, layers=layers,
                         order=tuple(OrderEntry(layer=i, cache=i) for i in range(len(layers))), final_norm=norm,
                         tie_word_embeddings=False,
                         embedding=part("token_embedding", vocab_size=self.vocab, hidden_size=D),
                         head=part("linear_head", vocab_size=self.vocab, hidden_size=D))
