"""Typed configuration of the Vipalorn decoder, read from its config.json.

Vipalorn lists its layers one by one; a layer names one of two mixers, that mixer's sizes and constants, and a routed
feed-forward (or none). Nothing about a layer is assumed from another layer. Keys read:

    architecture          "Vipalorn"
    vocab, width          sizes of the embedding table / the residual stream
    norm.eps              the eps of every norm
    residual_mult         factor on what a layer adds to the stream (default 1)
    logit_scale           factor on the logits (default 1)
    max_positions         optional: the longest sequence (default 131072; the design itself has no limit)
    layers[i].type        "latent_attention" or "delta"
    layers[i].mixer       latent_attention: heads, dim, rot_dim, vdim (default dim), kv_rank, scale,
                                            rot.{dims (default rot_dim), base}
                          delta: heads, kv_heads (default heads), dim, vdim (default dim), conv (default 1: a factor a
                                 channel)
    layers[i].mlp         null, or kind "moe" with expert.{ff, limit} and router.{experts, top}
"""

from __future__ import annotations

import dataclasses
from typing import Any, Mapping, Optional, Tuple

from ..errors import LoadError, UnsupportedError
from .base import ConfigReader
from .duzozen import DEFAULT_MAX_POSITIONS, _section
from .minerax import DeltaRuleConfig, _positive


@dataclasses.dataclass(frozen=True)
class RotationConfig:
    dims: int                     # the first ``dims`` dimensions of the rotated part rotate
    base: float


@dataclasses.dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int                      # unrotated query / key dimensions of a head
    rot_dim: int                  # rotated ones; the key's are shared by all heads
    vdim: int
    kv_rank: int                  # size of the cached latent
    scale: float
    rotation: RotationConfig


@dataclasses.dataclass(frozen=True)
class RoutedFfConfig:
    ff: int                       # inner size of an expert
    limit: float                  # where an expert's gate and up sums are cut off
    experts: int
    top: int


@dataclasses.dataclass(frozen=True)
class VipalornLayerConfig:
    kind: str                     # "latent_attention", "delta"
    mixer: Any
    mlp: Optional[RoutedFfConfig]


@dataclasses.dataclass(frozen=True)
class VipalornConfig:
    vocab: int
    width: int
    norm_eps: float
    residual_mult: float
    logit_scale: float
    max_positions: int
    layers: Tuple[VipalornLayerConfig, ...]

    @staticmethod
    def _latent(r: ConfigReader, where: str) -> LatentAttentionConfig:
        heads, dim, rot_dim = r.integer("heads"), r.integer("dim"), r.integer("rot_dim")
        vdim, kv_rank, scale = r.integer("vdim", dim), r.integer("kv_rank"), r.number("scale")
        _positive(where, heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale)
        rot = _section(r, "rot", where)
        dims, base = rot.integer("dims", rot_dim), rot.number("base")
        if dims <= 0 or dims % 2 or dims > rot_dim:
            raise LoadError(f"config.json: {where} rotates {dims} dimensions of {rot_dim}: an even number up to that is "
                            f"needed")
        _positive(where + " rot", base=base)
        return LatentAttentionConfig(heads, dim, rot_dim, vdim, kv_rank, scale, RotationConfig(dims, base))

    @staticmethod
    def _delta(r: ConfigReader, where: str) -> DeltaRuleConfig:
        heads = r.integer("heads")
        kv_heads, dim = r.integer("kv_heads", heads), r.integer("dim")
        vdim, conv = r.integer("vdim", dim), r.integer("conv", 1)
        _positive(where, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)
        if heads % kv_heads:
            raise LoadError(f"config.json: {where} has {heads} value heads, no multiple of {kv_heads} query/key heads")
        return DeltaRuleConfig(heads, kv_heads, dim, vdim, conv)

    @staticmethod
    def _mlp(r: Optional[ConfigReader], where: str) -> Optional[RoutedFfConfig]:
        if r is None:
            return None
        kind = r.string("kind")
        if kind != "moe":
            raise UnsupportedError(f"config.json: {where} has a feed-forward of kind '{kind}' (supported: moe)")
        where += " mlp"
        expert, router = _section(r, "expert", where), _section(r, "router", where)
        ff, limit = expert.integer("ff"), expert.number("limit")
        experts, top = router.integer("experts"), router.integer("top")
        _positive(where, ff=ff, limit=limit, experts=experts, top=top)
        if top > experts:
            raise LoadError(f"config.json: {where} chooses {top} of {experts} experts: no such choice")
        return RoutedFfConfig(ff, limit, experts, top)

    @classmethod
    def from_json(cls, values: Mapping[str, Any]) -> "VipalornConfig":
        r = ConfigReader(values)
        vocab, width = r.integer("vocab"), r.integer("width")
        eps = _section(r, "norm", "the model").number("eps")
        _positive("the model", vocab=vocab, width=width, eps=eps)
        residual_mult, logit_scale = r.number("residual_mult", 1.0), r.number("logit_scale", 1.0)
        entries = r.raw("layers")
        if not isinstance(entries, list) or not entries:
            raise LoadError("config.json: 'layers' must be a non-empty list")
        readers = {"latent_attention": cls._latent, "delta": cls._delta}
        layers = []
        for i, entry in enumerate(entries):
            where = f"layer {i}"
            if not isinstance(entry, Mapping):
                raise LoadError(f"config.json: {where} must be an object")
            layer = ConfigReader(entry, f"config.json {where}")
            kind = layer.string("type")
            if kind not in readers:
                raise UnsupportedError(f"config.json: {where} has a mixer of type '{kind}' "
                                       f"(supported: {', '.join(sorted(readers))})")
            mixer = readers[kind](_section(layer, "mixer", where), where)
            layers.append(VipalornLayerConfig(kind, mixer, cls._mlp(_section(layer, "mlp", where, required=False), where)))
        max_positions = r.integer("max_positions", DEFAULT_MAX_POSITIONS)
        _positive("the model", max_positions=max_positions)
        return cls(vocab, width, eps, residual_mult, logit_scale, max_positions, tuple(layers))
