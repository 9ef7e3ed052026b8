"""Typed configuration of the Vosurax decoder, read from its config.json.

Vosurax lists its layers one by one; a layer names one of two mixers, that mixer's sizes and constants, and a feed-forward
(or none). Nothing about a layer is assumed from another layer. Keys read:

    architecture          "Vosurax"
    vocab, width          sizes of the embedding table / the residual stream
    norm.eps              the eps of every RMS norm
    loop                  optional: layers start .. stop - 1 run ``times`` times in a row
    max_positions         optional: the longest sequence (default 131072; the design itself has no limit)
    layers[i].type        "parallel" or "retention"
    layers[i].mixer       parallel: left  {heads, kv_heads (default heads), dim, vdim (default dim), scale,
                                           mask.size (optional: causal chunks)}
                                    right {heads, dim, vdim (default dim), gate_cap}
                          retention: heads, dim, vdim (default dim), decay (one number a head),
                                     rot.{dims (default dim), base}
    layers[i].mlp         null; kind "dense" with ff; or kind "moe" with expert.ff, router.{experts, top} and
                          shared.ff (optional)
"""

from __future__ import annotations

import dataclasses
import math
from typing import Any, Mapping, Optional, Tuple

from ..errors import LoadError, UnsupportedError
from .base import ConfigReader
from .duzozen import DEFAULT_MAX_POSITIONS, _section
from .minerax import _positive


@dataclasses.dataclass(frozen=True)
class ChunkedAttentionConfig:
    heads: int
    kv_heads: int
    dim: int                      # size of a query / key head
    vdim: int                     # size of a value head
    scale: float
    chunk: Optional[int]          # positions of a causal chunk; None: every earlier key is seen


@dataclasses.dataclass(frozen=True)
class MatrixMemoryConfig:
    heads: int
    dim: int
    vdim: int
    gate_cap: float               # what the gates' arguments are capped at


@dataclasses.dataclass(frozen=True)
class ParallelMixerConfig:
    left: ChunkedAttentionConfig
    right: MatrixMemoryConfig


@dataclasses.dataclass(frozen=True)
class RotationConfig:
    dims: int                     # the first ``dims`` dimensions of a head rotate
    base: float


@dataclasses.dataclass(frozen=True)
class RetentionConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]      # one factor a head
    rotation: RotationConfig


@dataclasses.dataclass(frozen=True)
class DenseFfConfig:
    ff: int


@dataclasses.dataclass(frozen=True)
class RoutedFfConfig:
    ff: int                       # inner size of an expert
    experts: int
    top: int
    shared_ff: Optional[int]      # inner size of the expert every token uses; None: there is none


@dataclasses.dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int


@dataclasses.dataclass(frozen=True)
class VosuraxLayerConfig:
    kind: str                     # "parallel", "retention"
    mixer: Any
    mlp: Any                      # None, DenseFfConfig or RoutedFfConfig


@dataclasses.dataclass(frozen=True)
class VosuraxConfig:
    vocab: int
    width: int
    norm_eps: float
    max_positions: int
    layers: Tuple[VosuraxLayerConfig, ...]
    loop: Optional[LoopConfig]

    @staticmethod
    def _parallel(r: ConfigReader, where: str) -> ParallelMixerConfig:
        at = where + " left"
        left = _section(r, "left", where)
        heads, dim = left.integer("heads"), left.integer("dim")
        kv_heads, vdim, scale = left.integer("kv_heads", heads), left.integer("vdim", dim), left.number("scale")
        _positive(at, heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
        if heads % kv_heads:
            raise LoadError(f"config.json: {at} has {heads} query heads, no multiple of {kv_heads} key/value heads")
        mask = _section(left, "mask", at, required=False)
        chunk = mask.integer("size", None) if mask is not None else None
        if chunk is not None:
            _positive(at + " mask", size=chunk)
        at = where + " right"
        right = _section(r, "right", where)
        memory = MatrixMemoryConfig(right.integer("heads"), right.integer("dim"),
                                    right.integer("vdim", right.integer("dim")), right.number("gate_cap"))
        _positive(at, **dataclasses.asdict(memory))
        return ParallelMixerConfig(ChunkedAttentionConfig(heads, kv_heads, dim, vdim, scale, chunk), memory)

    @staticmethod
    def _retention(r: ConfigReader, where: str) -> RetentionConfig:
        heads, dim = r.integer("heads"), r.integer("dim")
        vdim = r.integer("vdim", dim)
        _positive(where, heads=heads, dim=dim, vdim=vdim)
        decay = r.raw("decay")
        if not isinstance(decay, list) or len(decay) != heads or \
                not all(isinstance(x, (int, float)) and not isinstance(x, bool) and math.isfinite(x) and x >= 0
                        for x in decay):
            raise LoadError(f"config.json: {where} decay must list one number (not negative) for each of the {heads} heads")
        rot = _section(r, "rot", where)
        dims, base = rot.integer("dims", dim), rot.number("base")
        if dims <= 0 or dims % 2 or dims > dim:
            raise LoadError(f"config.json: {where} rotates {dims} dimensions of {dim}: an even number up to that is needed")
        _positive(where + " rot", base=base)
        return RetentionConfig(heads, dim, vdim, tuple(float(x) for x in decay), RotationConfig(dims, base))

    @staticmethod
    def _mlp(r: Optional[ConfigReader], where: str):
        if r is None:
            return None
        kind = r.string("kind")
        where += " mlp"
        if kind == "dense":
            ff = r.integer("ff")
            _positive(where, ff=ff)
            return DenseFfConfig(ff)
        if kind != "moe":
            raise UnsupportedError(f"config.json: {where} is of kind '{kind}' (supported: dense, moe)")
        expert, router = _section(r, "expert", where), _section(r, "router", where)
        ff, experts, top = expert.integer("ff"), router.integer("experts"), router.integer("top")
        _positive(where, ff=ff, experts=experts, top=top)
        if top > experts:
            raise LoadError(f"config.json: {where} chooses {top} of {experts} experts: no such choice")
        shared = _section(r, "shared", where, required=False)
        shared_ff = shared.integer("ff") if shared is not None else None
        if shared_ff is not None:
            _positive(where + " shared", ff=shared_ff)
        return RoutedFfConfig(ff, experts, top, shared_ff)

    @classmethod
    def from_json(cls, values: Mapping[str, Any]) -> "VosuraxConfig":
        r = ConfigReader(values)
        vocab, width = r.integer("vocab"), r.integer("width")
        eps = _section(r, "norm", "the model").number("eps")
        _positive("the model", vocab=vocab, width=width, eps=eps)
        entries = r.raw("layers")
        if not isinstance(entries, list) or not entries:
            raise LoadError("config.json: 'layers' must be a non-empty list")
        readers = {"parallel": cls._parallel, "retention": cls._retention}
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
            layers.append(VosuraxLayerConfig(kind, mixer, cls._mlp(_section(layer, "mlp", where, required=False), where)))
        loop = _section(r, "loop", "the model", required=False)
        passes = None
        if loop is not None:
            passes = LoopConfig(loop.integer("start"), loop.integer("stop"), loop.integer("times"))
            if not 0 <= passes.start < passes.stop <= len(layers) or passes.times < 1:
                raise LoadError(f"config.json: a loop over layers {passes.start} .. {passes.stop - 1} of {len(layers)}, "
                                f"{passes.times} times, cannot run")
        max_positions = r.integer("max_positions", DEFAULT_MAX_POSITIONS)
        _positive("the model", max_positions=max_positions)
        return cls(vocab, width, eps, max_positions, tuple(layers), passes)
