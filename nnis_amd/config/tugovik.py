"""Typed configuration of Tugovik, read from its own config.json keys.

A Tugovik folder names its design in ``architecture`` and gives every size and
constant that may differ between models: ``vocab``, ``width``, ``norm.eps``
and ``layers``, each with ``type`` (``attention``, ``mamba2`` or ``rglru``),
the mixer's sizes in ``mixer`` and its feed-forward in ``mlp``: ``{"kind":
"moe", "expert": {"ff"}, "router": {"experts", "top", "scale", "groups":
{"count", "keep"}}, "shared": {"ff"}}`` or null (or absent) for none.  No size
has a default: a size that is missing is an error, so that a model never runs
on a guess.  A mechanism that the file does not mention at all does not exist
in that model: without ``loop`` every layer runs once, without ``token_side``
tokens have no input of their own in the layers, an attention without ``mask``
sees every earlier key, a router without ``groups`` chooses among all its
experts and one without ``scale`` leaves its weights as they are, and without
``shared`` there is no shared expert.
"""

from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Tuple

from ..errors import InvalidInput, Unsupported
from .mafalorn import _real
from .zifunex import _get, _int, _number

ARCHITECTURE = "Tugovik"
MIXERS = ("attention", "mamba2", "rglru")


@dataclass
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int = 0  # 0: every earlier key is seen

    @classmethod
    def from_dict(cls, raw, where):
        out = cls(_int(raw, "heads", where), _int(raw, "kv_heads", where), _int(raw, "dim", where), _int(raw, "vdim", where),
                  _number(raw, "scale", where))
        if out.heads % out.kv_heads:
            raise InvalidInput(f"config.json {where}: {out.heads} heads do not divide into {out.kv_heads} kv_heads")
        if raw.get("mask") is not None:
            out.chunk = _int(raw["mask"], "size", where + ".mask")
        return out


@dataclass
class StateSpaceSizes:
    heads: int
    vdim: int
    state: int
    groups: int
    conv: int
    norm_groups: int

    @classmethod
    def from_dict(cls, raw, where):
        out = cls(*(_int(raw, key, where) for key in ("heads", "vdim", "state", "groups", "conv", "norm_groups")))
        if out.heads % out.groups:
            raise InvalidInput(f"config.json {where}: {out.heads} heads do not divide into {out.groups} groups")
        if out.heads * out.vdim % out.norm_groups:
            raise InvalidInput(f"config.json {where}: {out.heads} heads of {out.vdim} do not divide into {out.norm_groups} norm_groups")
        return out


@dataclass
class UnitSizes:
    width: int
    blocks: int
    conv: int

    @classmethod
    def from_dict(cls, raw, where):
        out = cls(_int(raw, "width", where), _int(raw, "blocks", where), _int(raw, "conv", where))
        if out.width % out.blocks:
            raise InvalidInput(f"config.json {where}: a width of {out.width} does not divide into {out.blocks} blocks")
        return out


@dataclass
class RouterSizes:
    experts: int
    top: int
    scale: float
    expert_ff: int
    shared_ff: int = 0  # 0: no shared expert
    groups: Optional[Tuple[int, int]] = None  # (count, keep)


@dataclass
class LayerSizes:
    type: str
    attention: Optional[AttentionSizes] = None
    space: Optional[StateSpaceSizes] = None
    unit: Optional[UnitSizes] = None
    router: Optional[RouterSizes] = None


def _router(mlp, where) -> RouterSizes:
    form = _get(mlp, "kind", where)
    if form != "moe":
        raise Unsupported(f"config.json {where}.kind {form!r}; this design's feed-forward is a mixture of experts (moe)")
    router, spot = _get(mlp, "router", where), where + ".router"
    out = RouterSizes(_int(router, "experts", spot), _int(router, "top", spot),
                      _real(router, "scale", spot) if router.get("scale") is not None else 1.0,
                      _int(_get(mlp, "expert", where), "ff", where + ".expert"),
                      _int(mlp["shared"], "ff", where + ".shared") if mlp.get("shared") is not None else 0)
    if out.top > out.experts:
        raise InvalidInput(f"config.json {spot}: the {out.top} largest of {out.experts} outputs")
    groups = router.get("groups")
    if groups is not None:
        count, keep = _int(groups, "count", spot + ".groups"), _int(groups, "keep", spot + ".groups")
        if out.experts % count or keep > count or out.top > keep * (out.experts // count):
            raise InvalidInput(f"config.json {spot}.groups: {out.experts} experts in {count} equal groups of which {keep} are kept "
                               f"must leave {out.top} to choose")
        if count > 1:
            out.groups = (count, keep)
    return out


def _layer(layer, where) -> LayerSizes:
    kind, mixer = _get(layer, "type", where), _get(layer, "mixer", where)
    spot = where + ".mixer"
    if kind == "attention":
        out = LayerSizes(kind, attention=AttentionSizes.from_dict(mixer, spot))
    elif kind == "mamba2":
        out = LayerSizes(kind, space=StateSpaceSizes.from_dict(mixer, spot))
    elif kind == "rglru":
        out = LayerSizes(kind, unit=UnitSizes.from_dict(mixer, spot))
    else:
        raise Unsupported(f"config.json {where}.type {kind!r}; this design has the mixers {', '.join(MIXERS)}")
    if layer.get("mlp") is not None:  # (absent or null: the layer has no feed-forward)
        out.router = _router(layer["mlp"], where + ".mlp")
    return out


@dataclass
class TugovikConfig:
    vocab: int
    width: int
    eps: float
    layers: List[LayerSizes]
    loop: Optional[Tuple[int, int, int]] = None  # (start, stop, times)
    side_dim: int = 0  # 0: tokens have no input of their own in the layers
    raw: Dict[str, Any] = field(default_factory=dict)
    architecture: str = ARCHITECTURE

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "TugovikConfig":
        layers = _get(raw, "layers", "file")
        if not isinstance(layers, list) or not layers:
            raise InvalidInput("config.json layers must be a list with at least one layer")
        loop = None
        if raw.get("loop") is not None:
            start, stop, times = _int(raw["loop"], "start", "loop", least=0), _int(raw["loop"], "stop", "loop"), _int(raw["loop"], "times", "loop")
            if not start < stop <= len(layers):
                raise InvalidInput(f"config.json loop: layers {start} up to {stop} of {len(layers)}")
            loop = (start, stop, times)
        return cls(
            vocab=_int(raw, "vocab", "file"), width=_int(raw, "width", "file"), eps=_number(_get(raw, "norm", "file"), "eps", "norm"),
            layers=[_layer(layer, f"layers[{index}]") for index, layer in enumerate(layers)], loop=loop,
            side_dim=_int(raw["token_side"], "dim", "token_side") if raw.get("token_side") is not None else 0,
            raw=copy.deepcopy(raw))

    def order(self) -> List[int]:
        """The layers as they run."""
        indices = list(range(len(self.layers)))
        if self.loop is None:
            return indices
        start, stop, times = self.loop
        return indices[:start] + indices[start:stop] * times + indices[stop:]

    def to_dict(self) -> Dict[str, Any]:
        return copy.deepcopy(self.raw)
