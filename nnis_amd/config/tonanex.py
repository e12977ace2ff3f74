"""Typed configuration of Tonanex, read from its own config.json keys.

A Tonanex folder names its design in ``architecture`` and gives every size and
constant that may differ between models: ``vocab``, ``width``, ``norm.eps``,
``logit_softcap`` and ``layers``, each with ``type`` (``attention``), the
mixer's sizes in ``mixer`` and its feed-forward in ``mlp``: ``{"kind":
"dense", "ff": n}``, ``{"kind": "moe", "expert": {"ff", "limit"}, "router":
{"experts", "top"}, "shared": {"ff", "limit"}}`` or null (or absent) for none.
A layer with ``weights_of`` uses another layer's tensors with a cache of its
own; the rest of its entry, where it is there, equals that layer's.  No size
has a default: a size that is missing is an error, so that a model never runs
on a guess.  A mechanism that the file does not mention at all does not exist
in that model: without ``logit_softcap`` the logits leave as they are, an
attention without ``mask`` sees every earlier key, experts without ``limit``
hold nothing back, and without ``shared`` there is no shared expert.
"""

from __future__ import annotations

import copy
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from ..errors import InvalidInput, Unsupported
from .zifunex import _get, _int, _number

ARCHITECTURE = "Tonanex"
MIXERS = ("attention",)


@dataclass
class AttentionSizes:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int = 0  # 0: every earlier key is seen

    @classmethod
    def from_dict(cls, raw, where):
        out = cls(_int(raw, "heads", where), _int(raw, "kv_heads", where), _int(raw, "dim", where), _int(raw, "vdim", where),
                  _number(raw, "scale", where))
        if out.heads % out.kv_heads:
            raise InvalidInput(f"config.json {where}: {out.heads} heads do not divide into {out.kv_heads} kv_heads")
        if raw.get("mask") is not None:
            out.window = _int(raw["mask"], "size", where + ".mask")
        return out


@dataclass
class ExpertSizes:
    ff: int
    limit: Optional[float] = None  # None: nothing is held back

    @classmethod
    def from_dict(cls, raw, where):
        return cls(_int(raw, "ff", where), _number(raw, "limit", where) if raw.get("limit") is not None else None)


@dataclass
class RouterSizes:
    experts: int
    top: int
    expert: ExpertSizes
    shared: Optional[ExpertSizes] = None


@dataclass
class LayerSizes:
    type: str
    attention: AttentionSizes
    ff: Optional[int] = None  # a dense feed-forward's inner size
    router: Optional[RouterSizes] = None  # a mixture of experts


def _layer(layer, where) -> LayerSizes:
    kind, mixer = _get(layer, "type", where), _get(layer, "mixer", where)
    if kind not in MIXERS:
        raise Unsupported(f"config.json {where}.type {kind!r}; this design has the mixers {', '.join(MIXERS)}")
    out = LayerSizes(kind, AttentionSizes.from_dict(mixer, where + ".mixer"))
    mlp, spot = layer.get("mlp"), where + ".mlp"  # (absent or null: the layer has no feed-forward)
    if mlp is None:
        return out
    form = _get(mlp, "kind", spot)
    if form == "dense":
        out.ff = _int(mlp, "ff", spot)
    elif form == "moe":
        router = _get(mlp, "router", spot)
        out.router = RouterSizes(
            _int(router, "experts", spot + ".router"), _int(router, "top", spot + ".router"),
            ExpertSizes.from_dict(_get(mlp, "expert", spot), spot + ".expert"),
            ExpertSizes.from_dict(mlp["shared"], spot + ".shared") if mlp.get("shared") is not None else None)
        if out.router.top > out.router.experts:
            raise InvalidInput(f"config.json {spot}.router: the {out.router.top} largest of {out.router.experts} outputs")
    else:
        raise Unsupported(f"config.json {spot}.kind {form!r}; this design has dense and moe feed-forwards")
    return out


def _owners(layers) -> List[int]:
    """For each layer the one whose tensors it uses: itself, or where ``weights_of`` leads."""
    out = []
    for index, layer in enumerate(layers):
        at, passed = index, {index}
        while isinstance(layers[at], dict) and layers[at].get("weights_of") is not None:
            at = _int(layers[at], "weights_of", f"layers[{at}]", least=0)
            if at >= len(layers) or at in passed:
                raise InvalidInput(f"config.json layers[{index}].weights_of must lead to a layer with tensors of its own; got {layer['weights_of']}")
            passed.add(at)
        out.append(at)
    return out


@dataclass
class TonanexConfig:
    vocab: int
    width: int
    eps: float
    logit_softcap: float  # 0: logits leave as they are
    layers: List[LayerSizes]
    owners: List[int]  # for each layer the index of the layer whose tensors it uses
    raw: Dict[str, Any] = field(default_factory=dict)
    architecture: str = ARCHITECTURE

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "TonanexConfig":
        layers = _get(raw, "layers", "file")
        if not isinstance(layers, list) or not layers:
            raise InvalidInput("config.json layers must be a list with at least one layer")
        owners = _owners(layers)
        sizes = []
        for index, owner in enumerate(owners):
            if owner != index:
                for key in ("type", "mixer", "mlp"):
                    if key in layers[index] and layers[index][key] != layers[owner].get(key):
                        raise InvalidInput(f"config.json layers[{index}] uses layer {owner}'s tensors, but its {key!r} is another one")
            sizes.append(_layer(layers[owner], f"layers[{owner}]"))
        return cls(
            vocab=_int(raw, "vocab", "file"), width=_int(raw, "width", "file"), eps=_number(_get(raw, "norm", "file"), "eps", "norm"),
            logit_softcap=_number(raw, "logit_softcap", "file") if raw.get("logit_softcap") is not None else 0.0,
            layers=sizes, owners=owners, raw=copy.deepcopy(raw))

    def to_dict(self) -> Dict[str, Any]:
        return copy.deepcopy(self.raw)
