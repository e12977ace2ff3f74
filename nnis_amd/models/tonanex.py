"""Tonanex as a model description.  A pre-norm decoder with RMS norms, one of
them behind the embedding, whose mixer is grouped attention without a rotation
in a sliding window: queries and keys head by head over their root mean
square, a temperature a head, scores that fall with the logarithm of the
distance, a sigmoid gate a head on its output; whose feed-forward is gated by
SiLU, or a mixture of clamped experts weighted by the softmax over the chosen
logits beside a shared expert, or absent; whose embedding table is its head,
with capped logits.  A layer may run again with its weights at other places of
the order, every run with a cache of its own.  Tensor names are the
checkpoint's: layer i's start with ``l<i>.``.
"""

from __future__ import annotations

from ..config.tonanex import TonanexConfig
from .spec import ModelSpec, ScheduleEntry


def _norm(cfg: TonanexConfig, name: str):
    return {"kind": "rms", "width": cfg.width, "eps": cfg.eps, "weight": name}


def _attention(cfg: TonanexConfig, prefix: str, sizes):
    return {"kind": "causal_attention", "width": cfg.width, "heads": sizes.heads, "kv_heads": sizes.kv_heads, "head_dim": sizes.dim,
            "value_dim": sizes.vdim, "scale": sizes.scale, "window": sizes.window or None, "unit_heads": cfg.eps,
            "temperature": prefix + "temp", "decay": (prefix + "r1", prefix + "r2"), "head_gate": prefix + "g",
            "q": prefix + "q", "k": prefix + "k", "v": prefix + "v", "o": prefix + "o"}


def _feed_forward(cfg: TonanexConfig, prefix: str, layer):
    if layer.ff is not None:
        return {"kind": "gated", "width": cfg.width, "inner": layer.ff, "gate": prefix + "gate", "up": prefix + "up", "down": prefix + "down"}
    router = layer.router
    out = {"kind": "routed", "width": cfg.width, "inner": router.expert.ff, "limit": router.expert.limit, "experts": router.experts,
           "top": router.top, "scoring": "chosen_softmax", "activation": "clamped_swiglu", "router": prefix + "router",
           "router_bias": prefix + "router.b", "gate": prefix + "e{}.gate", "up": prefix + "e{}.up", "down": prefix + "e{}.down"}
    if router.shared is not None:
        out["shared"] = {"inner": router.shared.ff, "limit": router.shared.limit, "gate": prefix + "shared.gate",
                         "up": prefix + "shared.up", "down": prefix + "shared.down"}
    return out


def tonanex_spec(cfg: TonanexConfig) -> ModelSpec:
    layers, place = [], {}  # place: where the block of a layer with tensors of its own stands
    for index, layer in enumerate(cfg.layers):
        if cfg.owners[index] != index:
            continue
        prefix = f"l{index}."
        block = {"kind": "pre_norm", "width": cfg.width, "norm1": _norm(cfg, prefix + "norm1"),
                 "mixer": _attention(cfg, prefix + "mix.", layer.attention)}
        if layer.ff is not None or layer.router is not None:
            block.update(norm2=_norm(cfg, prefix + "norm2"), feed_forward=_feed_forward(cfg, prefix + "mlp.", layer))
        place[index] = len(layers)
        layers.append(block)
    spec = ModelSpec(
        architecture=cfg.architecture,
        width=cfg.width,
        vocab_size=cfg.vocab,
        max_positions=None,  # the design names no last position
        stored_dtype="bfloat16",
        embedding={"kind": "table", "vocab_size": cfg.vocab, "width": cfg.width, "weight": "embed", "norm": _norm(cfg, "embed.norm")},
        positions={},
        layers=layers,
        schedule=[ScheduleEntry(layer=place[owner]) for owner in cfg.owners],  # every run keeps a cache of its own
        final_norm=_norm(cfg, "final.norm"),
        head={"kind": "linear", "vocab_size": cfg.vocab, "width": cfg.width, "weight": "embed", "softcap": cfg.logit_softcap or None},
        stop_token_ids=(),
        config_json=cfg.to_dict(),
    )
    spec.validate()
    return spec
