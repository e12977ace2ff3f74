"""Tugovik as a model description.  A pre-norm decoder with RMS norms whose
weights lie around zero; whose mixers are grouped attention without a rotation
inside chunks of the sequence, Mamba-2 (a matrix state a head with one decay a
head and token, behind a short convolution, gated before a norm in parts), or
a real-gated linear recurrent unit beside a GELU branch; whose feed-forward is
a mixture of SiLU-gated experts with sigmoid scores, chosen among the best
groups, beside a shared expert with a gate of its own; where every token has
an input of its own in every layer, gated by the stream and normed on its way
into it.  A stretch of layers may run several times in a row with the same
weights, every run with a cache or state of its own.  Tensor names are the
checkpoint's: layer i's start with ``l<i>.``.
"""

from __future__ import annotations

from ..config.tugovik import TugovikConfig
from .spec import ModelSpec, ScheduleEntry


def _norm(cfg: TugovikConfig, name: str):
    return {"kind": "rms", "width": cfg.width, "eps": cfg.eps, "weight": name, "offset": 1.0}


def _attention(cfg, prefix, sizes):
    return {"kind": "causal_attention", "width": cfg.width, "heads": sizes.heads, "kv_heads": sizes.kv_heads, "head_dim": sizes.dim,
            "value_dim": sizes.vdim, "scale": sizes.scale, "chunk": sizes.chunk or None,
            "q": prefix + "q", "k": prefix + "k", "v": prefix + "v", "o": prefix + "o",
            "q_bias": prefix + "q.b", "k_bias": prefix + "k.b", "v_bias": prefix + "v.b"}


def _state_space(cfg, prefix, sizes):
    return {"kind": "mamba2", "width": cfg.width, "heads": sizes.heads, "value_dim": sizes.vdim, "states": sizes.state,
            "groups": sizes.groups, "taps": sizes.conv, "norm_parts": sizes.norm_groups, "eps": cfg.eps,
            "w_in": prefix + "in", "conv": prefix + "conv", "conv_bias": prefix + "conv.b", "dt_bias": prefix + "dt_bias",
            "a_log": prefix + "A_log", "d": prefix + "D", "norm": prefix + "norm", "w_out": prefix + "o"}


def _unit(cfg, prefix, sizes):
    return {"kind": "rg_lru", "width": cfg.width, "channels": sizes.width, "blocks": sizes.blocks, "taps": sizes.conv,
            "y": prefix + "y", "y_bias": prefix + "y.b", "x": prefix + "x", "x_bias": prefix + "x.b",
            "conv": prefix + "conv", "conv_bias": prefix + "conv.b", "r": prefix + "ra", "r_bias": prefix + "ra.b",
            "i": prefix + "ri", "i_bias": prefix + "ri.b", "rate": prefix + "lam", "o": prefix + "o"}


def _feed_forward(cfg, prefix, router):
    out = {"kind": "routed", "width": cfg.width, "inner": router.expert_ff, "experts": router.experts, "top": router.top,
           "groups": router.groups, "group_marks": 2, "scoring": "sigmoid", "weight_scale": router.scale, "activation": "silu_gated",
           "router": prefix + "router", "gate": prefix + "e{}.gate", "up": prefix + "e{}.up", "down": prefix + "e{}.down"}
    if router.shared_ff:
        out["shared"] = {"inner": router.shared_ff, "gate": prefix + "shared.gate", "up": prefix + "shared.up",
                         "down": prefix + "shared.down", "weight": prefix + "shared.sg"}
    return out


def _side(cfg, prefix, index):
    return {"norm": {"kind": "rms", "width": cfg.width, "eps": cfg.eps, "weight": prefix + "norm", "wide": True},
            "part": {"kind": "token_input", "width": cfg.width, "inner": cfg.side_dim, "vocab_size": cfg.vocab,
                     "table": "side.embed", "columns": len(cfg.layers) * cfg.side_dim, "first": index * cfg.side_dim,
                     "gate": prefix + "gate", "proj": prefix + "proj"}}


def tugovik_spec(cfg: TugovikConfig) -> ModelSpec:
    layers = []
    for index, layer in enumerate(cfg.layers):
        prefix = f"l{index}."
        if layer.type == "attention":
            mixer = _attention(cfg, prefix + "mix.", layer.attention)
        elif layer.type == "mamba2":
            mixer = _state_space(cfg, prefix + "mix.", layer.space)
        else:
            mixer = _unit(cfg, prefix + "mix.", layer.unit)
        block = {"kind": "pre_norm", "width": cfg.width, "norm1": _norm(cfg, prefix + "norm1"), "mixer": mixer}
        if layer.router is not None:
            block.update(norm2=_norm(cfg, prefix + "norm2"), feed_forward=_feed_forward(cfg, prefix + "mlp.", layer.router))
        if cfg.side_dim:
            block["side"] = _side(cfg, prefix + "side.", index)
        layers.append(block)
    spec = ModelSpec(
        architecture=cfg.architecture,
        width=cfg.width,
        vocab_size=cfg.vocab,
        max_positions=None,  # the design names no last position
        stored_dtype="bfloat16",
        embedding={"kind": "table", "vocab_size": cfg.vocab, "width": cfg.width, "weight": "embed"},
        positions={},
        layers=layers,
        schedule=[ScheduleEntry(layer=index) for index in cfg.order()],  # every run keeps a cache or state of its own
        final_norm=_norm(cfg, "final.norm"),
        head={"kind": "linear", "vocab_size": cfg.vocab, "width": cfg.width, "weight": "head"},
        stop_token_ids=(),
        config_json=cfg.to_dict(),
    )
    spec.validate()
    return spec
