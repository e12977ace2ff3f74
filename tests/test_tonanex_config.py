"""Tonanex on the CPU: its configuration reader, its model description, and the
plain implementation's own mechanisms against special cases."""

import json
import math

import pytest
import torch

import nnis_amd
import plain_tonanex as T
from nnis_amd.config.registry import spec_from_config
from nnis_amd.errors import InvalidInput, Unsupported
from nnis_amd.kernels import lib
from nnis_amd.models.decoder import DecoderModel
from nnis_amd.parts import build_part
from nnis_amd.parts.base import KVRequest
from tonanex_configs import TON_A, TON_B, TON_C, TONANEX_CONFIGS, again, attention, dense, layer, moe, tonanex


def test_the_architecture_is_chosen_by_its_name():
    cfg, spec = spec_from_config(TON_A)
    assert spec.architecture == "Tonanex" and spec.width == 96 and spec.vocab_size == 300 and spec.max_positions is None
    assert "Tonanex" in nnis_amd.config.registered_architectures()
    assert cfg.logit_softcap == 9.0 and spec.head["softcap"] == 9.0 and spec.head["weight"] == "embed"
    assert spec.embedding["norm"] == {"kind": "rms", "width": 96, "eps": 1e-5, "weight": "embed.norm"}
    assert spec_from_config(TON_B)[1].head["softcap"] is None
    with pytest.raises(Unsupported):
        spec_from_config(dict(TON_A, architecture="Tonanex2"))


def test_layers_run_in_order_with_the_tensors_they_name():
    _, spec = spec_from_config(TON_A)
    assert [e.layer for e in spec.schedule] == [0, 1, 0, 2, 1] and all(e.reads_cache_of is None for e in spec.schedule)
    assert len(spec.layers) == 3 and "feed_forward" not in spec.layers[1] and "norm2" not in spec.layers[1]
    names = {t.name: t.shape for t in DecoderModel(spec).tensors()}
    assert names["l0.mix.q"] == (128, 96) and names["l0.mix.v"] == (32, 96) and names["l0.mix.g"] == (4, 96) and names["l0.mix.o"] == (96, 64)
    assert names["l0.mix.temp"] == names["l0.mix.r1"] == names["l0.mix.r2"] == (4,)
    assert names["l0.mlp.router"] == (5, 96) and names["l0.mlp.router.b"] == (5,) and names["l0.mlp.e4.down"] == (96, 24)
    assert names["l0.mlp.shared.up"] == (40, 96) and "l0.mlp.e5.up" not in names and names["l3.mlp.gate"] == (136, 96)
    assert not any(name.startswith(("l2.", "l4.", "l1.mlp", "l1.norm2")) for name in names) and names["embed.norm"] == (96,)
    requests, shared = DecoderModel(spec).cache_requests()
    assert not shared and [r[1] for r in requests] == [KVRequest(2, 32, 37, 16), KVRequest(1, 16, 70, 48), KVRequest(2, 32, 37, 16),
                                                       KVRequest(1, 16, None, 48), KVRequest(1, 16, 70, 48)]  # every run has a cache of its own
    _, spec = spec_from_config(TON_C)  # layers 0 and 3 use the tensors of layer 2
    assert [e.layer for e in spec.schedule] == [1, 0, 1, 1]
    assert {t.name.split(".")[0] for t in DecoderModel(spec).tensors()} == {"embed", "l1", "l2", "final"}
    _, spec = spec_from_config(TON_B)
    ff = [block["feed_forward"] for block in spec.layers]
    assert ff[1]["limit"] is None and "shared" not in ff[1] and ff[2]["shared"]["limit"] == 2.5 and ff[0]["kind"] == "gated"


def test_missing_and_wrong_keys_are_refused():
    for path in (["vocab"], ["norm", "eps"], ["layers", 0, "mixer", "heads"], ["layers", 0, "mixer", "scale"], ["layers", 0, "mixer", "vdim"],
                 ["layers", 0, "mixer", "mask", "size"], ["layers", 3, "mlp", "ff"], ["layers", 0, "mlp", "router", "top"],
                 ["layers", 0, "mlp", "expert"], ["layers", 0, "mlp", "shared", "ff"], ["layers", 1, "type"]):
        raw = json.loads(json.dumps(TON_A))
        at = raw
        for key in path[:-1]:
            at = at[key]
        del at[path[-1]]
        with pytest.raises(InvalidInput):
            spec_from_config(raw)
    for change, error in ((lambda raw: raw["layers"][4].update(type="conv"), InvalidInput),  # (it uses layer 1's tensors, with another type)
                          (lambda raw: raw["layers"][3].update(type="conv"), Unsupported),
                          (lambda raw: raw["layers"][3]["mlp"].update(kind="gated"), Unsupported),
                          (lambda raw: raw["layers"][3]["mixer"].update(heads=4, kv_heads=3), InvalidInput),
                          (lambda raw: raw["layers"][2].update(weights_of=2), InvalidInput),
                          (lambda raw: raw["layers"][2].update(weights_of=9), InvalidInput),
                          (lambda raw: raw["layers"][2].update(weights_of=-1), InvalidInput),
                          (lambda raw: raw["layers"][0].update(weights_of=2), InvalidInput),  # each the other's
                          (lambda raw: raw["layers"][2]["mixer"].update(vdim=8), InvalidInput)):  # other sizes than its tensors have
        raw = json.loads(json.dumps(TON_A))
        change(raw)
        with pytest.raises(error):
            spec_from_config(raw)
    raw = tonanex(50, 16, [layer(attention(2, 1, 8, 8), moe(3, 4, 8))])
    with pytest.raises(InvalidInput):
        spec_from_config(raw)
    raw = json.loads(json.dumps(TON_A))
    for key in ("type", "mixer", "mlp"):  # what a layer says beside weights_of may be left out
        del raw["layers"][2][key]
    assert spec_from_config(raw)[1].schedule == spec_from_config(TON_A)[1].schedule


def test_parts_refuse_what_does_not_go_together():
    base = dict(kind="causal_attention", width=32, heads=2, kv_heads=1, head_dim=16, q="q", k="k", v="v", o="o")
    for more in (dict(temperature="t"), dict(decay=("a", "b")), dict(unit_heads=1e-5, q_bias="q.b", k_bias="k.b", v_bias="v.b")):
        with pytest.raises(InvalidInput):
            build_part("mixer", dict(base, **more))
    base = dict(kind="routed", width=32, inner=8, experts=4, top=2, router="r", up="e{}.up", down="e{}.down")
    for more in (dict(activation="clamped_swiglu"), dict(scoring="other"), dict(limit=1.0), dict(shared={"inner": 8, "gate": "a", "up": "b", "down": "c"}),
                 dict(activation="clamped_swiglu", gate="e{}.gate", limit=-1.0)):
        with pytest.raises(InvalidInput):
            build_part("feed_forward", dict(base, **more))
    with pytest.raises(InvalidInput):
        build_part("block", {"kind": "pre_norm", "width": 32, "norm1": {"kind": "rms", "width": 32, "eps": 1e-5, "weight": "n"},
                             "mixer": dict(kind="causal_attention", width=32, heads=2, kv_heads=1, head_dim=16, q="q", k="k", v="v", o="o"),
                             "norm2": {"kind": "rms", "width": 32, "eps": 1e-5, "weight": "n2"}})


def test_attention_modules_are_named_by_what_is_compiled_in():
    from nnis_amd.kernels import ops

    decay = (torch.ones(2), torch.ones(2))
    assert ops.attention_module_name(32, 16, terms=ops.HeadTerms(decay, True)) == "attn_hd32v16lg"
    assert ops.attention_module_name(64, 64, 5.0, ops.ScoreExtras(keep_first=2), None, ops.HeadTerms(decay)) == "attn_hd64clx"
    assert ops.attention_module_name(64, 64, terms=ops.HeadTerms(None, True)) == "attn_hd64g" and not ops.HeadTerms()
    defines = dict(lib.module_recipe("attn_hd32v16clgxp").defines)
    assert defines == {"NNIS_HEAD_DIM": "32", "NNIS_VALUE_DIM": "16", "NNIS_SCORE_CAP": "1", "NNIS_DISTANCE_LOG": "1", "NNIS_HEAD_GATES": "1",
                       "NNIS_SCORE_EXTRAS": "1", "NNIS_POOLED_BLOCKS": "1"}
    assert dict(lib.module_recipe("attn_hd32l").defines) == {"NNIS_HEAD_DIM": "32", "NNIS_DISTANCE_LOG": "1"}


def test_a_random_model_reads_back(tmp_path):
    for name, (config, seed) in TONANEX_CONFIGS.items():
        folder = nnis_amd.write_random_model(str(tmp_path / name), config, seed)
        plain = T.PlainTonanex(folder)
        logits = plain.logits([1, 5, 2])
        assert logits.shape == (3, config["vocab"]) and bool(torch.isfinite(logits).all())


# ---------------------------------------------------------------------------------------------
# the plain implementation's mechanisms against special cases
# ---------------------------------------------------------------------------------------------

def test_plain_distance_bias_and_window():
    assert float(T.distance_bias(torch.tensor(2.0), torch.tensor(0.5), torch.tensor(6.0))) == pytest.approx(2.0 * math.log(4.0))
    assert float(T.distance_bias(torch.tensor(2.0), torch.tensor(0.5), torch.tensor(0.0))) == 0.0
    width, sizes = 8, attention(1, 1, 4, 4, scale=1.0, window=3)
    generator = torch.Generator().manual_seed(1)
    w = {name: torch.randn(shape, generator=generator, dtype=torch.float64) for name, shape in
         {"q": (4, width), "k": (4, width), "v": (4, width), "o": (width, 4), "g": (1, width)}.items()}
    w.update(temp=torch.tensor([0.0], dtype=torch.float64), r1=torch.tensor([1.0], dtype=torch.float64), r2=torch.tensor([1.0], dtype=torch.float64))
    h = torch.randn(6, width, generator=generator, dtype=torch.float64)
    # a temperature of zero leaves the bias alone: weights 1 / (1 + n) over the last three tokens
    p = torch.tensor([1.0 / 3.0, 0.5, 1.0], dtype=torch.float64)
    p = p / p.sum()
    want = (p[:, None] * (h[3:6] @ w["v"].T)).sum(dim=0) * T.sigmoid(h[5] @ w["g"].T) @ w["o"].T
    assert torch.allclose(T.attention(h, w, sizes, 1e-5)[5], want)


def test_plain_router_and_experts():
    w = {"router": torch.eye(4, dtype=torch.float64), "router.b": torch.tensor([0.0, 0.0, 3.0, 0.0], dtype=torch.float64)}
    chosen, weights = T.choose(torch.tensor([[1.0, 2.0, -1.5, 0.5]], dtype=torch.float64), w, 2)
    assert chosen.tolist() == [[1, 2]] and float(weights[0, 0]) == pytest.approx(1.0 / (1.0 + math.exp(-0.5)))  # logits 2 and 1.5, the bias in
    one = {"gate": torch.ones(1, 1, dtype=torch.float64), "up": torch.ones(1, 1, dtype=torch.float64), "down": torch.ones(1, 1, dtype=torch.float64)}
    value = lambda g, u: g / (1.0 + math.exp(-1.702 * g)) * (u + 1.0)  # noqa: E731
    at = lambda z: float(T.clamped_expert(torch.tensor([[z]], dtype=torch.float64), one, 2.0))  # noqa: E731
    assert at(1.0) == pytest.approx(value(1.0, 1.0)) and at(5.0) == pytest.approx(value(2.0, 2.0))
    assert at(-5.0) == pytest.approx(value(-5.0, -2.0))  # the gate has no lower limit
