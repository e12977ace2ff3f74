"""Tugovik on the CPU: its configuration reader, its model description, and the
plain implementation's own mechanisms against special cases."""

import json
import math

import pytest
import torch

import nnis_amd
import plain_tugovik as T
from nnis_amd.config.registry import spec_from_config
from nnis_amd.errors import InvalidInput, Unsupported
from nnis_amd.models.decoder import DecoderModel
from nnis_amd.parts import build_part
from nnis_amd.parts.base import KVRequest, StateRequest
from tugovik_configs import TUG_A, TUG_B, TUG_C, TUGOVIK_CONFIGS, attention, layer, moe, tugovik


def test_the_architecture_is_chosen_by_its_name():
    cfg, spec = spec_from_config(TUG_A)
    assert spec.architecture == "Tugovik" and spec.width == 96 and spec.vocab_size == 300 and spec.max_positions is None
    assert "Tugovik" in nnis_amd.config.registered_architectures()
    assert cfg.loop == (1, 3, 2) and cfg.side_dim == 24 and spec_from_config(TUG_B)[0].loop is None
    assert spec.final_norm == {"kind": "rms", "width": 96, "eps": 1e-5, "weight": "final.norm", "offset": 1.0}
    with pytest.raises(Unsupported):
        spec_from_config(dict(TUG_A, architecture="Tugovik2"))


def test_layers_run_in_their_order_with_caches_of_their_own():
    _, spec = spec_from_config(TUG_A)
    assert [e.layer for e in spec.schedule] == [0, 1, 2, 1, 2, 3] and all(e.reads_cache_of is None for e in spec.schedule)
    model = DecoderModel(spec)
    names = {t.name: t.shape for t in model.tensors()}
    assert names["side.embed"] == (300, 4 * 24) and names["l2.side.gate"] == (24, 96) and names["l2.side.proj"] == (96, 24) and names["l2.side.norm"] == (96,)
    assert names["l0.mix.q"] == (128, 96) and names["l0.mix.q.b"] == (128,) and names["l0.mix.v.b"] == (32,) and names["l0.mix.o"] == (96, 64)
    assert names["l1.mix.in"] == (2 * 96 + 2 * 3 * 24 + 6, 96) and names["l1.mix.conv"] == (96 + 144, 4) and names["l1.mix.norm"] == (96,)
    assert names["l1.mix.A_log"] == names["l1.mix.D"] == names["l1.mix.dt_bias"] == (6,)
    assert names["l2.mix.ra"] == (3, 24, 24) and names["l2.mix.ri.b"] == (3, 24) and names["l2.mix.lam"] == (72,) and names["l2.mix.x.b"] == (72,)
    assert names["l0.mlp.router"] == (6, 96) and names["l0.mlp.shared.sg"] == (1, 96) and "l3.mlp.shared.sg" not in names
    assert not any(name.startswith(("l2.mlp", "l2.norm2")) for name in names)
    requests, shared = model.cache_requests()
    space, unit = (StateRequest((6, 16, 24)), StateRequest((4, 240))), (StateRequest((72,)), StateRequest((4, 72)))
    assert not shared and [r[1] for r in requests] == [KVRequest(2, 32, 37, 16), space, unit, space, unit, KVRequest(1, 16, 70, 48)]
    _, spec = spec_from_config(TUG_C)
    assert [e.layer for e in spec.schedule] == [0, 1, 2] * 3
    _, spec = spec_from_config(TUG_B)
    assert all("side" not in block for block in spec.layers) and spec.layers[4]["mixer"]["chunk"] is None
    assert spec.layers[0]["feed_forward"]["groups"] is None and "shared" not in spec.layers[0]["feed_forward"]


def test_missing_and_wrong_keys_are_refused():
    for path in (["vocab"], ["norm", "eps"], ["layers", 0, "mixer", "heads"], ["layers", 0, "mixer", "scale"], ["layers", 0, "mixer", "mask", "size"],
                 ["layers", 1, "mixer", "state"], ["layers", 1, "mixer", "norm_groups"], ["layers", 2, "mixer", "blocks"], ["layers", 2, "type"],
                 ["layers", 0, "mlp", "router", "top"], ["layers", 0, "mlp", "expert"], ["layers", 0, "mlp", "shared", "ff"],
                 ["layers", 0, "mlp", "router", "groups", "keep"], ["loop", "times"], ["token_side", "dim"]):
        raw = json.loads(json.dumps(TUG_A))
        at = raw
        for key in path[:-1]:
            at = at[key]
        del at[path[-1]]
        with pytest.raises(InvalidInput):
            spec_from_config(raw)
    for change, error in ((lambda raw: raw["layers"][0].update(type="conv"), Unsupported),
                          (lambda raw: raw["layers"][0]["mlp"].update(kind="dense"), Unsupported),
                          (lambda raw: raw["layers"][0]["mixer"].update(heads=3), InvalidInput),
                          (lambda raw: raw["layers"][1]["mixer"].update(groups=4), InvalidInput),
                          (lambda raw: raw["layers"][1]["mixer"].update(norm_groups=7), InvalidInput),
                          (lambda raw: raw["layers"][2]["mixer"].update(blocks=5), InvalidInput),
                          (lambda raw: raw["layers"][0]["mlp"]["router"].update(top=5), InvalidInput),  # two groups of two are kept
                          (lambda raw: raw["layers"][0]["mlp"]["router"].update(experts=7), InvalidInput),
                          (lambda raw: raw["loop"].update(stop=1), InvalidInput), (lambda raw: raw["loop"].update(stop=5), InvalidInput),
                          (lambda raw: raw["layers"].clear(), InvalidInput)):
        raw = json.loads(json.dumps(TUG_A))
        change(raw)
        with pytest.raises(error):
            spec_from_config(raw)


def test_parts_refuse_what_does_not_go_together():
    base = dict(kind="causal_attention", width=32, heads=2, kv_heads=1, head_dim=16, q="q", k="k", v="v", o="o")
    with pytest.raises(InvalidInput):
        build_part("mixer", dict(base, chunk=8, window=8))
    base = dict(kind="routed", width=32, inner=8, experts=4, top=2, router="r", up="e{}.up", down="e{}.down", gate="e{}.gate", activation="silu_gated")
    for more in (dict(weight_scale=2.0), dict(group_marks=3),
                 dict(identity=1, shared={"inner": 8, "gate": "a", "up": "b", "down": "c", "weight": "d"})):
        with pytest.raises(InvalidInput):
            build_part("feed_forward", dict(base, **more))
    with pytest.raises(InvalidInput):
        build_part("feed_forward", dict(kind="token_input", width=32, inner=8, vocab_size=9, table="t", columns=12, first=6, gate="g", proj="p"))
    names = {key: key for key in ("w_in", "conv", "conv_bias", "dt_bias", "a_log", "d", "norm", "w_out")}
    for more in (dict(groups=2), dict(norm_parts=5), dict(states=0)):
        with pytest.raises(InvalidInput):
            build_part("mixer", dict(dict(kind="mamba2", width=32, heads=3, value_dim=8, states=4, groups=1, taps=4, norm_parts=1, eps=1e-5, **names), **more))
    names = {key: key for key in ("y", "y_bias", "x", "x_bias", "conv", "conv_bias", "r", "r_bias", "i", "i_bias", "rate", "o")}
    with pytest.raises(InvalidInput):
        build_part("mixer", dict(kind="rg_lru", width=32, channels=30, blocks=4, taps=4, **names))


def test_a_random_model_reads_back(tmp_path):
    for name, (config, seed) in TUGOVIK_CONFIGS.items():
        folder = nnis_amd.write_random_model(str(tmp_path / name), config, seed)
        logits = T.PlainTugovik(folder).logits([1, 5, 2])
        assert logits.shape == (3, config["vocab"]) and bool(torch.isfinite(logits).all())
    assert T.order_of_layers(TUG_A) == [0, 1, 2, 1, 2, 3] and T.order_of_layers(TUG_B) == [0, 1, 2, 3, 4]


# ---------------------------------------------------------------------------------------------
# the plain implementation's mechanisms against special cases
# ---------------------------------------------------------------------------------------------

def test_plain_chunks():
    assert [[j for j in range(8) if T.sees(i, j, 3)] for i in (0, 2, 3, 5, 6)] == [[0], [0, 1, 2], [3], [3, 4, 5], [6]]
    assert T.sees(5, 0, None) and not T.sees(0, 1, None)
    width, (_, sizes) = 8, attention(1, 1, 4, 4, scale=1.0, chunk=3)
    generator = torch.Generator().manual_seed(1)
    w = {name: torch.randn(shape, generator=generator, dtype=torch.float64) for name, shape in
         {"q": (4, width), "k": (4, width), "v": (4, width), "o": (width, 4), "v.b": (4,)}.items()}
    w.update({"q.b": torch.zeros(4, dtype=torch.float64), "k.b": torch.zeros(4, dtype=torch.float64)})
    w["q"] = w["q"] * 0.0  # all scores zero: the mean of the chunk's values so far
    h = torch.randn(5, width, generator=generator, dtype=torch.float64)
    v = h @ w["v"].T + w["v.b"]
    assert torch.allclose(T.attention(h, w, sizes)[4], v[3:5].mean(dim=0) @ w["o"].T)


def test_plain_recurrences():
    one = torch.ones(3, 1, 1, dtype=torch.float64)
    # a rate of ln 2 and steps of one halve the state before each token: S = 1, 3/2, 7/4; y = 2 S + 3 x
    y, S = T.state_space(one, one, 2.0 * one, torch.ones(3, 1, dtype=torch.float64), torch.log(torch.tensor([math.log(2.0)], dtype=torch.float64)),
                         torch.tensor([3.0], dtype=torch.float64))
    assert y.flatten().tolist() == pytest.approx([5.0, 6.0, 6.5]) and float(S) == pytest.approx(1.75)
    # heads of one group read the same B and C
    x = torch.randn(2, 4, 3, dtype=torch.float64, generator=torch.Generator().manual_seed(1))
    B = torch.randn(2, 2, 5, dtype=torch.float64, generator=torch.Generator().manual_seed(2))
    dt, rate, D = torch.ones(2, 4, dtype=torch.float64), torch.zeros(4, dtype=torch.float64), torch.zeros(4, dtype=torch.float64)
    y, _ = T.state_space(x, B, B, dt, rate, D)
    assert torch.allclose(y[0], x[0] * (B[0] * B[0]).sum(-1).repeat_interleave(2)[:, None])
    # a = 1/2: what is added is sqrt(3/4) i u
    half = torch.full((2, 1), math.log(0.5), dtype=torch.float64)
    S, _ = T.rglru_scan(torch.tensor([[1.0], [0.0]], dtype=torch.float64), half, torch.ones(2, 1, dtype=torch.float64))
    assert S.flatten().tolist() == pytest.approx([math.sqrt(0.75), math.sqrt(0.75) / 2.0])
    y, kept = T.short_conv(torch.tensor([[1.0], [2.0], [4.0]], dtype=torch.float64), torch.tensor([[0.5, 1.0]], dtype=torch.float64),
                           torch.tensor([10.0], dtype=torch.float64))
    assert y.flatten().tolist() == [11.0, 12.5, 15.0] and kept.tolist() == [[4.0]]  # the last tap on the token itself
    parts = T.gated_parts_norm(torch.tensor([[3.0, 4.0, 1.0, 1.0]], dtype=torch.float64), torch.full((1, 4), 50.0, dtype=torch.float64),
                               torch.ones(4, dtype=torch.float64), 2, 0.0)
    assert torch.allclose(parts, torch.tensor([[3.0, 4.0, 1.0, 1.0]], dtype=torch.float64) / torch.tensor([12.5, 12.5, 1.0, 1.0]).double().sqrt())


def test_plain_router():
    w = {"router": torch.eye(6, dtype=torch.float64)}
    z = torch.tensor([[3.0, -5.0, 1.5, 1.4, 0.0, 2.0]], dtype=torch.float64)
    s = T.sigmoid(z)[0]
    chosen, weights = T.choose(z, w, {"experts": 6, "top": 2, "scale": 3.0})
    assert chosen.tolist() == [[0, 5]] and torch.allclose(weights[0], 3.0 * s[[0, 5]] / (s[0] + s[5]))
    # pairs of neighbours: the sums of their two largest are s2 + s3 > s4 + s5 > s0 + s1, although s0 is the largest of all
    chosen, _ = T.choose(z, w, {"experts": 6, "top": 2, "scale": 1.0, "groups": {"count": 3, "keep": 1}})
    assert chosen.tolist() == [[2, 3]]
    chosen, _ = T.choose(z, w, {"experts": 6, "top": 3, "scale": 1.0, "groups": {"count": 3, "keep": 2}})
    assert chosen.tolist() == [[5, 2, 3]]
    config = tugovik(50, 16, [layer(attention(2, 1, 8, 8), moe(3, 4, 8))])
    with pytest.raises(InvalidInput):
        spec_from_config(config)
