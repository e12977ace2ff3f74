"""Tugovik on the GPU against the plain implementation (``plain_tugovik``):
each mechanism alone, then whole models through the engine -- prompts whole, in
portions and token by token, unequal batches, slots and pages used again, keys
far away, at page borders and at a chunk's edge, long decoding, greedy
generation through the library's entry point, the trace runner.  32-bit is held
to rounding; bfloat16 to the error of the plain model run with its activations
rounded where the engine rounds them.
"""

import os

import numpy as np
import pytest
import torch
from safetensors.torch import load_file, save_file

import nnis_amd
import plain_tugovik as T
import replay
from gpu_helpers import cache_for, context, runtime
from tugovik_configs import TUGOVIK_CONFIGS, attention, layer, mamba2, moe, rglru, tugovik

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


def _relative(got, want):
    got, want = torch.as_tensor(np.asarray(got)).double(), torch.as_tensor(np.asarray(want)).double()
    return float((got - want).pow(2).mean().sqrt() / want.pow(2).mean().sqrt().clamp_min(1e-30))


def _close(got, want, dtype, what="", bf16=3e-2, fp32=3e-5):
    error = _relative(got.detach().float().cpu() if isinstance(got, torch.Tensor) else got, want)
    bound = fp32 if dtype == "float32" else bf16
    assert error <= bound, f"{what}: relative error {error:.3g} (bound {bound:.3g})"


def _rounding(dtype):
    return T.identity if dtype == "float32" else T.bf16_round


def _weights(part, dtype, seed, scale=None):
    """Random tensors for a part, by its own declarations: (for the plain functions in 64-bit, for the part)."""
    from nnis_amd.weights.random_init import _INIT_RULES

    generator = torch.Generator().manual_seed(seed)
    stored = {}
    for t in part.tensors():
        value = _INIT_RULES[t.init](t, generator, torch.bfloat16)
        for ending, factor in (scale or {}).items():
            if t.name.endswith(ending):
                value = (value.float() * factor).to(torch.bfloat16)
                break
        stored[t.name] = value
    wide = torch.float32 if dtype == "float32" else torch.bfloat16
    return {n: v.double() for n, v in stored.items()}, {n: v.to(wide).cuda() for n, v in stored.items()}


def _run_in_steps(forward, cache, rt, xs, cuts):
    """Runs sequences through ``forward(x, ctx)``, all of them in every step; ``cuts[i]`` lists where sequence i's portions end."""
    slots = [cache.acquire() for _ in xs]
    done = [0] * len(xs)
    outs = [[] for _ in xs]
    cuts = [list(c) for c in cuts]
    while any(cuts):
        batch = [i for i in range(len(xs)) if cuts[i]]
        ends = [cuts[i].pop(0) for i in batch]
        ctx = context(cache, [(slots[i], end - done[i]) for i, end in zip(batch, ends)])
        x = torch.cat([xs[i][done[i]:end] for i, end in zip(batch, ends)]).to(rt.dtype).cuda()
        y = forward(x, ctx)
        row = 0
        for i, end in zip(batch, ends):
            outs[i].append(y[row:row + end - done[i]].float().cpu())
            row += end - done[i]
            done[i] = end
    for slot in slots:
        cache.release(slot)
    return [torch.cat(o) for o in outs]


# portions for three sequences of 200, 3 and 67 tokens: whole; portions down to two tokens and single tokens, across the borders of
# pages and of the runs that kernels take at a time (16, 64 and 128 tokens); single tokens behind a prompt
LENGTHS = [200, 3, 67]
CUTS = ([[200], [3], [67]], [[61, 63, 64, 66, 128, 130, 131, 200], [1, 2, 3], [2, 4, 20, 65, 66, 67]],
        [[150] + list(range(151, 201)), [3], [60] + list(range(61, 68))], [[16, 33, 200], [2, 3], [17, 67]])


def _inputs(width, seed=5):
    generator = torch.Generator().manual_seed(seed)
    return [torch.randn(n, width, generator=generator).to(torch.bfloat16).double() for n in LENGTHS]


# ---------------------------------------------------------------------------------------------
# the mechanisms alone
# ---------------------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("channels, taps, ring, plain", [(24, 4, True, False), (24, 4, False, False), (40, 3, True, True), (16, 2, True, True), (20, 4, True, True),
                                                         (8, 1, True, False), (72, 5, True, True), (520, 4, True, False), (48, 2, False, True)])
def test_the_short_convolution(dtype, channels, taps, ring, plain):
    """With and without an activation, with a bias of the inputs (which counts before the start neither), its state as a ring
    by position and as the last inputs in order."""
    from nnis_amd.kernels import ops
    from nnis_amd.parts.base import StateRequest

    rt = runtime(dtype)
    generator = torch.Generator().manual_seed(channels + taps)
    w, bias = (torch.randn(shape, generator=generator).to(torch.bfloat16).double() for shape in ((channels, taps), (channels,)))
    x_bias = torch.randn(channels, generator=generator).double()
    xs = _inputs(channels)
    cache = cache_for([StateRequest((taps if ring else taps - 1, channels))], rt, max_tokens=1024, max_positions=512)
    device_w, device_b = w.to(rt.dtype).cuda(), bias.to(rt.dtype).cuda()

    def forward(x, ctx):
        wide = torch.cat([torch.zeros_like(x[:, :8]), x], dim=1)  # the rows are columns of wider ones
        state = cache.view(0).state if (ring or taps > 1) else None
        return ops.conv_silu(wide[:, 8:], channels, device_w, device_b, state, ctx, rt.empty(x.shape[0], channels),
                             x_bias=x_bias.float().cuda() if plain else None, activation=None if plain else "silu", ring=ring)

    want = []
    for x in xs:
        y = T.short_conv(x + x_bias if plain else x, w, bias)[0]
        want.append(y if plain else T.silu(y))
    for cuts in CUTS:
        for g, y, n in zip(_run_in_steps(forward, cache, rt, xs, cuts), want, LENGTHS):
            _close(g, y, dtype, f"convolution {cuts[0][:2]} length {n}", bf16=4e-3, fp32=1e-6)


def _attention_part(sizes, width):
    from nnis_amd.parts import build_part

    return build_part("mixer", dict(kind="causal_attention", width=width, heads=sizes["heads"], kv_heads=sizes["kv_heads"], head_dim=sizes["dim"],
                                    value_dim=sizes["vdim"], scale=sizes["scale"], chunk=(sizes.get("mask") or {}).get("size"),
                                    q="q", k="k", v="v", o="o", q_bias="q.b", k_bias="k.b", v_bias="v.b"))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, kv_heads, dim, vdim, chunk, width", [
    (4, 2, 32, 16, 37, 64), (6, 1, 16, 48, 70, 48), (2, 2, 32, 16, 1, 96), (3, 3, 16, 48, 64, 56), (2, 1, 40, 40, 33, 40), (2, 1, 16, 16, None, 56),
    (20, 1, 16, 16, 130, 64), (5, 1, 64, 64, 100, 72), (1, 1, 32, 16, 2, 24)])
def test_attention_inside_chunks(dtype, heads, kv_heads, dim, vdim, chunk, width):
    rt = runtime(dtype)
    _, sizes = attention(heads, kv_heads, dim, vdim, scale=0.4, chunk=chunk)
    mixer = _attention_part(sizes, width)
    plain_w, part_w = _weights(mixer, dtype, 3, scale={".b": 25.0, "q": 8.0, "k": 8.0, "v": 5.0, "o": 5.0})
    mixer.check(rt)
    mixer.bind(part_w, rt)
    cache = cache_for([mixer.cache_request()], rt, max_tokens=1024, max_positions=512)
    xs, rnd = _inputs(width), _rounding(dtype)
    want = [T.attention(x, plain_w, sizes, rnd) for x in xs]
    for name in ("q.b", "v.b") if chunk != 1 else ("v.b",):  # (a bias of the keys moves every score of a query alike)
        assert _relative(T.attention(xs[0], dict(plain_w, **{name: plain_w[name] * 0.0}), sizes, rnd), want[0]) > 1e-2, name
    for cuts in CUTS:
        got = _run_in_steps(lambda x, ctx: mixer.forward(x, ctx, cache.view(0), rt), cache, rt, xs, cuts)
        for g, w, n in zip(got, want, LENGTHS):
            _close(g, w, dtype, f"attention {cuts[0][:2]} length {n}", bf16=4e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk, heads, kv_heads", [(37, 1, 1), (64, 5, 1), (65, 2, 2), (128, 1, 1), (9, 1, 1)])
def test_the_chunks_edge_decides(dtype, chunk, heads, kv_heads):
    """One key stands out.  It is the first of the query's chunk or the last of the chunk before; the query is its chunk's
    first token, one in the middle, and its last; it comes in a prompt, in a portion, and alone.  The output tells."""
    rt = runtime(dtype)
    width = 32
    _, sizes = attention(heads, kv_heads, 32, 16, scale=0.05, chunk=chunk)
    mixer = _attention_part(sizes, width)
    plain_w, part_w = _weights(mixer, dtype, 11, scale={"v": 20.0, "o": 20.0})
    for name, count, first in (("q", heads, 0), ("k", kv_heads, 8)):
        reads = torch.zeros(32, width, dtype=torch.float64)
        reads[:8, first:first + 8] = torch.eye(8, dtype=torch.float64)
        plain_w[name], plain_w[name + ".b"] = reads.repeat(count, 1), torch.zeros(32 * count, dtype=torch.float64)
        for key in (name, name + ".b"):
            part_w[key] = plain_w[key].to(part_w[key].dtype).cuda()
    mixer.bind(part_w, rt)
    cache = cache_for([mixer.cache_request()], rt, max_tokens=1024, max_positions=1024)
    generator = torch.Generator().manual_seed(1)
    start = chunk * (180 // chunk + 1)
    for last in sorted({start, start + chunk // 2, start + chunk - 1}):
        n, share = last + 1, {}
        for what, place in (("inside", start), ("outside", start - 1)):
            x = (0.05 * torch.randn(n, width, generator=generator)).to(torch.bfloat16).double()
            x[place, 8:16] = 8.0
            x[last, :8] = 8.0
            want = T.attention(x, plain_w, sizes)
            without = x.clone()
            without[place, 8:16] = -8.0
            share[what] = _relative(T.attention(without, plain_w, sizes)[last], want[last])
            for cuts in ([n], [n - 3, n], [n - 1, n], [start - 2] + list(range(start - 1, n + 1)) if n - start < 40 else [n - 5, n - 2, n - 1, n]):
                got = _run_in_steps(lambda h, ctx: mixer.forward(h, ctx, cache.view(0), rt), cache, rt, [x], [cuts])[0]
                _close(got[last], want[last], dtype, f"mark {what} at {place} (chunks of {chunk}, {n} tokens), cuts {cuts[:2]}")
                _close(got, want, dtype, f"mark {what} at {place}, all tokens, cuts {cuts[:2]}")
        assert (share["inside"] > 0.3 or last == start) and share["outside"] < 1e-9, share


SPACES = [  # heads, channels a head, states, groups, taps, parts of the norm, width
    (6, 16, 24, 3, 4, 2, 64), (4, 32, 64, 1, 4, 1, 48), (2, 48, 128, 2, 3, 4, 40), (3, 20, 12, 1, 2, 1, 56), (2, 16, 200, 1, 4, 2, 24), (1, 16, 8, 1, 1, 1, 32),
    (5, 8, 30, 5, 4, 5, 40), (8, 64, 16, 4, 2, 8, 72), (3, 16, 40, 1, 4, 3, 24)]


def _space_part(heads, vdim, states, groups, taps, parts, width, eps=1e-5):
    from nnis_amd.parts import build_part

    return build_part("mixer", dict(kind="mamba2", width=width, heads=heads, value_dim=vdim, states=states, groups=groups, taps=taps, norm_parts=parts, eps=eps,
                                    w_in="in", conv="conv", conv_bias="conv.b", dt_bias="dt_bias", a_log="A_log", d="D", norm="norm", w_out="o"))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", SPACES)
def test_a_state_space_alone(dtype, sizes):
    rt = runtime(dtype)
    heads, vdim, states, groups, taps, parts, width = sizes
    mixer = _space_part(*sizes)
    plain_w, part_w = _weights(mixer, dtype, 3, scale={"in": 25.0, "conv": 2.0, "o": 5.0})
    mixer.check(rt)
    mixer.bind(part_w, rt)
    cache = cache_for([mixer.cache_request()], rt, max_tokens=1024, max_positions=512)
    xs, rnd = _inputs(width), _rounding(dtype)
    described = {"heads": heads, "vdim": vdim, "state": states, "groups": groups, "norm_groups": parts}
    want = [T.mamba2(x, plain_w, described, 1e-5, rnd) for x in xs]
    for name in ("D", "dt_bias", "A_log", "conv.b"):  # every one of them moves the output
        other = dict(plain_w, **{name: plain_w[name] * 0.5 - 0.5})
        assert _relative(T.mamba2(xs[0], other, described, 1e-5, rnd), want[0]) > 3e-3, name
    for cuts in CUTS:
        got = _run_in_steps(lambda x, ctx: mixer.forward(x, ctx, cache.view(0), rt), cache, rt, xs, cuts)
        for g, w, n in zip(got, want, LENGTHS):
            _close(g, w, dtype, f"state space {cuts[0][:2]} length {n}")


@pytest.mark.parametrize("heads, P, N, groups", [(4, 32, 64, 2), (2, 16, 128, 1), (3, 48, 24, 3), (2, 16, 256, 2), (1, 64, 32, 1), (5, 16, 40, 1)])
def test_the_state_spaces_kernels_agree(heads, P, N, groups):
    """The chunks on the matrix cores, the token-by-token kernel and, token by token behind them, the step with the convolution
    in it, on bfloat16 rows: outputs and states, over lengths around a chunk's, from a state that is there already."""
    from nnis_amd.kernels import ops
    from nnis_amd.parts.base import StateRequest

    rt = runtime("bfloat16")
    generator = torch.Generator().manual_seed(N)
    channels = heads * P + 2 * groups * N
    rate = (0.02 + torch.rand(heads, generator=generator)).cuda()
    dt_bias, D = torch.randn(heads, generator=generator).cuda() - 1.0, torch.randn(heads, generator=generator).cuda()
    taps = torch.zeros(1, channels)
    taps[0] = 1.0
    for lengths in ([1, 64, 63], [65, 16, 128], [300, 2, 129]):
        total = sum(lengths)
        rows = torch.randn(total, channels + heads * P + heads, generator=generator).to(torch.bfloat16).cuda()
        z, xbc, dt = rows[:, :heads * P], rows[:, heads * P:heads * P + channels].contiguous(), rows[:, heads * P + channels:]
        outs, states = [], []
        for which in ("chunks", "scan", "plain"):
            cache = cache_for([StateRequest((heads, P, N))], rt, max_tokens=2048, max_positions=1024)
            slots = [cache.acquire() for _ in lengths]
            state = cache.view(0).state
            state.copy_(torch.randn(state.shape, generator=torch.Generator().manual_seed(1)))
            first = state.double().cpu()
            ctx = context(cache, list(zip(slots, lengths)))
            if which != "plain":
                outs.append(ops.state_space(xbc, dt, z, rate, dt_bias, D, state, ctx, groups, torch.empty(total, heads * P, device="cuda"),
                                            longest=None if which == "chunks" else 1).double().cpu())
                states.append(state[slots].double().cpu())
                continue
            wide, at, ys, ends = rows.double().cpu(), 0, [], []
            for slot, n in zip(slots, lengths):
                part = wide[at:at + n]
                x, B, C = (part[:, a:b] for a, b in ((heads * P, 2 * heads * P), (2 * heads * P, 2 * heads * P + groups * N),
                                                     (2 * heads * P + groups * N, heads * P + channels)))
                y, S = T.state_space(x.reshape(n, heads, P), B.reshape(n, groups, N), C.reshape(n, groups, N),
                                     T.softplus(part[:, heads * P + channels:] + dt_bias.double().cpu()), torch.log(rate.double().cpu()), D.double().cpu(),
                                     first[slot].transpose(1, 2))
                ys.append(y.reshape(n, heads * P) * T.silu(part[:, :heads * P]))
                ends.append(S.transpose(1, 2))
                at += n
            for got, state_of in zip(outs, states):
                assert _relative(got, torch.cat(ys)) < 1e-4 and _relative(state_of, torch.stack(ends)) < 1e-4, lengths
        assert _relative(outs[1], torch.cat(ys)) < 1e-5  # (token by token: 32-bit sums of exact products)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_state_space_reads_a_key_from_far_back(dtype):
    """States that hardly decay: token 3's x, written under a B of its own, is read 700 tokens later by a C that asks for it."""
    rt = runtime(dtype)
    heads, vdim, states, groups, taps, parts, width = 2, 16, 32, 1, 1, 1, 112
    mixer = _space_part(heads, vdim, states, groups, taps, parts, width)
    plain_w, part_w = _weights(mixer, dtype, 3, scale={"o": 10.0})
    inner = heads * vdim
    w_in = torch.zeros(2 * inner + 2 * states + heads, width, dtype=torch.float64)
    w_in[:inner, 96] = 2.0  # z: open
    w_in[inner:2 * inner, :inner] = torch.eye(inner)
    w_in[2 * inner:2 * inner + states, 32:64] = torch.eye(states)
    w_in[2 * inner + states:2 * inner + 2 * states, 64:96] = torch.eye(states)
    fixed = {"in": w_in, "conv": torch.ones_like(plain_w["conv"]), "conv.b": plain_w["conv.b"] * 0.0, "A_log": torch.full((heads,), -9.0).double(),
             "dt_bias": torch.zeros(heads).double(), "D": torch.zeros(heads).double()}
    for name, value in fixed.items():
        plain_w[name], part_w[name] = value.to(torch.bfloat16).double(), value.to(torch.bfloat16).to(part_w[name].dtype).cuda()
    mixer.bind(part_w, rt)
    cache = cache_for([mixer.cache_request()], rt, max_tokens=1024, max_positions=1024)
    n = 710
    x = (0.02 * torch.randn(n, width, generator=torch.Generator().manual_seed(2))).to(torch.bfloat16).double()
    x[:, 96] = 1.0
    x[3, :inner] = torch.linspace(1.0, 4.0, inner).double()
    x[3, 32 + 5], x[n - 1, 64 + 5] = 6.0, 6.0
    x = x.to(torch.bfloat16).double()
    described = {"heads": heads, "vdim": vdim, "state": states, "groups": groups, "norm_groups": parts}
    want = T.mamba2(x, plain_w, described, 1e-5, _rounding(dtype))
    without = x.clone()
    without[3, :inner] = 0.0
    assert _relative(T.mamba2(without, plain_w, described, 1e-5)[n - 1], want[n - 1]) > 0.5
    for cuts in ([n], [n - 2, n], [2, 4, 500, n - 1, n], [690] + list(range(691, n + 1))):
        got = _run_in_steps(lambda h, ctx: mixer.forward(h, ctx, cache.view(0), rt), cache, rt, [x], [cuts])[0]
        _close(got[n - 1], want[n - 1], dtype, f"far token, cuts {cuts[:2]}", bf16=2e-2)


UNITS = [(72, 3, 4, 64), (80, 5, 4, 48), (60, 1, 3, 40), (64, 4, 2, 56), (8, 1, 4, 24), (48, 4, 1, 32), (264, 1, 4, 40), (512, 2, 4, 24), (640, 1, 3, 32)]


def _unit_part(channels, blocks, taps, width):
    from nnis_amd.parts import build_part

    return build_part("mixer", dict(kind="rg_lru", width=width, channels=channels, blocks=blocks, taps=taps, y="y", y_bias="y.b", x="x", x_bias="x.b",
                                    conv="conv", conv_bias="conv.b", r="ra", r_bias="ra.b", i="ri", i_bias="ri.b", rate="lam", o="o"))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("channels, blocks, taps, width", UNITS)
def test_a_gated_linear_unit_alone(dtype, channels, blocks, taps, width):
    rt = runtime(dtype)
    mixer = _unit_part(channels, blocks, taps, width)
    plain_w, part_w = _weights(mixer, dtype, 3, scale={"ra": 15.0, "ri": 15.0, ".b": 4.0, "y": 12.0, "x": 12.0, "conv": 3.0, "o": 5.0})
    mixer.check(rt)
    mixer.bind(part_w, rt)
    cache = cache_for([mixer.cache_request()], rt, max_tokens=1024, max_positions=512)
    xs, rnd = _inputs(width), _rounding(dtype)
    want = [T.rglru(x, plain_w, {"blocks": blocks}, rnd) for x in xs]
    for name in ("ra", "ri", "ra.b", "ri.b", "lam", "x.b", "y.b", "conv.b"):  # every one of them moves the output
        other = dict(plain_w, **{name: plain_w[name] * 0.5 - (0.5 if name == "lam" else 0.0)})
        assert _relative(T.rglru(xs[0], other, {"blocks": blocks}, rnd), want[0]) > 3e-3, name
    for cuts in CUTS:
        got = _run_in_steps(lambda x, ctx: mixer.forward(x, ctx, cache.view(0), rt), cache, rt, xs, cuts)
        for g, w, n in zip(got, want, LENGTHS):
            _close(g, w, dtype, f"unit {cuts[0][:2]} length {n}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_gated_linear_unit_holds_a_value_for_long(dtype):
    """Rates so small that a token's share is there 700 tokens later: decays within a thousandth of one, whose complement is
    what is added.  The first token is no special case."""
    rt = runtime(dtype)
    channels, blocks, taps, width = 32, 2, 2, 40
    mixer = _unit_part(channels, blocks, taps, width)
    plain_w, part_w = _weights(mixer, dtype, 3, scale={"ra": 5.0, "x": 12.0, "y": 12.0, "o": 5.0})
    for w in (plain_w, part_w):
        w["lam"][:] = torch.linspace(-14.0, -7.0, channels).to(torch.bfloat16)
        w["x.b"][:], w["conv.b"][:] = 0.0, 0.0
        w["conv"][:, :1] = 0.0  # u is the current token's
        w["conv"][:, 1:] = 1.0
    mixer.bind(part_w, rt)
    cache = cache_for([mixer.cache_request()], rt, max_tokens=1024, max_positions=1024)
    n = 710
    x = (0.05 * torch.randn(n, width, generator=torch.Generator().manual_seed(2))).to(torch.bfloat16).double()
    x[0] *= 200.0
    x = x.to(torch.bfloat16).double()
    want = T.rglru(x, plain_w, {"blocks": blocks}, _rounding(dtype))
    without = x.clone()
    without[0] = 0.0
    assert _relative(T.rglru(without, plain_w, {"blocks": blocks})[n - 1], want[n - 1]) > 0.3
    for cuts in ([n], [n - 2, n], [1, 2, 4, 500, n - 1, n], [690] + list(range(691, n + 1))):
        got = _run_in_steps(lambda h, ctx: mixer.forward(h, ctx, cache.view(0), rt), cache, rt, [x], [cuts])[0]
        _close(got[n - 1], want[n - 1], dtype, f"far token, cuts {cuts[:2]}", bf16=2e-2)
        _close(got, want, dtype, f"all tokens, cuts {cuts[:2]}", bf16=2e-2)


ROUTERS = [  # outputs, top, groups (count, keep) or None, shared, width
    (8, 2, (2, 1), True, 64), (6, 2, (3, 2), True, 40), (16, 2, (4, 2), True, 96), (64, 6, (8, 3), True, 128), (63, 4, (9, 2), False, 32), (96, 3, (8, 2), True, 64),
    (130, 5, (26, 4), True, 32), (5, 2, None, True, 48), (1, 1, None, True, 24), (12, 3, (12, 3), False, 56), (9, 3, (3, 1), True, 20),
    (70, 2, None, False, 36), (17, 2, None, True, 32)]


@pytest.mark.parametrize("rows", [1, 5, 40, 300])
@pytest.mark.parametrize("outputs, top, groups, shared, width", ROUTERS)
def test_the_router_with_sigmoid_scores(outputs, top, groups, shared, width, rows):
    """From rows, from logits, and behind the norm of a stream, with and without a part still to be added: choices as dense
    weights and as lists; the shared expert's weight beside them."""
    from nnis_amd.kernels import ops

    generator = torch.Generator().manual_seed(outputs + rows)
    stream = torch.randn(rows, width, generator=generator)
    delta = torch.randn(rows, width, generator=generator).to(torch.bfloat16)
    gain = (1.0 + 0.2 * torch.randn(width, generator=generator)).to(torch.bfloat16)
    w = (torch.randn(outputs + int(shared), width, generator=generator) * 2.0 * width ** -0.5).to(torch.bfloat16).float()
    total = stream.double() + delta.double()
    h = T.over_rms(total, 1e-5) * gain.double()
    router = {"experts": outputs, "top": top, "scale": 1.7}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    wanted, weights = T.choose(h, {"router": w[:outputs].double()}, router)
    # rows whose choice is clear: neither a group's mark nor an expert's score is close to the next one's
    s = T.sigmoid(h @ w[:outputs].double().T)
    clear = torch.ones(rows, dtype=torch.bool)
    if groups and groups[1] < groups[0]:
        size = outputs // groups[0]
        marks = torch.topk(s.view(rows, groups[0], size), min(2, size), dim=-1).values.sum(-1)
        ordered = marks.sort(dim=1, descending=True).values
        clear &= ordered[:, groups[1] - 1] - ordered[:, groups[1]] > 4e-3
        kept = torch.zeros_like(marks).scatter(1, torch.topk(marks, groups[1], dim=1).indices, 1.0).repeat_interleave(size, dim=1)
        s = torch.where(kept > 0, s, torch.zeros_like(s))
    ordered = s.sort(dim=1, descending=True).values
    if top < outputs:
        clear &= ordered[:, top - 1] - ordered[:, top] > 4e-3
    assert float(clear.double().mean()) > 0.5 or rows < 8
    dense_want = torch.zeros(rows, outputs, dtype=torch.float64).scatter(1, wanted, weights)
    share = T.sigmoid(h @ w[outputs:].double().T)[:, 0] if shared else None

    def made():
        return (torch.empty(rows, outputs, device="cuda"), torch.empty(rows, device="cuda"),
                (torch.empty(rows, top, dtype=torch.int32, device="cuda"), torch.empty(rows, top, device="cuda")))

    def check(gates, keep, chosen=None, bound=2e-5):
        assert float((gates.cpu().double() - dense_want).abs()[clear].max() if bool(clear.any()) else 0.0) < bound
        if shared:
            assert float((keep.cpu().double() - share).abs().max()) < bound
        if chosen is not None and bool(clear.any()):
            listed = torch.zeros(rows, outputs, dtype=torch.float64).scatter(1, chosen[0].cpu().long(), chosen[1].cpu().double())
            assert float((listed - dense_want).abs()[clear].max()) < bound

    rule = dict(groups=groups, scoring="sigmoid", weight_scale=1.7, group_marks=2, shared_gate=shared)
    gates, keep, chosen = made()
    ops.route(h.float().cuda(), w.cuda(), None, outputs, top, gates, keep, chosen=chosen, **rule)
    check(gates, keep, chosen)
    logits = ops.router_logits(h.float().cuda(), w.cuda(), torch.empty(rows, w.shape[0], device="cuda"))
    gates, keep, _ = made()
    ops.route_top(logits, None, outputs, top, gates, keep, **rule)
    check(gates, keep)
    for h_dtype in (torch.float32, torch.bfloat16):
        gates, keep, chosen = made()
        x = stream.clone().cuda()
        got = ops.route_norm(x, delta.cuda(), gain.float().cuda(), 1e-5, torch.empty(rows, width, device="cuda", dtype=h_dtype), w.cuda(), None, outputs,
                             top, gates, keep, chosen=chosen, weight_bf16=w.to(torch.bfloat16).cuda(), **rule)
        many = rows > 256 and h_dtype == torch.bfloat16 and width % 32 == 0 and outputs <= 64  # (the logits of the rounded rows)
        check(gates, keep, chosen, bound=1e-2 if many else 2e-5)
        assert _relative(x.cpu(), total) < 1e-6 and _relative(got.float().cpu(), h) < (1e-6 if h_dtype == torch.float32 else 4e-3)
        ops.route_norm(x, None, gain.cuda(), 1e-5, got, w.cuda(), None, outputs, top, gates, keep, **rule)  # the sum is in the stream now
        check(gates, keep)


def _routed(width, inner, experts, top, groups, scale, shared, dtype):
    from nnis_amd.parts import build_part

    rt = runtime(dtype)
    description = dict(kind="routed", width=width, inner=inner, experts=experts, top=top, groups=groups, group_marks=2, scoring="sigmoid", weight_scale=scale,
                       activation="silu_gated", router="router", gate="e{}.gate", up="e{}.up", down="e{}.down")
    if shared is not None:
        description["shared"] = dict(inner=shared, gate="shared.gate", up="shared.up", down="shared.down", weight="shared.sg")
    part = build_part("feed_forward", description)
    plain_w, part_w = _weights(part, dtype, 3, scale={".gate": 10.0, ".up": 10.0, ".down": 10.0})
    part.check(rt)
    part.bind(part_w, rt)
    mlp = {"router": {"experts": experts, "top": top, "scale": scale}}
    if groups is not None:
        mlp["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared is not None:
        mlp["shared"] = {"ff": shared}
    return rt, part, plain_w, mlp


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(64, 24, 6, 2, (3, 2), 1.5, 40), (48, 64, 3, 1, None, 1.0, None), (96, 16, 9, 3, (3, 1), 0.5, 16), (40, 72, 70, 4, None, 2.0, 136),
                                   (128, 8, 2, 2, (2, 2), 1.0, 8), (8, 8, 1, 1, None, 3.0, 24)])
def test_routed_feed_forward_alone(dtype, sizes):
    """All three ways through the experts' products, with the shared expert's weight a token: 1 to 700 rows."""
    rt, part, plain_w, mlp = _routed(*sizes, dtype)
    width, experts, top = sizes[0], sizes[2], sizes[3]
    for rows in (1, 2, 15, 16, 17, 70, 95, 96, 257, 700):
        x = torch.randn(rows, width, generator=torch.Generator().manual_seed(rows)).to(torch.bfloat16).double()
        want, chosen = T.routed_feed_forward(x, plain_w, mlp, _rounding(dtype))
        again = T.choose(x + 3e-3 * torch.randn(x.shape, generator=torch.Generator().manual_seed(1)).double(), plain_w, mlp["router"])[0]
        clear = (again.sort(dim=1).values == chosen.sort(dim=1).values).all(dim=1)  # (a choice that a nudge of the row does not change)
        assert float(clear.double().mean()) > 0.8
        got = part.forward(x.to(rt.dtype).cuda(), None, rt).float().cpu()
        _close(got[clear], want[clear], dtype, f"{rows} rows", bf16=2e-2)
        if rows == 700 and sizes[6] is not None:
            unweighted = T.routed_feed_forward(x, dict(plain_w, **{"shared.sg": plain_w["shared.sg"] * 0.0}), mlp, _rounding(dtype))[0]
            assert _relative(unweighted, want) > 1e-2  # the shared expert's weight matters


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width, inner, layers, index", [(64, 24, 3, 1), (96, 8, 1, 0), (40, 136, 2, 1), (256, 16, 4, 3), (24, 5, 2, 1)])
def test_a_tokens_own_input(dtype, width, inner, layers, index):
    from nnis_amd.parts import build_part

    rt = runtime(dtype)
    part = build_part("feed_forward", dict(kind="token_input", width=width, inner=inner, vocab_size=50, table="table", columns=layers * inner,
                                           first=index * inner, gate="side.gate", proj="side.proj"))
    norm = build_part("norm", dict(kind="rms", width=width, eps=1e-5, weight="side.norm", wide=True))
    plain_w, part_w = _weights(part, dtype, 3, scale={"side.gate": 15.0, "side.proj": 10.0})
    part.bind(part_w, rt)
    gain = (1.0 + 0.3 * torch.randn(width, generator=torch.Generator().manual_seed(9))).to(torch.bfloat16)
    norm.bind({"side.norm": gain.to(rt.dtype).cuda()}, rt)
    plain_w["side.norm"] = gain.double()
    cache = cache_for([None], rt)
    for rows in (1, 3, 17, 64, 300):
        generator = torch.Generator().manual_seed(rows)
        x = torch.randn(rows, width, generator=generator).to(torch.bfloat16).double()
        ids = torch.randint(0, 50, (rows,), generator=generator, dtype=torch.int32)
        table = plain_w["table"][ids.long()][:, index * inner:(index + 1) * inner]
        want = x + T.token_side(x, table, plain_w, 1e-5, _rounding(dtype))
        ctx = context(cache, [(cache.acquire(), rows)])
        ctx.ids = ids.cuda()
        stream = x.float().cuda()
        norm.post_step(stream, part.forward(x.to(rt.dtype).cuda(), ctx, rt), rt)
        _close(stream, want, dtype, f"{rows} rows", bf16=1e-2)
        ids[0] = -1  # a padding row
        ctx.ids = ids.cuda()
        got = part.forward(x.to(rt.dtype).cuda(), ctx, rt)
        assert not bool(got[0].any()) and bool(torch.isfinite(got.float()).all())


# ---------------------------------------------------------------------------------------------
# whole models through the engine
# ---------------------------------------------------------------------------------------------

def _sharpen(folder, steady):
    """A random model's weights are too small for its mixers to matter.  Projections are scaled so that each matters, the head
    so that logits are of order one to ten; routers so that few scores are saturated.  ``steady`` (for bfloat16, where a
    close choice falls the other way by rounding): routers read a code of the token that the first channels of the stream carry
    and that no layer writes to."""
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    for key in tensors:
        if key.endswith((".mix.q", ".mix.k", ".mix.v", ".mix.o", ".up", ".e.gate", ".down", ".mix.y", ".mix.x", ".mix.ra", ".mix.ri")) or \
                (key.endswith(".gate") and ".mlp." in key):
            factor = 7.0
        elif key.endswith((".mix.in", ".side.gate", ".side.proj", ".b")):
            factor = 10.0 if not key.endswith(".b") or ".mix.conv" not in key else 3.0
        elif key.endswith((".mlp.router", ".shared.sg")):
            factor = 0.6
        elif key == "embed":
            factor = 40.0
        elif key == "head":
            factor = 10.0
        else:
            continue
        tensors[key] = (tensors[key].float() * factor).to(torch.bfloat16)
    if steady:
        width = tensors["embed"].shape[1]
        code = min(8, width // 4)
        tensors["embed"][:, :code] = torch.where(tensors["embed"][:, :code] > 0, 0.8, -0.8).to(torch.bfloat16)
        for key, t in tensors.items():
            if key.endswith((".mix.o", ".down")):
                t[:code] = 0.0
            elif key.endswith(".side.norm"):
                t[:code] = 0.0
            elif key.endswith(".mlp.router"):
                t[:, :code] *= (width / code) ** 0.5
                t[:, code:] = 0.0
    save_file(tensors, path)


def _folder(path, config, seed, dtype="float32"):
    nnis_amd.write_random_model(str(path), config, seed)
    _sharpen(str(path), steady=dtype == "bfloat16")
    return str(path)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {(name, dtype): _folder(tmp_path_factory.mktemp(f"tugovik_{name}_{dtype}"), config, seed, dtype)
            for name, (config, seed) in TUGOVIK_CONFIGS.items() for dtype in DTYPES}


def _ids(count, vocab, seed):
    generator = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (count,), generator=generator).tolist()


class Yardstick:
    """What the engine may differ from the plain 64-bit logits by, as root mean square relative to the logits' own: in
    32-bit, rounding (5e-5 over a prompt, 2e-4 at a single position); in bfloat16, three times what rounding the plain
    model's activations to bfloat16 does on the same tokens (a single position: four times the worst position's)."""

    def __init__(self, plain):
        self.plain, self.known = plain, {}
        self.least = (0.0, 0.0)
        self.least = self.twin(_ids(64, plain.config["vocab"], 999))[1:]

    def twin(self, ids):
        key = tuple(ids)
        if key not in self.known:
            want, twin = self.plain.logits(ids), self.plain.logits(ids, T.bf16_round)
            rows = [_relative(twin[i], want[i]) for i in range(len(ids))]
            self.known[key] = (want, _relative(twin, want), max(rows))
        return self.known[key]

    def check(self, got, ids, dtype, what, rows=None):
        want, overall, worst = self.twin(ids)
        assert dtype == "float32" or 1e-4 < overall < 0.3, overall
        single = isinstance(rows, int)
        want = want if rows is None else want[rows]
        error = _relative(got, want)
        bound = (2e-4 if single else 5e-5) if dtype == "float32" else (4.0 * max(worst, self.least[1]) if single else 3.0 * max(overall, self.least[0]))
        assert error <= bound, f"{what}: relative error {error:.3g} (bound {bound:.3g})"


def _collect(engine, slot, ids, cuts):
    from nnis_amd.engine.batch import StepEntry

    rows, done = [], 0
    for end in cuts:
        rows.append(engine.step([StepEntry(slot, ids[done:end], list(range(end - done)))]).cpu())
        done = end
    return torch.cat(rows)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(TUGOVIK_CONFIGS))
def test_the_stream_after_every_layer(folders, name, dtype):
    from nnis_amd.engine.batch import StepEntry
    from nnis_amd.parts.lazy import PendingNorm

    plain = T.PlainTugovik(folders[name, dtype])
    engine = nnis_amd.load_engine(folders[name, dtype], dtype=dtype, max_tokens=256)
    ids = _ids(90, TUGOVIK_CONFIGS[name][0]["vocab"], 10)  # (no token's state-space output all but cancels)
    want, twin = [], []
    plain.logits(ids, stream_after=want)
    plain.logits(ids, T.bf16_round, stream_after=twin)  # what rounding to bfloat16 alone does to the stream behind each layer
    seen = []
    for block in engine.model.layers:
        def watched(stream, ctx, view, rt, following=None, inner=block.forward):
            out = inner(stream, ctx, view, rt, following=following)
            x, left = (out.x, out.delta) if isinstance(out, PendingNorm) else out
            seen.append(x.clone() if left is None else x + left.float())
            return out
        block.forward = watched
    slot = engine.start_sequence()
    engine.step([StepEntry(slot, ids, [0])])
    assert len(seen) == len(want) == len(T.order_of_layers(TUGOVIK_CONFIGS[name][0]))
    for run, (got, expected, rounded) in enumerate(zip(seen, want, twin)):
        assert _relative(got.cpu(), expected) < (1e-5 if dtype == "float32" else max(1e-2, 3.0 * _relative(rounded, expected))), f"layer {run}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(TUGOVIK_CONFIGS))
def test_prompts_whole_in_portions_and_token_by_token(folders, name, dtype):
    config = TUGOVIK_CONFIGS[name][0]
    plain = T.PlainTugovik(folders[name, dtype])
    engine = nnis_amd.load_engine(folders[name, dtype], dtype=dtype, max_tokens=1024)
    ids = _ids(230, config["vocab"], 1)
    yard = Yardstick(plain)
    for cuts in ([230], [2, 4, 5, 63, 64, 66, 128, 129, 150], [100] + list(range(101, 151)), list(range(1, 41)), [200, 230], [16, 80, 144, 230]):
        slot = engine.start_sequence()
        got = _collect(engine, slot, ids, cuts)
        engine.end_sequence(slot)
        yard.check(got, ids, dtype, f"{name} cuts {cuts[:3]}..", rows=slice(0, cuts[-1]))
        for place in (0, 1, 2, cuts[-1] - 1):  # every position by itself, the first tokens among them
            yard.check(got[place], ids, dtype, f"{name} cuts {cuts[:3]}.. position {place}", rows=place)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_prompt_twice(folders, dtype):
    """Rows enough for every kernel for many rows; the same shape twice, so that the second is replayed from a graph, with
    another step between the two."""
    from nnis_amd.engine.batch import StepEntry

    config = TUGOVIK_CONFIGS["A"][0]
    plain = T.PlainTugovik(folders["A", dtype])
    engine = nnis_amd.load_engine(folders["A", dtype], dtype=dtype, max_tokens=2048)
    yard = Yardstick(plain)
    prompts = [_ids(n, config["vocab"], n) for n in (450, 449, 450)]
    for turn, ids in enumerate(prompts):
        slot = engine.start_sequence()
        got = engine.step([StepEntry(slot, ids, list(range(len(ids))))]).cpu()
        yard.check(got, ids, dtype, f"prompt {turn}")
        engine.step([StepEntry(slot, [3], [0])])
        engine.end_sequence(slot)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C"])
def test_unequal_batches_equal_each_request_alone(folders, name, dtype):
    """Requests of different lengths start together, are decoded together and end one after the other; their slots and
    pages go to requests that start later.  Every logit equals the plain model's on that request alone."""
    from nnis_amd.engine.batch import StepEntry

    config = TUGOVIK_CONFIGS[name][0]
    plain = T.PlainTugovik(folders[name, dtype])
    engine = nnis_amd.load_engine(folders[name, dtype], dtype=dtype, max_tokens=64 * 9, max_slots=4)
    yard = Yardstick(plain)
    for batch_seed, lengths in ((0, [1, 70, 130, 9]), (1, [65, 3, 128]), (2, [2, 2, 200, 64])):
        requests = [_ids(n + decode, config["vocab"], 100 * batch_seed + i) for i, (n, decode) in enumerate(zip(lengths, (12, 5, 9, 1)))]
        slots = [engine.start_sequence() for _ in requests]
        at = list(lengths)
        logits = engine.step([StepEntry(s, r[:n], list(range(n))) for s, r, n in zip(slots, requests, lengths)]).cpu()
        row = 0
        for i, n in enumerate(lengths):
            yard.check(logits[row:row + n], requests[i], dtype, f"{name} batch {batch_seed} prompt {i}", rows=slice(0, n))
            row += n
        live = list(range(len(requests)))
        while live:
            live = [i for i in live if at[i] < len(requests[i]) or engine.end_sequence(slots[i])]
            if not live:
                break
            logits = engine.step([StepEntry(slots[i], [requests[i][at[i]]], [0]) for i in live]).cpu()
            for row, i in enumerate(live):
                yard.check(logits[row], requests[i], dtype, f"{name} batch {batch_seed} request {i} position {at[i]}", rows=at[i])
                at[i] += 1
        assert engine.free_slots() == 4 and engine.free_pages() == 9


@pytest.mark.parametrize("dtype", DTYPES)
def test_twenty_sequences_decode_together(folders, dtype):
    """More rows than the kernels for few rows and one tile of sequences take; each logit is the request's own."""
    from nnis_amd.engine.batch import StepEntry

    config = TUGOVIK_CONFIGS["A"][0]
    plain = T.PlainTugovik(folders["A", dtype])
    engine = nnis_amd.load_engine(folders["A", dtype], dtype=dtype, max_tokens=64 * 40, max_slots=20)
    yard = Yardstick(plain)
    requests = [_ids(5 + 4 * i, config["vocab"], 500 + i) for i in range(20)]
    slots = [engine.start_sequence() for _ in requests]
    engine.step([StepEntry(s, r[:-3], []) for s, r in zip(slots, requests)])
    for back in (3, 2, 1):
        logits = engine.step([StepEntry(s, [r[-back]], [0]) for s, r in zip(slots, requests)]).cpu()
        for row, request in enumerate(requests):
            yard.check(logits[row], request, dtype, f"request {row}, {back} from its end", rows=len(request) - back)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_across_chunks_and_pages(tmp_path, dtype):
    """330 tokens one by one behind a prompt of 3: the borders of chunks of 5 and 70 tokens and of five pages are crossed by
    decoded tokens, a third layer sees all of them; states and convolutions' rings go round many times."""
    layers = [layer(attention(2, 1, 16, 16, chunk=5), moe(3, 1, 24)), layer(mamba2(2, 16, 16, 1, 3)), layer(attention(2, 1, 16, 16, chunk=70)),
              layer(rglru(32, 2, 4), moe(4, 2, 16, (2, 1), 1.5, shared=24)), layer(attention(2, 1, 16, 16))]
    config = tugovik(vocab=200, width=64, layers=layers, loop=(1, 4, 2), side=16)
    folder = _folder(tmp_path / "m", config, 7, dtype)
    plain = T.PlainTugovik(folder)
    engine = nnis_amd.load_engine(folder, dtype=dtype, max_tokens=512)
    ids = _ids(330, config["vocab"], 4)
    slot = engine.start_sequence()
    got = _collect(engine, slot, ids, [3] + list(range(4, 331)))
    yard = Yardstick(plain)
    yard.check(got, ids, dtype, "long decoding")
    yard.check(got[-1], ids, dtype, "long decoding, the last token", rows=len(ids) - 1)


@pytest.mark.parametrize("name", sorted(TUGOVIK_CONFIGS))
def test_greedy_generation_through_the_entry_point(folders, name):
    """``nnis_amd.generate``: the library's scheduler, batches and selection on the device.  In 32-bit the tokens are
    the plain model's, unless two logits are closer than rounding."""
    config = TUGOVIK_CONFIGS[name][0]
    plain = T.PlainTugovik(folders[name, "float32"])
    prompts = [_ids(n, config["vocab"], 50 + n) for n in (1, 19, 70)]
    got = nnis_amd.generate(folders[name, "float32"], prompts, max_new_tokens=10, dtype="float32", stop_token_ids=[])
    for prompt, tokens in zip(prompts, got):
        assert len(tokens) == 10
        logits = plain.logits(prompt + tokens)[len(prompt) - 1:-1]
        for row, token in zip(logits, tokens):
            assert float(row[token]) >= float(row.max()) - 1e-4 * float(row.abs().max()), "a generated token is not the plain model's best"
    got16 = nnis_amd.generate(folders[name, "bfloat16"], prompts, max_new_tokens=6, dtype="bfloat16", stop_token_ids=[])
    assert [len(t) for t in got16] == [6, 6, 6]


def test_the_command_line_runs_the_model(folders):
    import subprocess
    import sys

    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    done = subprocess.run([sys.executable, os.path.join(root, "bin", "nnis"), "generate", "--model", folders["B", "float32"], "--prompt-ids", "5,17,3",
                           "--max-new-tokens", "4", "--dtype", "float32"], capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr[-2000:]
    plain = T.PlainTugovik(folders["B", "float32"])
    assert [int(t) for t in done.stdout.strip().splitlines()[-1].split(",")] == plain.greedy([5, 17, 3], 4)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_trace_runner_replays_schedules(folders, tmp_path, dtype):
    """The same requests whole, with their last tokens one by one, and in unequal batches whose slots are used again,
    through ``bin/trace_run`` in a cache too small to hold the schedules side by side."""
    config = TUGOVIK_CONFIGS["A"][0]
    plain = T.PlainTugovik(folders["A", dtype])
    rng = np.random.default_rng(3)
    requests = {f"r{i}": rng.integers(0, config["vocab"], size=n).tolist() for i, n in enumerate([1, 7, 40, 65, 97, 130])}
    schedules = (("w", replay.whole(requests)), ("t", replay.tail_one_by_one(requests)), ("b", replay.unequal_batches(requests, batch=3, decode=32)))
    steps = [{"entries": [dict(e, id=tag + e["id"]) for e in step["entries"]], "end": [tag + n for n in step.get("end", [])]}
             for tag, schedule in schedules for step in schedule]
    rows = replay.run_trace(folders["A", dtype], dtype, steps, str(tmp_path), max_tokens=6 * 64, vocab=config["vocab"])
    yard = Yardstick(plain)
    for tag, _ in schedules:
        for name, ids in requests.items():
            got = np.stack([rows[(tag + name, p)] for p in range(len(ids))])
            yard.check(got, ids, dtype, f"schedule {tag} request {name}")


HEAD_SIZES = [(32, 16), (16, 48), (40, 40), (16, 16)]  # attention modules that are built beforehand


@pytest.mark.parametrize("seed", range(8))
def test_other_sizes_drawn_from_a_seed(tmp_path, seed):
    """Configurations whose every size is drawn at random, in 32-bit against the plain model, and in bfloat16 against its
    rounded twin: prompt, a portion, single tokens."""
    import random

    r = random.Random(seed)
    layers = []
    for _ in range(r.randint(1, 5)):
        kind = r.choice("AMR")
        if kind == "A":
            dim, vdim = r.choice(HEAD_SIZES)
            groups = r.randint(1, 2)
            mixer = attention(r.randint(1, 3) * groups, groups, dim, vdim, scale=r.uniform(0.1, 0.6), chunk=r.choice([None, r.randint(1, 90)]))
        elif kind == "M":
            groups = r.randint(1, 3)
            heads, vdim = groups * r.randint(1, 3), r.choice([8, 16, 12, 32])
            mixer = mamba2(heads, vdim, r.choice([8, 20, 32, 48, 72, 7]), groups, r.randint(1, 5), r.choice([1, heads]))
        else:
            blocks = r.randint(1, 4)
            mixer = rglru(blocks * r.choice([8, 24, 10, 40]), blocks, r.randint(1, 5))
        groups = r.choice([None, (r.randint(2, 3), 1)])
        experts = (groups[0] if groups else 1) * r.randint(1, 4)
        top = r.randint(1, experts // groups[0] if groups else experts)
        mlp = r.choice([None, moe(experts, top, r.randint(4, 40), groups, r.choice([None, r.uniform(0.4, 3.0)]), shared=r.choice([None, r.randint(4, 60)]))])
        layers.append(layer(mixer, mlp))
    start = r.randrange(len(layers))
    config = tugovik(vocab=r.randint(20, 400), width=8 * r.randint(2, 15), layers=layers, loop=r.choice([None, (start, r.randint(start + 1, len(layers)), r.randint(1, 3))]),
                     side=r.choice([None, r.randint(3, 40)]), eps=r.choice([1e-5, 1e-6, 1e-3]))
    ids = _ids(80, config["vocab"], seed)
    for dtype in DTYPES:
        folder = _folder(tmp_path / f"m{seed}{dtype}", config, seed, dtype)
        plain = T.PlainTugovik(folder)
        want, twin = plain.logits(ids), plain.logits(ids, T.bf16_round)
        engine = nnis_amd.load_engine(folder, dtype=dtype, max_tokens=256)
        slot = engine.start_sequence()
        got = _collect(engine, slot, ids, [66, 70] + list(range(71, 81)))
        bound = 5e-5 if dtype == "float32" else 3.0 * max(_relative(twin, want), 3e-3)
        assert _relative(got, want) < bound, f"seed {seed}, {dtype}: {_relative(got, want):.3g} (bound {bound:.3g}) {config}"
