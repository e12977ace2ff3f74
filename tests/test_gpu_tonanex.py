"""Tonanex on the GPU against the plain implementation (``plain_tonanex``):
each mechanism alone, then whole models through the engine -- prompts whole, in
portions and token by token, unequal batches, slots and pages used again, keys
far away, at page borders and at the window's edge, long decoding, greedy
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
import plain_tonanex as T
import replay
from gpu_helpers import cache_for, context, runtime
from tonanex_configs import TONANEX_CONFIGS, again, attention, dense, layer, moe, tonanex

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


# ---------------------------------------------------------------------------------------------
# the mechanisms alone
# ---------------------------------------------------------------------------------------------

@pytest.mark.parametrize("packed", [False, True])
@pytest.mark.parametrize("tokens, width, scale", [(1, 8, 1.0), (37, 56, 3.0), (5, 1032, 1.0), (3, 4096, 0.5), (2, 8456, 1.0)])
def test_a_normed_embedding(packed, tokens, width, scale):
    from nnis_amd.kernels import ops

    generator = torch.Generator().manual_seed(tokens + width)
    table = torch.randn(50, width, generator=generator).to(torch.bfloat16)
    weight = (1.0 + 0.3 * torch.randn(width, generator=generator)).to(torch.bfloat16)
    ids = torch.randint(0, 50, (tokens,), generator=generator, dtype=torch.int32)
    want = T.rms_norm(table.double()[ids.long()] * scale, weight.double(), 1e-5)
    held = ops.pack_weight(table.cuda()) if packed else table.cuda()
    got = ops.embed_norm(ids.cuda(), held, weight.cuda(), 1e-5, torch.empty(tokens, width, device="cuda"), scale)
    assert _relative(got.cpu(), want) < 1e-6
    if not packed:
        got = ops.embed_norm(ids.cuda(), table.float().cuda(), weight.float().cuda(), 1e-5, torch.empty(tokens, width, device="cuda"), scale)
        assert _relative(got.cpu(), want) < 1e-6
    ids[0] = -1  # a padding row
    got = ops.embed_norm(ids.cuda(), held, weight.cuda(), 1e-5, torch.empty(tokens, width, device="cuda"), scale)
    assert not bool(got[0].any())


def _attention_part(sizes, width, eps=1e-5):
    from nnis_amd.parts import build_part

    return build_part("mixer", dict(kind="causal_attention", width=width, heads=sizes["heads"], kv_heads=sizes["kv_heads"], head_dim=sizes["dim"],
                                    value_dim=sizes["vdim"], scale=sizes["scale"], window=(sizes.get("mask") or {}).get("size"), unit_heads=eps,
                                    temperature="temp", decay=("r1", "r2"), head_gate="g", q="q", k="k", v="v", o="o"))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, kv_heads, dim, vdim, window, width", [
    (4, 2, 32, 16, 37, 64), (6, 1, 16, 48, 70, 48), (2, 2, 32, 16, 1, 96), (3, 3, 16, 48, 64, 56), (6, 2, 24, 40, 33, 40), (2, 1, 16, 16, None, 56),
    (20, 1, 16, 16, 130, 64), (1, 1, 32, 16, None, 24)])
def test_attention_alone(dtype, heads, kv_heads, dim, vdim, window, width):
    """Grouped heads, values of their own size, heads over their root mean square, temperatures (one of them negative),
    scores that fall with the distance by numbers that matter, gates that matter.  Whole prompts; then portions down to
    two tokens and single tokens across the borders of pages and of the window; three unequal sequences in every step."""
    rt = runtime(dtype)
    sizes = attention(heads, kv_heads, dim, vdim, scale=0.4, window=window)
    mixer = _attention_part(sizes, width)
    plain_w, part_w = _weights(mixer, dtype, 3, scale={"g": 20.0, "v": 5.0, "o": 5.0, "temp": 1.5})
    for w in (plain_w, part_w):
        w["temp"][0] = -1.25
        w["r2"][heads - 1] = 4.0
    mixer.check(rt)
    mixer.bind(part_w, rt)
    cache = cache_for([mixer.cache_request()], rt, max_tokens=1024, max_positions=512)
    generator = torch.Generator().manual_seed(5)
    lengths = [200, 3, 67]
    xs = [torch.randn(n, width, generator=generator).to(torch.bfloat16).double() for n in lengths]
    rnd = _rounding(dtype)
    want = [T.attention(x, plain_w, sizes, 1e-5, rnd) for x in xs]
    for name in ("temp", "r1", "r2", "g"):  # every number of the heads moves the output
        other = dict(plain_w, **{name: plain_w[name] * 0.5})
        if window != 1 or name == "g":
            assert _relative(T.attention(xs[0], other, sizes, 1e-5, rnd), want[0]) > 1e-2, name
    for cuts in ([[200], [3], [67]], [[61, 63, 64, 66, 128, 130, 131, 200], [1, 2, 3], [2, 4, 64, 65, 66, 67]],
                 [[150] + list(range(151, 201)), [3], [60] + list(range(61, 68))]):
        got = _run_in_steps(lambda x, ctx: mixer.forward(x, ctx, cache.view(0), rt), cache, rt, xs, cuts)
        for g, w, n in zip(got, want, lengths):
            _close(g, w, dtype, f"attention {cuts[0][:2]} length {n}", bf16=4e-2)


def _reading_attention(dtype, window, heads=1, kv_heads=1, width=32, dim=32, vdim=16, max_tokens=2048, r1=0.5, r2=0.25):
    """Heads whose queries read the input's first eight channels and whose keys read the next eight, so that a token whose
    key channels are set takes the weight of a query whose query channels are set.  The keys also read channel 16, which
    ``_quiet_input`` sets to one in every token: the norm of a key then leaves an unmarked token's eight channels as small
    as they were, where without it they would be noise of a mark's size."""
    rt = runtime(dtype)
    sizes = attention(heads, kv_heads, dim, vdim, scale=0.5, window=window)
    mixer = _attention_part(sizes, width)
    plain_w, part_w = _weights(mixer, dtype, 11, scale={"v": 20.0, "o": 20.0})
    reads = {"q": torch.zeros(dim, width, dtype=torch.float64), "k": torch.zeros(dim, width, dtype=torch.float64)}
    reads["q"][:8, :8] = torch.eye(8, dtype=torch.float64)
    reads["k"][:8, 8:16] = torch.eye(8, dtype=torch.float64)
    reads["k"][8, 16] = 1.0
    for name, count in (("q", heads), ("k", kv_heads)):
        plain_w[name] = reads[name].repeat(count, 1)
        part_w[name] = plain_w[name].to(part_w[name].dtype).cuda()
    for name, value in (("temp", 1.0), ("r1", r1), ("r2", r2)):
        plain_w[name] = torch.full((heads,), value, dtype=torch.float64)
        part_w[name] = plain_w[name].to(part_w[name].dtype).cuda()
    mixer.bind(part_w, rt)
    cache = cache_for([mixer.cache_request()], rt, max_tokens=max_tokens, max_positions=1024)
    return rt, sizes, mixer, plain_w, cache


def _quiet_input(n, width, generator, mark, last):
    x = (0.002 * torch.randn(n, width, generator=generator)).to(torch.bfloat16).double()
    x[:, 16] = 1.0
    x[mark, 8:16] = 8.0  # the norms make a marked key and the last query of size 2 a channel: a score of 0.5 * 32, against scores near 0
    x[last, :8] = 8.0
    return x


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window, heads, kv_heads", [(37, 1, 1), (64, 6, 1), (65, 2, 2), (128, 1, 1), (9, 1, 1)])
def test_the_windows_edge_decides(dtype, window, heads, kv_heads):
    """The marked token stands just inside the window and just outside it, at page borders too; the last token comes in a
    prompt, in a portion, and alone.  The output tells the two apart."""
    rt, sizes, mixer, plain_w, cache = _reading_attention(dtype, window, heads, kv_heads)
    width = 32
    generator = torch.Generator().manual_seed(1)
    for n in (180, 192, 193):
        share = {}
        for what, place in (("inside", n - window), ("outside", n - window - 1)):
            x = _quiet_input(n, width, generator, place, n - 1)
            want = T.attention(x, plain_w, sizes, 1e-5)
            without = x.clone()
            without[place, 8:16] = x[place - 1, 8:16]
            share[what] = _relative(T.attention(without, plain_w, sizes, 1e-5)[n - 1], want[n - 1])
            for cuts in ([n], [n - 3, n], [n - 1, n], [100] + list(range(101, n + 1))):
                got = _run_in_steps(lambda h, ctx: mixer.forward(h, ctx, cache.view(0), rt), cache, rt, [x], [cuts])[0]
                _close(got[n - 1], want[n - 1], dtype, f"mark {what} at {place} (window {window}, {n} tokens), cuts {cuts[:2]}")
                _close(got, want, dtype, f"mark {what} at {place}, all tokens, cuts {cuts[:2]}")
        assert share["inside"] > 0.3 and share["outside"] < 1e-6, share


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads, kv_heads", [(1, 1), (6, 1)])
def test_a_far_key_counts_at_its_distance(dtype, heads, kv_heads):
    """Without a window the marked token lies up to 800 tokens back, at page borders too, and competes with a second mark
    nearby: the weights between the two follow the distances.  Prompts, portions and single tokens; the plan of the decode
    step cuts such lengths into runs of keys."""
    rt, sizes, mixer, plain_w, cache = _reading_attention(dtype, None, heads, kv_heads, r1=0.4, r2=0.5)
    width, n = 32, 810
    generator = torch.Generator().manual_seed(2)
    for far, near in ((0, 800), (63, 700), (64, 640), (500, 801), (745, 746)):
        x = _quiet_input(n, width, generator, far, n - 1)
        x[near, 8:16] = 8.0
        x[far, 20] = x[near, 21] = 24.0  # (their values differ)
        want = T.attention(x, plain_w, sizes, 1e-5)
        without = x.clone()
        without[far, 8:16] = 0.0
        assert _relative(T.attention(without, plain_w, sizes, 1e-5)[n - 1], want[n - 1]) > 0.05  # the far key counts
        flat = T.attention(x, dict(plain_w, r1=plain_w["r1"] * 0.0), sizes, 1e-5)
        if near - far > 100:
            assert _relative(flat[n - 1], want[n - 1]) > 0.05
        for cuts in ([n], [n - 2, n], [n - 1, n], [790] + list(range(791, n + 1))):
            got = _run_in_steps(lambda h, ctx: mixer.forward(h, ctx, cache.view(0), rt), cache, rt, [x], [cuts])[0]
            _close(got[n - 1], want[n - 1], dtype, f"far key at {far}, cuts {cuts[:2]}", bf16=2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_decay_beside_the_other_options_of_the_scores(dtype):
    """A cap, kept first keys, a sink, the decay and gates in one module: the cap bends the scaled score before the decay
    is taken off, the sink and the kept keys are as without it."""
    from nnis_amd.parts import build_part

    rt = runtime(dtype)
    heads, kv_heads, dim, vdim, window, keep, cap, width = 4, 2, 32, 16, 20, 3, 4.0, 48
    mixer = build_part("mixer", dict(kind="causal_attention", width=width, heads=heads, kv_heads=kv_heads, head_dim=dim, value_dim=vdim, scale=0.4,
                                     window=window, keep_first=keep, softcap=cap, sink="sink", unit_heads=1e-5, temperature="temp",
                                     decay=("r1", "r2"), head_gate="g", q="q", k="k", v="v", o="o"))
    plain_w, part_w = _weights(mixer, dtype, 7, scale={"g": 20.0, "v": 5.0, "o": 5.0, "sink": 50.0})
    mixer.bind(part_w, rt)
    cache = cache_for([mixer.cache_request()], rt, max_tokens=512, max_positions=512)
    rnd = _rounding(dtype)
    n = 150
    x = torch.randn(n, width, generator=torch.Generator().manual_seed(3)).to(torch.bfloat16).double()
    q = rnd(T.unit_rms(rnd(x @ plain_w["q"].T).view(n, heads, dim), 1e-5) * plain_w["temp"][None, :, None])
    k = rnd(T.unit_rms(rnd(x @ plain_w["k"].T).view(n, kv_heads, dim), 1e-5))
    v = rnd(x @ plain_w["v"].T).view(n, kv_heads, vdim)
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    seen = (j <= i) & ((i - j < window) | (j < keep))
    out = torch.zeros(n, heads, vdim, dtype=torch.float64)
    for head in range(heads):
        s = q[:, head] @ k[:, head // 2].T * 0.4
        s = cap * torch.tanh(s / cap) - T.distance_bias(plain_w["r1"][head], plain_w["r2"][head], (i - j).clamp_min(0).double())
        e = torch.exp(torch.where(seen, s, torch.full_like(s, -float("inf"))))
        p = e / (e.sum(dim=1, keepdim=True) + torch.exp(plain_w["sink"][head]))
        out[:, head] = p @ v[:, head // 2] * T.sigmoid(rnd(x @ plain_w["g"].T))[:, head, None]
    want = rnd(out.reshape(n, heads * vdim)) @ plain_w["o"].T
    for cuts in ([n], [70, 72, n], [100] + list(range(101, n + 1))):
        got = _run_in_steps(lambda h, ctx: mixer.forward(h, ctx, cache.view(0), rt), cache, rt, [x], [cuts])[0]
        _close(got, want, dtype, f"cuts {cuts[:2]}", bf16=4e-2)


@pytest.mark.parametrize("outputs, top, rows, width", [(5, 2, 40, 96), (3, 1, 300, 64), (70, 4, 260, 200), (1, 1, 7, 8), (4, 4, 33, 1030)])
def test_the_router_weighs_over_the_chosen_logits(outputs, top, rows, width):
    """Weights are the softmax over the chosen logits, a bias among them; as dense gates and as lists; from normed rows and
    from a stream that the kernel norms itself (a part's output still to be added to it)."""
    from nnis_amd.kernels import ops

    generator = torch.Generator().manual_seed(outputs)
    stream = torch.randn(rows, width, generator=generator)
    delta = torch.randn(rows, width, generator=generator).to(torch.bfloat16)
    gain = (1.0 + 0.2 * torch.randn(width, generator=generator)).to(torch.bfloat16)
    w, bias = torch.randn(outputs, width, generator=generator), 2.0 * torch.randn(outputs, generator=generator)
    total = stream.double() + delta.double()
    h = T.rms_norm(total, gain.double(), 1e-5)
    wanted, weights = T.choose(h, {"router": w.double(), "router.b": bias.double()}, top)
    z = (h @ w.double().T + bias.double()).sort(dim=1, descending=True).values
    clear = torch.ones(rows, dtype=torch.bool) if top == outputs else (z[:, top - 1] - z[:, top] > 1e-3)
    assert float(clear.float().mean()) > 0.95
    dense_want = torch.zeros(rows, outputs, dtype=torch.float64).scatter(1, wanted, weights)
    if outputs > top:
        bare = torch.topk(h @ w.double().T, top, dim=1).indices
        assert outputs == 1 or rows < 10 or bool((bare.sort(dim=1).values != wanted.sort(dim=1).values).any())  # the bias decides some

    def check(gates, chosen):
        assert float((gates.cpu().double() - dense_want).abs()[clear].max()) < 2e-5
        if top < outputs or top == 1:
            assert torch.equal(chosen[0].cpu().long()[clear][:, 0], wanted[clear][:, 0])  # the best first
        listed = torch.zeros(rows, outputs, dtype=torch.float64).scatter(1, chosen[0].cpu().long(), chosen[1].cpu().double())
        assert float((listed - dense_want).abs()[clear].max()) < 2e-5

    def made():
        return (torch.empty(rows, outputs, device="cuda"), torch.empty(rows, device="cuda"),
                (torch.empty(rows, top, dtype=torch.int32, device="cuda"), torch.empty(rows, top, device="cuda")))

    rule = dict(bias=bias.cuda(), scoring="chosen_softmax")
    gates, keep, chosen = made()
    ops.route(h.float().cuda(), w.cuda(), None, outputs, top, gates, keep, chosen=chosen, **rule)
    check(gates, chosen)
    logits = ops.router_logits(h.float().cuda(), w.cuda(), torch.empty(rows, outputs, device="cuda"))
    apart, keep = ops.route_top(logits, None, outputs, top, torch.empty(rows, outputs, device="cuda"), keep, **rule)
    assert float((apart - gates)[clear.cuda()].abs().max()) < 1e-4
    for h_dtype in (torch.float32, torch.bfloat16):
        gates, keep, chosen = made()
        x = stream.clone().cuda()
        got = ops.route_norm(x, delta.cuda(), gain.cuda(), 1e-5, torch.empty(rows, width, device="cuda", dtype=h_dtype), w.cuda(), None, outputs,
                             top, gates, keep, chosen=chosen, **rule)
        check(gates, chosen)
        assert _relative(x.cpu(), total) < 1e-6 and _relative(got.float().cpu(), h) < (1e-6 if h_dtype == torch.float32 else 4e-3)
        ops.route_norm(x, None, gain.cuda(), 1e-5, got, w.cuda(), None, outputs, top, gates, keep, **rule)  # the sum is in the stream now
        check(gates, chosen)
        assert _relative(x.cpu(), total) < 1e-6


ROUTED_SIZES = [  # width, inner, experts, top, limit, shared, its limit
    (64, 24, 5, 2, 1.0, 40, 0.7), (48, 64, 3, 1, None, None, None), (96, 16, 9, 3, 0.5, 16, 0.5), (40, 72, 70, 4, 2.0, 136, None),
    (128, 8, 2, 2, 7.0, 8, 1.0), (8, 8, 1, 1, 1.0, None, None)]


def _routed(width, inner, experts, top, limit, shared, shared_limit, dtype):
    from nnis_amd.parts import build_part

    rt = runtime(dtype)
    description = dict(kind="routed", width=width, inner=inner, experts=experts, top=top, scoring="chosen_softmax", activation="clamped_swiglu",
                       limit=limit, router="router", router_bias="router.b", gate="e{}.gate", up="e{}.up", down="e{}.down")
    if shared is not None:
        description["shared"] = dict(inner=shared, limit=shared_limit, gate="shared.gate", up="shared.up", down="shared.down")
    part = build_part("feed_forward", description)
    plain_w, part_w = _weights(part, dtype, 3, scale={"router.b": 10.0, ".gate": 10.0, ".up": 10.0, ".down": 10.0})
    part.check(rt)
    part.bind(part_w, rt)
    mlp = {"router": {"experts": experts, "top": top}, "expert": {"limit": float("inf") if limit is None else limit}}
    if shared is not None:
        mlp["shared"] = {"limit": float("inf") if shared_limit is None else shared_limit}
    return rt, part, plain_w, mlp


def _clear(x, plain_w, top, margin=1e-2):
    z = (x @ plain_w["router"].T + plain_w["router.b"]).sort(dim=1, descending=True).values
    return torch.ones(x.shape[0], dtype=torch.bool) if top == z.shape[1] else (z[:, top - 1] - z[:, top] > margin)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", ROUTED_SIZES)
def test_routed_feed_forward_alone(dtype, sizes):
    """All three ways through the experts' products: few rows (experts that nobody chose are left out), some (all experts
    multiplied), many (every expert's rows gathered), 1 to 700 rows, row counts at and around a tile's."""
    rt, part, plain_w, mlp = _routed(*sizes, dtype)
    width, top = sizes[0], sizes[3]
    for rows in (1, 2, 7, 15, 16, 17, 70, 95, 96, 257, 320, 321, 700):
        x = torch.randn(rows, width, generator=torch.Generator().manual_seed(rows)).to(torch.bfloat16).double()
        want, chosen = T.routed_feed_forward(x, plain_w, mlp, _rounding(dtype))
        clear = _clear(x, plain_w, top)
        assert float(clear.float().mean()) > 0.8
        got = part.forward(x.to(rt.dtype).cuda(), None, rt).float().cpu()
        _close(got[clear], want[clear], dtype, f"{rows} rows", bf16=2e-2)
        if rows == 700:
            assert len(set(chosen.flatten().tolist())) > sizes[2] // 2
            unheld = T.routed_feed_forward(x, plain_w, dict(mlp, expert={"limit": float("inf")}), _rounding(dtype))[0]
            assert sizes[4] is None or sizes[4] > 5.0 or _relative(unheld, want) > 1e-2  # the limit holds something back


@pytest.mark.parametrize("rows", [5, 16, 60, 100, 400])
@pytest.mark.parametrize("who", ["one", "two of many", "all"])
def test_experts_under_uneven_routing(rows, who):
    """Every token chooses the same expert (its tiles are full, all others empty), two experts take all tokens, or every
    expert is everybody's: what the router chose decides what is multiplied, and no row is lost or counted twice."""
    sizes = (64, 40, 6, 6 if who == "all" else (1 if who == "one" else 2), 1.0, 24, 2.0)
    rt, part, plain_w, mlp = _routed(*sizes, "bfloat16")
    favour = torch.zeros(6, dtype=torch.float64)
    favour[{"one": [4], "two of many": [0, 5], "all": []}[who]] = 100.0
    plain_w["router.b"] = favour
    part.router_bias = favour.float().cuda()
    x = torch.randn(rows, 64, generator=torch.Generator().manual_seed(rows)).to(torch.bfloat16).double()
    want, chosen = T.routed_feed_forward(x, plain_w, mlp, T.bf16_round)
    assert set(chosen.flatten().tolist()) == {"one": {4}, "two of many": {0, 5}, "all": set(range(6))}[who]
    _close(part.forward(x.to(torch.bfloat16).cuda(), None, rt), want, "bfloat16", f"{rows} rows, {who}", bf16=2e-2)


def test_experts_with_more_tiles_than_blocks_at_once():
    """So many rows that a block of the tiled products takes two column blocks one after the other, and the last run of a
    row block (three column blocks, the last one part full) only one."""
    rt, part, plain_w, mlp = _routed(648, 264, 20, 3, 1.0, 136, 2.0, "bfloat16")
    x = torch.randn(3000, 648, generator=torch.Generator().manual_seed(6)).to(torch.bfloat16).double()
    want = T.routed_feed_forward(x, plain_w, mlp, T.bf16_round)[0]
    clear = _clear(x, plain_w, 3)
    assert float(clear.float().mean()) > 0.8
    got = part.forward(x.to(torch.bfloat16).cuda(), None, rt).float().cpu()
    _close(got[clear], want[clear], "bfloat16", "3000 rows", bf16=2e-2)
    apart = torch.cat([part.forward(x[i:i + 300].to(torch.bfloat16).cuda(), None, rt).float().cpu() for i in range(0, 3000, 300)])
    _close(got, apart.double(), "bfloat16", "in ten parts", bf16=1e-2)


@pytest.mark.parametrize("rows", [1, 9, 16, 40, 100, 333])
def test_experts_end_in_the_residual_stream(rows):
    """The last kernel adds to the 32-bit stream and prepares the norm that follows: what the next projection then makes
    of it equals norm and product apart."""
    from nnis_amd.parts import build_part
    from nnis_amd.parts.lazy import PendingNorm, ResidualInto
    from nnis_amd.parts.linear import Projection

    sizes = (96, 40, 5, 2, 1.0, 72, 2.0)
    rt, part, plain_w, mlp = _routed(*sizes, "bfloat16")
    generator = torch.Generator().manual_seed(rows)
    stream = torch.randn(rows, 96, generator=generator)
    norms = []
    for name in ("one", "two"):
        weight = (1.0 + 0.2 * torch.randn(96, generator=generator)).to(torch.bfloat16)
        norm = build_part("norm", {"kind": "rms", "width": 96, "eps": 1e-5, "weight": name})
        norm.bind({name: weight.cuda()}, rt)
        norms.append((norm, weight.double()))
    w = torch.randn(50, 96, generator=generator).to(torch.bfloat16)
    h = T.bf16_round(T.rms_norm(stream.double(), norms[0][1], 1e-5))
    clear = _clear(T.rms_norm(stream.double(), norms[0][1], 1e-5), plain_w, 2)
    total = stream.double() + T.routed_feed_forward(h, plain_w, mlp, T.bf16_round)[0]
    want = T.rms_norm(total, norms[1][1], 1e-5) @ w.double().T
    pending = PendingNorm(norms[0][0], stream.clone().cuda(), None, rt)
    out = part.forward(pending, None, rt, into=ResidualInto(pending, norms[1][0], rt))
    assert isinstance(out, PendingNorm) and out.norm is norms[1][0]
    assert _relative(out.residual.cpu()[clear], total[clear]) < 1e-2
    projection = Projection(w.cuda(), rt)
    got = out.fused(projection.weight, rt.empty(rows, 50), rt.ops.EPILOGUE_STORE)
    _close(got[clear.cuda()], want[clear], "bfloat16", "the next projection", bf16=2e-2)


def test_expert_kernels_refuse_sizes_that_do_not_fit():
    from nnis_amd.errors import KernelError

    rt, part, _, _ = _routed(64, 24, 5, 2, 1.0, 40, 0.7, "bfloat16")
    ops, x = rt.ops, torch.zeros(17, 64, dtype=torch.bfloat16, device="cuda")
    gates, out = torch.zeros(17, 5, device="cuda"), torch.empty(17, 64, dtype=torch.bfloat16, device="cuda")
    with pytest.raises(KernelError):
        ops.experts_few(x, part.up.weight, part.down.weight, part.regions, gates, out)  # more rows than the few
    with pytest.raises(KernelError):
        ops.experts_few(x[:4], part.up.weight, part.down.weight, ops.ExpertRegions(4, 64, 64, "clamped_swiglu", 1.0, 1.0), gates[:4, :4].contiguous(), out[:4])
    with pytest.raises(KernelError):
        ops.experts_many(x, part.up.weight, part.down.weight, part.regions, torch.zeros(17, 6, dtype=torch.int32, device="cuda"),
                         torch.zeros(17, 6, device="cuda"), out)  # more choices than experts


# ---------------------------------------------------------------------------------------------
# whole models through the engine
# ---------------------------------------------------------------------------------------------

def _sharpen(folder):
    """A random model's weights are too small for its mixers to matter.  Gates, values and the experts' projections are
    scaled so that each matters and limits are met; routers so that few choices are close; the table so that logits are of
    order one to ten."""
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    for key in tensors:
        if key.endswith(".mix.g"):
            factor = 20.0
        elif key.endswith((".mix.v", ".mix.o", ".up", ".gate", ".down")):
            factor = 7.0
        elif key.endswith((".mlp.router", ".mix.temp")):
            factor = 2.0
        elif key.endswith(".router.b") or key == "embed":
            factor = 10.0
        else:
            continue
        tensors[key] = (tensors[key].float() * factor).to(torch.bfloat16)
    save_file(tensors, path)


def _folder(path, config, seed):
    nnis_amd.write_random_model(str(path), config, seed)
    _sharpen(str(path))
    return str(path)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: _folder(tmp_path_factory.mktemp(f"tonanex_{name}"), config, seed) for name, (config, seed) in TONANEX_CONFIGS.items()}


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
            assert 1e-4 < self.known[key][1] < 0.3, self.known[key][1]
        return self.known[key]

    def check(self, got, ids, dtype, what, rows=None):
        want, overall, worst = self.twin(ids)
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
@pytest.mark.parametrize("name", sorted(TONANEX_CONFIGS))
def test_the_stream_after_every_layer(folders, name, dtype):
    from nnis_amd.engine.batch import StepEntry
    from nnis_amd.parts.lazy import PendingNorm

    plain = T.PlainTonanex(folders[name])
    engine = nnis_amd.load_engine(folders[name], dtype=dtype, max_tokens=256)
    ids = _ids(90, TONANEX_CONFIGS[name][0]["vocab"], 8)
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
    assert len(seen) == len(want) == len(TONANEX_CONFIGS[name][0]["layers"])
    for run, (got, expected, rounded) in enumerate(zip(seen, want, twin)):
        assert _relative(got.cpu(), expected) < (1e-5 if dtype == "float32" else max(1e-2, 3.0 * _relative(rounded, expected))), f"layer {run}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(TONANEX_CONFIGS))
def test_prompts_whole_in_portions_and_token_by_token(folders, name, dtype):
    config = TONANEX_CONFIGS[name][0]
    plain = T.PlainTonanex(folders[name])
    engine = nnis_amd.load_engine(folders[name], dtype=dtype, max_tokens=1024)
    ids = _ids(230, config["vocab"], 1)
    yard = Yardstick(plain)
    for cuts in ([230], [2, 4, 5, 63, 64, 66, 128, 129, 150], [100] + list(range(101, 151)), list(range(1, 41)), [200, 230]):
        slot = engine.start_sequence()
        got = _collect(engine, slot, ids, cuts)
        engine.end_sequence(slot)
        yard.check(got, ids, dtype, f"{name} cuts {cuts[:3]}..", rows=slice(0, cuts[-1]))
        for place in (0, 1, 2, cuts[-1] - 1):  # every position by itself, the first tokens among them
            yard.check(got[place], ids, dtype, f"{name} cuts {cuts[:3]}.. position {place}", rows=place)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C"])
def test_unequal_batches_equal_each_request_alone(folders, name, dtype):
    """Requests of different lengths start together, are decoded together and end one after the other; their slots and
    pages go to requests that start later.  Every logit equals the plain model's on that request alone."""
    from nnis_amd.engine.batch import StepEntry

    config = TONANEX_CONFIGS[name][0]
    plain = T.PlainTonanex(folders[name])
    engine = nnis_amd.load_engine(folders[name], dtype=dtype, max_tokens=64 * 9, max_slots=4)
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
    """More rows than the kernels for few rows take: a decode step multiplies all experts, and each logit is the request's own."""
    from nnis_amd.engine.batch import StepEntry

    config = TONANEX_CONFIGS["A"][0]
    plain = T.PlainTonanex(folders["A"])
    engine = nnis_amd.load_engine(folders["A"], dtype=dtype, max_tokens=64 * 40, max_slots=20)
    yard = Yardstick(plain)
    requests = [_ids(5 + 4 * i, config["vocab"], 500 + i) for i in range(20)]
    slots = [engine.start_sequence() for _ in requests]
    engine.step([StepEntry(s, r[:-3], []) for s, r in zip(slots, requests)])
    for back in (3, 2, 1):
        logits = engine.step([StepEntry(s, [r[-back]], [0]) for s, r in zip(slots, requests)]).cpu()
        for row, request in enumerate(requests):
            yard.check(logits[row], request, dtype, f"request {row}, {back} from its end", rows=len(request) - back)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_across_windows_and_pages(tmp_path, dtype):
    """330 tokens one by one behind a prompt of 3: windows of 5 and 70 tokens pass over decoded tokens, a third layer sees
    all of them; five page borders are crossed."""
    layers = [layer(attention(2, 1, 16, 16, window=5), dense(40)), layer(attention(2, 1, 16, 16, window=70), moe(4, 2, 16, 1.0, shared=24, shared_limit=1.0)),
              layer(attention(2, 1, 16, 16))]
    config = tonanex(vocab=200, width=64, layers=layers + [again(layers, 1)], softcap=12.0)
    folder = _folder(tmp_path / "m", config, 7)
    plain = T.PlainTonanex(folder)
    engine = nnis_amd.load_engine(folder, dtype=dtype, max_tokens=512)
    ids = _ids(330, config["vocab"], 4)
    slot = engine.start_sequence()
    got = _collect(engine, slot, ids, [3] + list(range(4, 331)))
    yard = Yardstick(plain)
    yard.check(got, ids, dtype, "long decoding")
    yard.check(got[-1], ids, dtype, "long decoding, the last token", rows=len(ids) - 1)


@pytest.mark.parametrize("name", sorted(TONANEX_CONFIGS))
def test_greedy_generation_through_the_entry_point(folders, name):
    """``nnis_amd.generate``: the library's scheduler, batches and selection on the device.  In 32-bit the tokens are
    the plain model's, unless two logits are closer than rounding."""
    config = TONANEX_CONFIGS[name][0]
    plain = T.PlainTonanex(folders[name])
    prompts = [_ids(n, config["vocab"], 50 + n) for n in (1, 19, 70)]
    got = nnis_amd.generate(folders[name], prompts, max_new_tokens=10, dtype="float32", stop_token_ids=[])
    for prompt, tokens in zip(prompts, got):
        assert len(tokens) == 10
        logits = plain.logits(prompt + tokens)[len(prompt) - 1:-1]
        for row, token in zip(logits, tokens):
            assert float(row[token]) >= float(row.max()) - 1e-4 * float(row.abs().max()), "a generated token is not the plain model's best"
    got16 = nnis_amd.generate(folders[name], prompts, max_new_tokens=6, dtype="bfloat16", stop_token_ids=[])
    assert [len(t) for t in got16] == [6, 6, 6]


def test_the_command_line_runs_the_model(folders):
    import subprocess
    import sys

    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    done = subprocess.run([sys.executable, os.path.join(root, "bin", "nnis"), "generate", "--model", folders["B"], "--prompt-ids", "5,17,3",
                           "--max-new-tokens", "4", "--dtype", "float32"], capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr[-2000:]
    plain = T.PlainTonanex(folders["B"])
    assert [int(t) for t in done.stdout.strip().splitlines()[-1].split(",")] == plain.greedy([5, 17, 3], 4)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_trace_runner_replays_schedules(folders, tmp_path, dtype):
    """The same requests whole, with their last tokens one by one, and in unequal batches whose slots are used again,
    through ``bin/trace_run`` in a cache too small to hold the schedules side by side."""
    config = TONANEX_CONFIGS["A"][0]
    plain = T.PlainTonanex(folders["A"])
    rng = np.random.default_rng(3)
    requests = {f"r{i}": rng.integers(0, config["vocab"], size=n).tolist() for i, n in enumerate([1, 7, 40, 65, 97, 130])}
    schedules = (("w", replay.whole(requests)), ("t", replay.tail_one_by_one(requests)), ("b", replay.unequal_batches(requests, batch=3, decode=32)))
    steps = [{"entries": [dict(e, id=tag + e["id"]) for e in step["entries"]], "end": [tag + n for n in step.get("end", [])]}
             for tag, schedule in schedules for step in schedule]
    rows = replay.run_trace(folders["A"], dtype, steps, str(tmp_path), max_tokens=6 * 64, vocab=config["vocab"])
    yard = Yardstick(plain)
    for tag, _ in schedules:
        for name, ids in requests.items():
            got = np.stack([rows[(tag + name, p)] for p in range(len(ids))])
            yard.check(got, ids, dtype, f"schedule {tag} request {name}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_model_without_the_optional_mechanisms(tmp_path, dtype):
    """No cap of the logits, no window, no limits, no shared expert, a layer without a feed-forward at either end."""
    config = tonanex(vocab=120, width=48, layers=[layer(attention(2, 1, 16, 16)), layer(attention(2, 1, 32, 16), moe(3, 2, 24)), layer(attention(2, 2, 16, 48))])
    folder = _folder(tmp_path / "bare", config, 41)
    plain = T.PlainTonanex(folder)
    engine = nnis_amd.load_engine(folder, dtype=dtype, max_tokens=512)
    ids = _ids(100, config["vocab"], 6)
    slot = engine.start_sequence()
    got = _collect(engine, slot, ids, [70] + list(range(71, 101)))
    Yardstick(plain).check(got, ids, dtype, "a model without the optional mechanisms")


HEAD_SIZES = [(32, 16), (16, 48), (24, 40), (16, 16)]  # attention modules that are built beforehand


def test_other_sizes_drawn_from_a_seed(tmp_path):
    """Configurations whose every size is drawn at random, in 32-bit against the plain model: prompt, a portion, single tokens."""
    import random

    for seed in range(6):
        r = random.Random(seed)
        layers = []
        for index in range(r.randint(1, 5)):
            if layers and r.random() < 0.35:
                layers.append(again(layers, r.randrange(len(layers))))
                continue
            dim, vdim = r.choice(HEAD_SIZES)
            groups = r.randint(1, 2)
            experts = r.randint(1, 6)
            mlp = r.choice([None, dense(r.randint(8, 90)),
                            moe(experts, r.randint(1, experts), r.randint(4, 40), r.choice([None, r.uniform(0.3, 8.0)]),
                                shared=r.choice([None, r.randint(4, 60)]), shared_limit=r.choice([None, r.uniform(0.3, 8.0)]))])
            layers.append(layer(attention(r.randint(1, 3) * groups, groups, dim, vdim, scale=r.uniform(0.1, 0.6),
                                          window=r.choice([None, r.randint(1, 90)])), mlp))
        config = tonanex(vocab=r.randint(20, 400), width=4 * r.randint(3, 30), layers=layers, softcap=r.choice([None, r.uniform(2.0, 30.0)]),
                         eps=r.choice([1e-5, 1e-6, 1e-3]))
        folder = _folder(tmp_path / f"m{seed}", config, seed)
        plain = T.PlainTonanex(folder)
        engine = nnis_amd.load_engine(folder, dtype="float32", max_tokens=256)
        ids = _ids(80, config["vocab"], seed)
        want = plain.logits(ids)
        slot = engine.start_sequence()
        got = _collect(engine, slot, ids, [66, 70] + list(range(71, 81)))
        assert _relative(got, want) < 5e-5, f"seed {seed}: {config}"
