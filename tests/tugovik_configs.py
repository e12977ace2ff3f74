"""Small Tugovik configurations for the tests: every size differs between them
where it can (grouped heads 2:1, 3:1, 4:1 and 1:1; values narrower and wider
than the keys; chunks shorter and longer than a page, of one position, and
none; state spaces whose channels and states the matrix cores take and others;
1 to 4 groups, norms in 1 to 4 parts; recurrent units of 1 to 4 parts; 1 to 4
taps; routers with groups of 2 and 3 experts and without; a shared expert of
another size and none; layers without a feed-forward; stretches of layers that
run again; inputs of the tokens' own and none)."""


def attention(heads, kv_heads, dim, vdim, scale=0.3, chunk=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk:
        mixer["mask"] = {"size": chunk}
    return "attention", mixer


def mamba2(heads, vdim, state, groups=1, conv=4, norm_groups=1):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}


def rglru(width, blocks, conv=4):
    return "rglru", {"width": width, "blocks": blocks, "conv": conv}


def moe(experts, top, ff, groups=None, scale=None, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if groups is not None:
        out["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if scale is not None:
        out["router"]["scale"] = scale
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer, mlp=None):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


def tugovik(vocab, width, layers, loop=None, side=None, eps=1e-5):
    out = {"architecture": "Tugovik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    if side is not None:
        out["token_side"] = {"dim": side}
    return out


# all three mixers, the middle of the order twice; groups of two experts, a shared one; inputs of the tokens' own
TUG_A = tugovik(300, 96, [
    layer(attention(4, 2, 32, 16, chunk=37), moe(6, 2, 24, (3, 2), 2.0, shared=40)), layer(mamba2(6, 16, 24, 3, 4, 2), moe(5, 2, 16, None, 1.25, shared=24)),
    layer(rglru(72, 3)), layer(attention(3, 1, 16, 48, scale=0.4, chunk=70), moe(4, 1, 32))], loop=(1, 3, 2), side=24)
# sizes that the general kernels take; a chunk of one position; no loop, no inputs of the tokens' own
TUG_B = tugovik(257, 64, [
    layer(mamba2(3, 20, 12, 1, 2), moe(3, 1, 40, None, 0.7)), layer(rglru(60, 1, 3)), layer(attention(2, 2, 16, 16, scale=0.2, chunk=1), moe(8, 3, 16, (2, 1))),
    layer(mamba2(2, 8, 40, 2, 1, 1), moe(2, 2, 24, shared=24)), layer(attention(2, 1, 16, 16))], eps=3e-6)
# the whole order three times, groups of three experts of which one is kept, no mask
TUG_C = tugovik(512, 128, [
    layer(rglru(64, 4), moe(9, 3, 40, (3, 1), 1.75, shared=72)), layer(mamba2(2, 32, 64, 2, 3, 4)),
    layer(attention(4, 1, 16, 16, scale=0.25), moe(4, 2, 16, (4, 3), 0.9))], loop=(0, 3, 3), side=8)

TUGOVIK_CONFIGS = {"A": (TUG_A, 61), "B": (TUG_B, 62), "C": (TUG_C, 79)}
