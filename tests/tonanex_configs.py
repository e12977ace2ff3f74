"""Small Tonanex configurations for the tests: every size differs between them
where it can (grouped heads 2:1, 3:1, 6:1 and 1:1; values narrower and wider
than the keys; windows shorter and longer than a page and none; experts 1 to 3
of 3 to 9, with a shared expert of the same size, of another, and without;
limits that hold much and little back; layers that use another layer's tensors,
an earlier one's, a later one's and by way of a third; layers without a
feed-forward; with and without capped logits)."""


def attention(heads, kv_heads, dim, vdim, scale=0.3, window=None):
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        out["mask"] = {"size": window}
    return out


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit=None, shared=None, shared_limit=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if limit is not None:
        out["expert"]["limit"] = limit
    if shared is not None:
        out["shared"] = {"ff": shared}
        if shared_limit is not None:
            out["shared"]["limit"] = shared_limit
    return out


def layer(mixer, mlp=None):
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def again(layers, index):
    """One more run of layer ``index``'s tensors."""
    return dict(layers[index], weights_of=index)


def tonanex(vocab, width, layers, softcap=None, eps=1e-5):
    out = {"architecture": "Tonanex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if softcap is not None:
        out["logit_softcap"] = softcap
    return out


# experts first; the shared layer runs between others; a layer without a feed-forward
_A = [layer(attention(4, 2, 32, 16, window=37), moe(5, 2, 24, 1.5, shared=40, shared_limit=0.8)), layer(attention(6, 1, 16, 48, scale=0.4, window=70)),
      layer(attention(3, 1, 16, 48, scale=0.25), dense(136))]
TON_A = tonanex(300, 96, [_A[0], _A[1], again(_A, 0), _A[2], dict(_A[1], weights_of=1)], softcap=9.0)
# dense first; no window and windows of 1 and 64; one expert of three; no shared expert; no limit; no cap
_B = [layer(attention(2, 2, 16, 16, scale=0.2, window=64), dense(80)), layer(attention(2, 2, 16, 16, window=1), moe(3, 1, 40)),
      layer(attention(2, 1, 32, 16, scale=0.35), moe(4, 4, 16, 2.5, shared=16, shared_limit=2.5))]
TON_B = tonanex(257, 64, _B + [again(_B, 2)], eps=3e-6)
# a layer whose tensors a later one owns, one that points to it by way of another; head sizes that the row kernel takes
_C = layer(attention(4, 2, 24, 40, scale=0.22, window=20), moe(9, 3, 40, 1.0, shared=72, shared_limit=3.0))
TON_C = tonanex(512, 128, [dict(_C, weights_of=2), layer(attention(3, 3, 32, 16, window=130), dense(72)), _C, dict(_C, weights_of=0)], softcap=30.0)

TONANEX_CONFIGS = {"A": (TON_A, 61), "B": (TON_B, 62), "C": (TON_C, 63)}
