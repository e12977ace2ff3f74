"""Tonanex, plainly: one function a mechanism over whole sequences in 64-bit,
written from the design's equations and sharing nothing with the library.

Notation.  x: the residual stream [tokens, width].  R(v, w) = v / sqrt(mean(v^2)
+ eps) * w.  A layer is x <- x + mixer(R(x, w1)), then, where it has a
feed-forward, x <- x + ff(R(x, w2)).  ``rnd`` rounds where an engine that keeps
activations in bfloat16 rounds them (the identity by default).
"""

import json
import math
import os

import torch
from safetensors.torch import load_file


def identity(x):
    return x


def bf16_round(x):
    return x.to(torch.bfloat16).to(x.dtype)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def rms_norm(v, w, eps):
    return v / torch.sqrt((v * v).mean(dim=-1, keepdim=True) + eps) * w


def unit_rms(v, eps):
    """v over its own root mean square (no weight)."""
    return v / torch.sqrt((v * v).mean(dim=-1, keepdim=True) + eps)


def distance_bias(r1, r2, n):
    """What a score gives up for a key n >= 0 positions back: r1 * ln(1 + r2 n)."""
    return r1 * torch.log1p(r2 * n)


def attention(h, w, sizes, eps, rnd=identity):
    """h [tokens, width].  w: q, k, v, temp, r1, r2, g, o.  Queries and keys head by head over their root mean square;
    s(i, j) = (q_i . k_j) * scale * temp_h - r1_h ln(1 + r2_h (i - j)) for 0 <= i - j < size; softmax over those keys;
    a head's output times sigmoid of its row of Wg h; Wo on the heads' outputs one after the other."""
    n = h.shape[0]
    heads, groups, dim, vdim = sizes["heads"], sizes["kv_heads"], sizes["dim"], sizes["vdim"]
    q = unit_rms(rnd(h @ w["q"].T).view(n, heads, dim), eps)
    k = rnd(unit_rms(rnd(h @ w["k"].T).view(n, groups, dim), eps))
    v = rnd(h @ w["v"].T).view(n, groups, vdim)
    q = rnd(q * w["temp"][None, :, None])
    gates = sigmoid(rnd(h @ w["g"].T))
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    seen = j <= i
    if sizes.get("mask"):
        seen = seen & (i - j < sizes["mask"]["size"])
    back = (i - j).clamp_min(0).to(h.dtype)
    out = torch.zeros(n, heads, vdim, dtype=h.dtype)
    for head in range(heads):
        group = head // (heads // groups)
        s = q[:, head] @ k[:, group].T * sizes["scale"] - distance_bias(w["r1"][head], w["r2"][head], back)
        p = torch.softmax(torch.where(seen, s, torch.full_like(s, -math.inf)), dim=1)
        out[:, head] = (p @ v[:, group]) * gates[:, head, None]
    return rnd(out.reshape(n, heads * vdim)) @ w["o"].T


def dense_feed_forward(h, w, rnd=identity):
    """Wdown (silu(Wgate h) * (Wup h))."""
    a = h @ w["gate"].T
    return rnd(a * sigmoid(a) * (h @ w["up"].T)) @ w["down"].T


def clamped_expert(h, w, limit, rnd=identity):
    """g = min(Wgate h, limit), u = Wup h held in [-limit, limit]; Wdown (g sigmoid(1.702 g) (u + 1))."""
    limit = math.inf if limit is None else limit
    g = torch.clamp(rnd(h @ w["gate"].T), max=limit)
    u = torch.clamp(rnd(h @ w["up"].T), min=-limit, max=limit)
    return rnd(g * sigmoid(1.702 * g) * (u + 1.0)) @ w["down"].T


def choose(h, w, top):
    """z = Wrouter h + b; the ``top`` largest, weighted by a softmax over themselves.  Returns (chosen, weights) [tokens, top]."""
    z = h @ w["router"].T + w["router.b"]
    best = torch.topk(z, top, dim=-1)
    return best.indices, torch.softmax(best.values, dim=-1)


def routed_feed_forward(h, w, mlp, rnd=identity):
    """The chosen experts' outputs, weighted and added; a shared expert, where there is one, added for every token.
    Returns (out, chosen [tokens, top])."""
    chosen, weights = choose(h, w, mlp["router"]["top"])
    out = torch.zeros(h.shape[0], h.shape[1], dtype=h.dtype)
    for e in range(mlp["router"]["experts"]):
        rows, place = torch.nonzero(chosen == e, as_tuple=True)
        if rows.numel():
            out[rows] += weights[rows, place, None] * clamped_expert(h[rows], _sub(w, f"e{e}."), mlp["expert"].get("limit"), rnd)
    if mlp.get("shared"):
        out = out + clamped_expert(h, _sub(w, "shared."), mlp["shared"].get("limit"), rnd)
    return out, chosen


def _sub(weights, prefix):
    return {name[len(prefix):]: value for name, value in weights.items() if name.startswith(prefix)}


def owner(layers, index):
    """The layer whose tensors layer ``index`` uses."""
    while layers[index].get("weights_of") is not None:
        index = layers[index]["weights_of"]
    return index


class PlainTonanex:
    """The whole model over one sequence from its first token, from a folder with config.json and model.safetensors."""

    def __init__(self, folder):
        with open(os.path.join(folder, "config.json")) as handle:
            self.config = json.load(handle)
        self.w = {name: value.double() for name, value in load_file(os.path.join(folder, "model.safetensors")).items()}

    def logits(self, ids, rnd=identity, stream_after=None):
        """Logits [tokens, vocab]; ``stream_after`` (a list) gets the stream after every layer."""
        cfg, w = self.config, self.w
        eps = cfg["norm"]["eps"]
        x = rms_norm(w["embed"][torch.as_tensor(list(ids), dtype=torch.long)], w["embed.norm"], eps)
        for index, layer in enumerate(cfg["layers"]):
            prefix = f"l{owner(cfg['layers'], index)}."
            h = rnd(rms_norm(x, w[prefix + "norm1"], eps))
            x = x + rnd(attention(h, _sub(w, prefix + "mix."), layer["mixer"], eps, rnd))
            mlp = layer.get("mlp")
            if mlp is not None:
                h = rnd(rms_norm(x, w[prefix + "norm2"], eps))
                if mlp["kind"] == "dense":
                    y = dense_feed_forward(h, _sub(w, prefix + "mlp."), rnd)
                else:
                    y, _ = routed_feed_forward(h, _sub(w, prefix + "mlp."), mlp, rnd)
                x = x + rnd(y)
            if stream_after is not None:
                stream_after.append(x.clone())
        z = rnd(rms_norm(x, w["final.norm"], eps)) @ w["embed"].T
        cap = cfg.get("logit_softcap")
        return cap * torch.tanh(z / cap) if cap else z

    def greedy(self, ids, count):
        ids, out = list(ids), []
        for _ in range(count):
            out.append(int(self.logits(ids)[-1].argmax()))
            ids.append(out[-1])
        return out
