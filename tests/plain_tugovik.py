"""Tugovik, plainly: one function a mechanism over whole sequences in 64-bit,
written from the design's equations and sharing nothing with the library.

Notation.  x: the residual stream [tokens, width].  N(v, w) = v / sqrt(mean(v^2)
+ eps) * (1 + w).  A layer is x <- x + mixer(N(x, w1)), then, where it has a
feed-forward, x <- x + ff(N(x, w2)), then, where tokens have an input of their
own a layer, x <- x + side(x, token).  ``rnd`` rounds where an engine that
keeps activations in bfloat16 rounds them (the identity by default).
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


def silu(x):
    return x * sigmoid(x)


def gelu_tanh(x):
    return 0.5 * x * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


def softplus(x):
    return torch.where(x > 30.0, x, torch.log1p(torch.exp(torch.clamp(x, max=30.0))))


def over_rms(v, eps):
    return v / torch.sqrt((v * v).mean(dim=-1, keepdim=True) + eps)


def zero_centred_norm(v, w, eps):
    return over_rms(v, eps) * (1.0 + w)


def sees(i, j, chunk):
    """Whether position i sees position j: not later, and in the same chunk of ``chunk`` positions (None: all earlier)."""
    return j <= i and (not chunk or i // chunk == j // chunk)


def attention(h, w, sizes, rnd=identity):
    """h [tokens, width] from position 0 on.  w: q, k, v, their biases q.b, k.b, v.b, o.  s(i, j) = (q_i . k_j) scale
    over the keys of i's own chunk up to i; softmax; Wo on the heads' outputs one after the other."""
    n = h.shape[0]
    heads, groups, dim, vdim = sizes["heads"], sizes["kv_heads"], sizes["dim"], sizes["vdim"]
    chunk = (sizes.get("mask") or {}).get("size")
    q = rnd(rnd(h @ w["q"].T) + w["q.b"]).view(n, heads, dim)
    k = rnd(rnd(h @ w["k"].T) + w["k.b"]).view(n, groups, dim)
    v = rnd(rnd(h @ w["v"].T) + w["v.b"]).view(n, groups, vdim)
    at = torch.arange(n)
    seen = at[None, :] <= at[:, None]
    if chunk:
        seen = seen & (at[None, :] // chunk == at[:, None] // chunk)
    out = torch.zeros(n, heads, vdim, dtype=h.dtype)
    for head in range(heads):
        group = head // (heads // groups)
        s = q[:, head] @ k[:, group].T * sizes["scale"]
        p = torch.softmax(torch.where(seen, s, torch.full_like(s, -math.inf)), dim=1)
        out[:, head] = p @ v[:, group]
    return rnd(out.reshape(n, heads * vdim)) @ w["o"].T


def short_conv(x, weight, bias, before=None):
    """Per channel y_t = b + sum_j weight[:, j] x_(t - (taps - 1) + j); ``before``: the taps - 1 inputs ahead of the first
    (zeros by default).  Returns (y, the last taps - 1 inputs)."""
    taps = weight.shape[1]
    before = torch.zeros(taps - 1, x.shape[1], dtype=x.dtype) if before is None else before
    rows = torch.cat([before, x], dim=0)
    y = bias + sum(weight[:, j] * rows[j:j + x.shape[0]] for j in range(taps))
    return y, rows[rows.shape[0] - (taps - 1):]


def state_space(x, B, C, dt, a_log, D, state=None):
    """x [tokens, heads, P], B and C [tokens, groups, N], dt [tokens, heads] (behind softplus).  S [heads, N, P]:
    S <- exp(-exp(a_log) dt) S + dt B x^T,  y = S^T C + D x; head h uses group h // (heads / groups).  Returns (y, S)."""
    n, heads, P = x.shape
    groups, N = B.shape[1], B.shape[2]
    of_head = torch.arange(heads) // (heads // groups)
    S = torch.zeros(heads, N, P, dtype=x.dtype) if state is None else state
    rows = []
    for t in range(n):
        keep = torch.exp(-torch.exp(a_log) * dt[t])[:, None, None]
        S = keep * S + dt[t][:, None, None] * B[t][of_head][:, :, None] * x[t][:, None, :]
        rows.append(torch.einsum("hnp,hn->hp", S, C[t][of_head]) + D[:, None] * x[t])
    return torch.stack(rows), S


def gated_parts_norm(y, z, weight, parts, eps):
    """y silu(z), then each of ``parts`` equal parts over its own root mean square, times the weight."""
    y = y * silu(z)
    n, inner = y.shape
    return over_rms(y.view(n, parts, inner // parts), eps).reshape(n, inner) * weight


def mamba2(h, w, sizes, eps, rnd=identity):
    """w: in, conv, conv.b, dt_bias, A_log, D, norm, o.  The rows of ``in``: z, x, B, C, dt."""
    n = h.shape[0]
    heads, P, N, G = sizes["heads"], sizes["vdim"], sizes["state"], sizes["groups"]
    inner = heads * P
    rows = h @ w["in"].T
    z = rnd(rows[:, :inner])
    xbc = rnd(rows[:, inner:2 * inner + 2 * G * N])
    dt = softplus(rows[:, 2 * inner + 2 * G * N:] + w["dt_bias"])
    xbc = rnd(silu(short_conv(xbc, w["conv"], w["conv.b"])[0]))
    x, B, C = xbc[:, :inner], xbc[:, inner:inner + G * N], xbc[:, inner + G * N:]
    y, _ = state_space(x.view(n, heads, P), B.view(n, G, N), C.view(n, G, N), dt, w["A_log"], w["D"])
    y = gated_parts_norm(y.reshape(n, inner), z, w["norm"], sizes["norm_groups"], eps)
    return rnd(y) @ w["o"].T


def rglru_gates(u, w, blocks):
    """(log a, i) of the real-gated linear recurrent unit for u [tokens, width]."""
    n, width = u.shape
    parts = u.view(n, blocks, width // blocks)
    r = sigmoid(torch.einsum("nbi,boi->nbo", parts, w["ra"]) + w["ra.b"]).reshape(n, width)
    i = sigmoid(torch.einsum("nbi,boi->nbo", parts, w["ri"]) + w["ri.b"]).reshape(n, width)
    return -8.0 * r * softplus(w["lam"]), i


def rglru_scan(u, log_a, i, state=None):
    """S <- a S + sqrt(1 - a^2) i u element by element.  Returns (S at every token, the last S)."""
    S = torch.zeros(u.shape[1], dtype=u.dtype) if state is None else state
    rows = []
    for t in range(u.shape[0]):
        S = torch.exp(log_a[t]) * S + torch.sqrt(-torch.expm1(2.0 * log_a[t])) * i[t] * u[t]
        rows.append(S)
    return torch.stack(rows), S


def rglru(h, w, sizes, rnd=identity):
    """w: y, y.b, x, x.b, conv, conv.b, ra, ra.b, ri, ri.b, lam, o."""
    y = gelu_tanh(rnd(h @ w["y"].T) + w["y.b"])
    u = rnd(short_conv(rnd(h @ w["x"].T) + w["x.b"], w["conv"], w["conv.b"])[0])
    log_a, i = rglru_gates(u, w, sizes["blocks"])
    S, _ = rglru_scan(u, log_a, i)
    return rnd(S * y) @ w["o"].T


def expert(h, w, rnd=identity):
    """Wdown (silu(Wgate h) * (Wup h))."""
    return rnd(silu(rnd(h @ w["gate"].T)) * rnd(h @ w["up"].T)) @ w["down"].T


def choose(h, w, router):
    """s = sigmoid(Wrouter h).  The ``top`` largest are chosen, among the experts of the ``keep`` of ``count`` groups with
    the largest sums of their two largest scores where there are groups; the weights are the chosen scores over their
    sum, times scale.  Returns (chosen, weights) [tokens, top]."""
    s = sigmoid(h @ w["router"].T)
    pick = s
    groups = router.get("groups")
    if groups:
        n, experts = s.shape
        size = experts // groups["count"]
        parts = s.view(n, groups["count"], size)
        marks = torch.topk(parts, min(2, size), dim=-1).values.sum(-1)
        best = torch.topk(marks, groups["keep"], dim=-1).indices
        open_ = torch.zeros(n, groups["count"], dtype=torch.bool).scatter(1, best, True)
        pick = torch.where(open_.repeat_interleave(size, dim=1), s, torch.full_like(s, -1.0))
    chosen = torch.topk(pick, router["top"], dim=-1).indices
    weights = torch.gather(s, 1, chosen)
    return chosen, weights / (weights.sum(-1, keepdim=True) + 1e-20) * router.get("scale", 1.0)


def routed_feed_forward(h, w, mlp, rnd=identity):
    """The chosen experts' outputs, weighted and added; the shared expert's times sigmoid(Wsg h).  Returns (out, chosen)."""
    chosen, weights = choose(h, w, mlp["router"])
    out = torch.zeros(h.shape[0], h.shape[1], dtype=h.dtype)
    for e in range(mlp["router"]["experts"]):
        rows, place = torch.nonzero(chosen == e, as_tuple=True)
        if rows.numel():
            out[rows] += weights[rows, place, None] * expert(h[rows], _sub(w, f"e{e}."), rnd)
    if mlp.get("shared"):
        out = out + sigmoid(h @ w["shared.sg"].T) * expert(h, _sub(w, "shared."), rnd)
    return out, chosen


def token_side(x, part, w, eps, rnd=identity):
    """x: the stream; part [tokens, dim]: the tokens' own input for this layer.  w: side.gate, side.proj, side.norm.
    What is added to the stream."""
    g = rnd(gelu_tanh(rnd(x) @ w["side.gate"].T) * part)
    return over_rms(rnd(g @ w["side.proj"].T), eps) * w["side.norm"]


def _sub(weights, prefix):
    return {name[len(prefix):]: value for name, value in weights.items() if name.startswith(prefix)}


def order_of_layers(config):
    """The layers as they run: start .. stop - 1 of ``loop`` ``times`` times in a row."""
    order = list(range(len(config["layers"])))
    loop = config.get("loop")
    if loop:
        order = order[:loop["start"]] + order[loop["start"]:loop["stop"]] * loop["times"] + order[loop["stop"]:]
    return order


MIXERS = {"attention": lambda h, w, sizes, eps, rnd: attention(h, w, sizes, rnd), "mamba2": mamba2,
          "rglru": lambda h, w, sizes, eps, rnd: rglru(h, w, sizes, rnd)}


class PlainTugovik:
    """The whole model over one sequence from its first token, from a folder with config.json and model.safetensors."""

    def __init__(self, folder):
        with open(os.path.join(folder, "config.json")) as handle:
            self.config = json.load(handle)
        self.w = {name: value.double() for name, value in load_file(os.path.join(folder, "model.safetensors")).items()}

    def logits(self, ids, rnd=identity, stream_after=None):
        """Logits [tokens, vocab]; ``stream_after`` (a list) gets the stream after every layer run."""
        cfg, w = self.config, self.w
        eps = cfg["norm"]["eps"]
        ids = torch.as_tensor(list(ids), dtype=torch.long)
        x = w["embed"][ids]
        for index in order_of_layers(cfg):
            layer, own = cfg["layers"][index], _sub(w, f"l{index}.")
            h = rnd(zero_centred_norm(x, own["norm1"], eps))
            x = x + rnd(MIXERS[layer["type"]](h, _sub(own, "mix."), layer["mixer"], eps, rnd))
            if layer.get("mlp") is not None:
                h = rnd(zero_centred_norm(x, own["norm2"], eps))
                x = x + rnd(routed_feed_forward(h, _sub(own, "mlp."), layer["mlp"], rnd)[0])
            if cfg.get("token_side"):
                dim = cfg["token_side"]["dim"]
                x = x + token_side(x, w["side.embed"][ids][:, index * dim:(index + 1) * dim], own, eps, rnd)
            if stream_after is not None:
                stream_after.append(x.clone())
        return rnd(zero_centred_norm(x, w["final.norm"], eps)) @ w["head"].T

    def greedy(self, ids, count):
        ids, out = list(ids), []
        for _ in range(count):
            out.append(int(self.logits(ids)[-1].argmax()))
            ids.append(out[-1])
        return out
