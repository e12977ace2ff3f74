"""Gated feed-forward: down( act(gate x) * up x ), act = SiLU
(/root/reference/crates/nnis-model/src/runtime.rs:1054-1087;
/root/reference/crates/nnis-model/src/fused_swiglu.rs:14-28), the tanh form
of GELU, or ReLU.  Gate and up are one fused projection whose first ``inner`` output
columns are the gate."""

from __future__ import annotations

import torch

from ..errors import InvalidInput, Unsupported
from ..weights.random_init import register_init_rule
from .base import FeedForward, TensorSpec, register_part
from .linear import Projection


class GatedFeedForward(FeedForward):
    graph_safe = True

    def __init__(self, width, inner, gate, up, down, activation="silu"):
        if activation not in ("silu", "gelu_tanh", "relu"):
            raise Unsupported(f"gated feed-forward activation {activation!r}; silu, gelu_tanh and relu are built")
        self.activation = activation
        self.width, self.inner = int(width), int(inner)
        self.names = {"gate": gate, "up": up, "down": down}
        self.gate_up = None
        self.down = None

    def tensors(self):
        return [
            TensorSpec(self.names["gate"], (self.inner, self.width)),
            TensorSpec(self.names["up"], (self.inner, self.width)),
            TensorSpec(self.names["down"], (self.width, self.inner)),
        ]

    def bind(self, weights, rt):
        if rt.dtype == torch.bfloat16:
            rt.ops.unit_rows(rt.device)  # (made here, outside any captured step)
        self.gate_up = Projection(torch.cat([weights[self.names["gate"]], weights[self.names["up"]]], dim=0), rt)
        self.down = Projection(weights[self.names["down"]], rt)

    def weight_bytes(self):
        return self.gate_up.weight_bytes() + self.down.weight_bytes()

    takes_pending_norm = True
    adds_to_residual = True

    def forward(self, x, ctx, rt, into=None):
        from .lazy import PendingNorm

        if isinstance(x, PendingNorm) and self.activation == "silu" and x.can_fuse(self.gate_up.weight):
            # (residual sum,) norm, both projections and the gating in one kernel
            hidden = x.fused(self.gate_up.weight, rt.empty(x.rows, self.inner), rt.ops.EPILOGUE_SILU)
        else:
            if isinstance(x, PendingNorm):
                x = x.materialize()
            ops = rt.ops
            if (rt.dtype == torch.bfloat16 and x.dtype == torch.bfloat16 and isinstance(self.gate_up.weight, ops.PackedWeight)
                    and 0 < x.shape[0] <= ops.UNIT_ROWS_MOST and x.is_contiguous() and x.data_ptr() % 16 == 0):
                # both projections with the gating in their epilogue, on rows that are normed already
                hidden = ops.gated_linear(x, self.gate_up.weight, rt.empty(x.shape[0], self.inner), self.activation)
            else:
                gate_up = self.gate_up(x, rt)
                hidden = ops.gated_act(gate_up, rt.empty(x.shape[0], self.inner), self.activation)
        if into is not None and into.can_take(hidden, self.down.weight):
            return into.take(hidden, self.down.weight)  # the down projection adds to the stream itself
        return self.down(hidden, rt)


register_part("feed_forward", "gated", GatedFeedForward)


class PolyNormFeedForward(FeedForward):
    """down(act(up x)) with act(z) = a N(z) + b N(z^2) + c N(z^3) + e: powers element by element, N a division of a
    token's inner row by its root mean square (eps inside the root); (a, b, c, e) are the four numbers of ``act``.
    The statistics and the polynomial are 32-bit."""

    graph_safe = True

    def __init__(self, width, inner, eps, up, down, act):
        self.width, self.inner, self.eps = int(width), int(inner), float(eps)
        self.names = {"up": up, "down": down, "act": act}
        self.up = self.down = self.coefficients = None

    def tensors(self):
        return [TensorSpec(self.names["up"], (self.inner, self.width)), TensorSpec(self.names["down"], (self.width, self.inner)),
                TensorSpec(self.names["act"], (4,), init="poly_coefficients")]

    def bind(self, weights, rt):
        self.up = Projection(weights[self.names["up"]], rt)
        self.down = Projection(weights[self.names["down"]], rt)
        self.coefficients = weights[self.names["act"]].float().contiguous()

    def weight_bytes(self):
        return self.up.weight_bytes() + self.down.weight_bytes() + 16

    def forward(self, x, ctx, rt):
        z = self.up(x, rt)
        return self.down(rt.ops.poly_norm(z, self.coefficients, self.eps, rt.empty(x.shape[0], self.inner)), rt)


class RoutedFeedForward(FeedForward):
    """A mixture of ``experts`` small feed-forwards, down_e(relu(up_e x)^2) or (``activation="silu_gated"``)
    down_e(silu(gate_e x) * up_e x), of which a token uses ``top``:

        s = softmax(W_r x) over experts + identity outputs       32-bit
        chosen = the ``top`` largest of s + correction           (the lower index on a tie)
        out = sum over chosen e of s_e * expert_e(x),            expert_e(x) = x for the last ``identity`` outputs

    The weights are the scores themselves, not renormalised; ``correction`` (a tensor's name or None) enters the
    choice only.  ``scoring="chosen_softmax"``: chosen are the ``top`` largest logits instead, and the weights are the
    softmax over the chosen logits alone; ``router_bias`` (a name): joins the logits.  ``activation="clamped_swiglu"``:
    down_e(a sigmoid(1.702 a) (u + 1)), a = min(gate_e x, limit), u = up_e x held within plus or minus ``limit`` (None:
    not held).  ``shared`` (``inner``, ``limit``, ``gate``, ``up``, ``down``): one more expert of the same form, with an
    inner size and a limit of its own, that every token uses with weight one, or with ``weight`` (a name) times
    sigmoid(w . x), w the row of that tensor.  ``scoring="sigmoid"``: scores are sigmoid(W_r x), and the weights are the
    chosen scores over their sum (+ 1e-20), times ``weight_scale``.

    ``groups`` (count, keep): the outputs, identity outputs included, form ``count`` equal groups of
    neighbours; a group's mark is its largest corrected score (with ``group_marks=2`` the sum of its two largest), and only outputs of the ``keep`` groups with the largest
    marks can be chosen.  The experts' up projections are one product over all experts, gated row by row with the
    scores (zero for the experts not chosen) before one down projection over all of them."""

    graph_safe = True

    def __init__(self, width, inner, experts, top, router, up, down, identity=0, correction=None, activation="relu_squared", gate=None,
                 groups=None, scoring="softmax", router_bias=None, limit=None, shared=None, weight_scale=1.0, group_marks=1):
        """``up``, ``down`` and ``gate``: names with ``{}`` in the expert's place."""
        self.width, self.inner, self.experts, self.top, self.identity = int(width), int(inner), int(experts), int(top), int(identity or 0)
        if min(self.width, self.inner, self.experts, self.top) <= 0 or self.identity < 0 or self.top > self.experts + self.identity:
            raise InvalidInput(f"a router of {experts} experts and {identity} identity outputs cannot choose {top}")
        if activation not in ("relu_squared", "silu_gated", "clamped_swiglu") or (activation != "relu_squared") != (gate is not None):
            raise InvalidInput(f"experts are relu_squared, or silu_gated or clamped_swiglu with gate projections; got {activation!r}")
        self.activation, self.limit = activation, 0.0 if limit is None else float(limit)
        if scoring not in ("softmax", "chosen_softmax", "sigmoid"):
            raise InvalidInput(f"a router weighs by softmax, chosen_softmax or sigmoid; got {scoring!r}")
        self.weight_scale, self.group_marks = float(weight_scale), int(group_marks)
        if (self.weight_scale != 1.0 and scoring != "sigmoid") or self.group_marks not in (1, 2):
            raise InvalidInput(f"weights are scaled under sigmoid scores and a group's mark adds up one or two; got {weight_scale} and {group_marks}")
        if self.limit < 0.0 or (limit is not None and (activation != "clamped_swiglu" or self.limit == 0.0)):
            raise InvalidInput(f"a positive limit belongs to clamped_swiglu experts; got {limit!r} with {activation!r}")
        self.scoring = scoring
        self.shared = None if shared is None else dict(shared, inner=int(shared["inner"]), limit=float(shared.get("limit") or 0.0))
        if self.shared is not None and (activation == "relu_squared" or self.shared["inner"] <= 0):
            raise InvalidInput("a shared expert has the form of gated experts and a size of its own")
        self.shared_weight = None if self.shared is None else self.shared.get("weight")
        if self.shared_weight and self.identity:
            raise InvalidInput("a router weighs identity outputs or a shared expert for each token, not both")
        self.groups = None
        if groups is not None and int(groups[0]) > 1:
            count, keep = int(groups[0]), int(groups[1])
            outputs = self.experts + self.identity
            if outputs % count or not 1 <= keep <= count or self.top > keep * (outputs // count):
                raise InvalidInput(f"{outputs} router outputs in {count} equal groups of which {keep} are kept cannot choose {top}")
            self.groups = (count, keep)
        self.names = {"router": router, "up": up, "down": down, "correction": correction, "gate": gate, "router_bias": router_bias}

    def tensors(self):
        n, outputs = self.names, self.experts + self.identity
        out = [TensorSpec(n["router"], (outputs, self.width), init="router")]
        if n["correction"]:
            out.append(TensorSpec(n["correction"], (outputs,), init="small"))
        if n["router_bias"]:
            out.append(TensorSpec(n["router_bias"], (outputs,), init="small"))
        if self.shared is not None:
            inner = self.shared["inner"]
            out += [TensorSpec(self.shared["gate"], (inner, self.width)), TensorSpec(self.shared["up"], (inner, self.width)),
                    TensorSpec(self.shared["down"], (self.width, inner))]
            if self.shared_weight:
                out.append(TensorSpec(self.shared_weight, (1, self.width), init="router"))
        for e in range(self.experts):
            if n["gate"]:
                out.append(TensorSpec(n["gate"].format(e), (self.inner, self.width)))
            out += [TensorSpec(n["up"].format(e), (self.inner, self.width)), TensorSpec(n["down"].format(e), (self.width, self.inner))]
        return out

    def check(self, rt):
        if self.experts + self.identity + bool(self.shared_weight) > rt.ops.ROUTE_MOST_OUTPUTS or self.width > rt.ops.ROUTE_MOST_CHANNELS:
            raise Unsupported(f"the router kernels take up to {rt.ops.ROUTE_MOST_OUTPUTS} outputs of rows of up to "
                              f"{rt.ops.ROUTE_MOST_CHANNELS} channels, got {self.experts + self.identity} and {self.width}")

    def bind(self, weights, rt):
        n, ops = self.names, rt.ops
        stored = weights[n["router"]]
        if self.shared_weight:  # (the shared expert's logit is one more output of the router's product)
            stored = torch.cat([stored, weights[self.shared_weight]], dim=0)
        self.router = stored.float().contiguous()  # its logits are a 32-bit product under either runtime
        self.router_stored = stored.contiguous() if stored.dtype == torch.bfloat16 else None
        self.correction = weights[n["correction"]].float().contiguous() if n["correction"] else None
        self.router_bias = weights[n["router_bias"]].float().contiguous() if n["router_bias"] else None
        # one product over all experts: expert by expert its up rows (behind its gate rows, where it has them), the shared
        # expert's behind them.  Where the experts' own kernels are to run, an inner size is filled up with zeros.
        extra = 0 if self.shared is None else self.shared["inner"]
        grouped = (rt.dtype == torch.bfloat16 and n["gate"] is not None and not self.identity and self.experts <= ops.EXPERTS_MOST
                   and self.top <= ops.ROUTE_MOST_LISTED and self.width <= ops.ROUTE_FUSED_MOST_CHANNELS
                   and ops.packs(weights[n["up"].format(0)]))
        step = ops.ExpertRegions.STEP if grouped else 1
        self.padded, extra = -(-self.inner // step) * step, -(-extra // step) * step

        def filled(name, size, dim):
            w = weights[name]
            if w.shape[dim] == size:
                return w
            shape = list(w.shape)
            shape[dim] = size - w.shape[dim]
            return torch.cat([w, w.new_zeros(shape)], dim=dim)

        names = (n["gate"], n["up"]) if n["gate"] else (n["up"],)
        rows = [filled(name.format(e), self.padded, 0) for e in range(self.experts) for name in names]
        columns = [filled(n["down"].format(e), self.padded, 1) for e in range(self.experts)]
        if self.shared is not None:
            rows += [filled(self.shared["gate"], extra, 0), filled(self.shared["up"], extra, 0)]
            columns.append(filled(self.shared["down"], extra, 1))
        self.up = Projection(torch.cat(rows, dim=0), rt)
        self.down = Projection(torch.cat(columns, dim=1), rt)
        self.extra = extra
        self.regions = None
        if grouped:
            self.regions = ops.ExpertRegions(self.experts, self.padded, extra, self.activation, self.limit,
                                             0.0 if self.shared is None else self.shared["limit"])

    def weight_bytes(self):
        return self.up.weight_bytes() + self.down.weight_bytes() + self.router.numel() * 4

    def weight_bytes_for(self, rows):
        """What a step of ``rows`` tokens reads: where experts that nobody chose are left out, the expected share of them
        under a router that chooses evenly."""
        if self.regions is None or rows > self.few_rows:
            return self.weight_bytes()
        unread = self.experts * (1.0 - self.top / self.experts) ** rows * self.padded
        return self.weight_bytes() - int((self.up.weight_bytes() + self.down.weight_bytes()) * unread / self.regions.hidden)

    few_rows = 16  # up to this many rows the experts that nobody chose are left out
    many_rows = 96  # from this many on an expert's products run over the rows that chose it; in between all experts are multiplied
    takes_pending_norm = True
    adds_to_residual = True
    can_leave_share = True  # ``forward(..., share_later=True)`` leaves the identity outputs' share to a consumer that adds it in a kernel of its own

    def _route(self, x, rt, listed):
        """(normed rows, gates, keep, choices as lists or None): the router's own kernel, with the norm before it where
        that is still to run.  ``keep``: the identity outputs' share of each row, or the shared expert's weight."""
        from .lazy import PendingNorm

        ops = rt.ops
        pending = isinstance(x, PendingNorm)
        tokens = x.rows if pending else x.shape[0]
        gates, keep = rt.empty(tokens, self.experts, dtype=torch.float32), rt.empty(tokens, dtype=torch.float32)
        chosen = (rt.empty(tokens, self.top, dtype=torch.int32), rt.empty(tokens, self.top, dtype=torch.float32)) if listed else None
        rule = dict(groups=self.groups, bias=self.router_bias, scoring=self.scoring, weight_scale=self.weight_scale,
                    group_marks=self.group_marks, shared_gate=bool(self.shared_weight))
        if (pending and getattr(x.norm, "fusable_rms", False) and x.x.dtype == torch.float32 and x.x.is_contiguous()
                and x.ready is None and self.width <= ops.ROUTE_FUSED_MOST_CHANNELS):
            h = ops.route_norm(x.x, x.delta, x.norm.weight, x.norm.eps, rt.empty(tokens, self.width), self.router, self.correction,
                               self.experts, self.top, gates, keep, chosen=chosen, weight_bf16=self.router_stored, **rule)
            x.residual = x.x
            return h, gates, keep, chosen
        if pending:
            x = x.materialize()
        if self.width <= ops.ROUTE_FUSED_MOST_CHANNELS:
            ops.route(x, self.router, self.correction, self.experts, self.top, gates, keep, chosen=chosen, **rule)
        else:
            logits = ops.router_logits(x, self.router, rt.empty(tokens, self.router.shape[0], dtype=torch.float32))
            ops.route_top(logits, self.correction, self.experts, self.top, gates, keep, **rule)
        return x, gates, keep, chosen

    def forward(self, x, ctx, rt, share_later=False, into=None):
        """With ``share_later`` and identity outputs: returns (y, (keep, x)), where the output is y + keep[row] * x[row]."""
        ops = rt.ops
        tokens = x.rows if hasattr(x, "rows") else x.shape[0]
        many = self.regions is not None and tokens >= self.many_rows
        x, gates, keep, chosen = self._route(x, rt, many)
        shared_weights = keep if self.shared_weight else None
        if self.regions is not None and (many or tokens <= self.few_rows):
            def run(out, stream=None):
                if many:
                    return ops.experts_many(x, self.up.weight, self.down.weight, self.regions, chosen[0], chosen[1], out, stream, shared_weights)
                return ops.experts_few(x, self.up.weight, self.down.weight, self.regions, gates, out, stream, shared_weights)

            if into is not None and hasattr(into, "take_by") and into.can_take(x, self.down.weight):
                return into.take_by(lambda *stream: run(None, stream))  # (the last kernel adds to the stream itself)
            y = rt.empty(tokens, self.width)
            run(y)
            return y
        z = self.up(x, rt)
        inner, extra = self.experts * self.padded, self.extra
        hidden = rt.empty(tokens, inner + extra)
        if not extra:
            ops.routed_act(z, gates, hidden, self.activation, self.limit)
        else:
            ops.routed_act(z[:, :2 * inner], gates, hidden[:, :inner], self.activation, self.limit, inner=self.padded)
            ops.routed_act(z[:, 2 * inner:], None if shared_weights is None else shared_weights.view(tokens, 1), hidden[:, inner:], self.activation, self.shared["limit"], inner=extra)
        if into is not None and not self.identity and into.can_take(hidden, self.down.weight):
            return into.take(hidden, self.down.weight)
        y = self.down(hidden, rt)
        if self.identity and share_later:
            return y, (keep, x)
        if self.identity:
            rt.ops.rows_axpy(y, x, keep)
        return y


class TokenInput(FeedForward):
    """An input of a token's own, gated by the stream: W_p (gelu_tanh(W_g x) * e), e the columns first .. first + inner - 1
    of the token's row of a table that the layers share."""

    graph_safe = True

    def __init__(self, width, inner, vocab_size, table, columns, first, gate, proj):
        self.width, self.inner, self.vocab_size = int(width), int(inner), int(vocab_size)
        self.columns, self.first = int(columns), int(first)
        if min(self.width, self.inner) <= 0 or not 0 <= self.first <= self.columns - self.inner:
            raise InvalidInput(f"a token's input of {inner} columns from {first} on does not fit a table of {columns}")
        self.names = {"table": table, "gate": gate, "proj": proj}
        self.table = self.gate = self.proj = None

    def tensors(self):
        n = self.names
        return [TensorSpec(n["table"], (self.vocab_size, self.columns), init="token_input"), TensorSpec(n["gate"], (self.inner, self.width)),
                TensorSpec(n["proj"], (self.width, self.inner))]

    def bind(self, weights, rt):
        self.table = weights[self.names["table"]].contiguous()
        self.gate = Projection(weights[self.names["gate"]], rt)
        self.proj = Projection(weights[self.names["proj"]], rt)

    def weight_bytes(self):
        return self.gate.weight_bytes() + self.proj.weight_bytes()

    def forward(self, x, ctx, rt):
        if isinstance(self.gate.weight, rt.ops.PackedWeight) and x.dtype == self.table.dtype == torch.bfloat16:
            return self.proj(rt.ops.token_gate_rows(x, self.gate.weight, ctx.ids, self.table, self.first, rt.empty(x.shape[0], self.inner)), rt)
        z = self.gate(x, rt, out_dtype=torch.float32)
        return self.proj(rt.ops.token_gate(z, ctx.ids, self.table, self.first, rt.empty(x.shape[0], self.inner)), rt)


# what a random model draws: a token's own input of the size of one
register_init_rule("token_input", lambda spec, generator, dtype: torch.randn(tuple(spec.shape), generator=generator).to(dtype), replace=True)
register_part("feed_forward", "token_input", TokenInput)

# what a random model draws: coefficients of a size that matters, router rows that spread the scores
register_init_rule("poly_coefficients", lambda spec, generator, dtype: (0.5 + 0.25 * torch.randn(tuple(spec.shape), generator=generator)).to(dtype),
                   replace=True)
register_init_rule("router", lambda spec, generator, dtype: (0.3 * torch.randn(tuple(spec.shape), generator=generator)).to(dtype), replace=True)
register_part("feed_forward", "poly_norm", PolyNormFeedForward)
register_part("feed_forward", "routed", RoutedFeedForward)
