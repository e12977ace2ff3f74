"""A norm that has not run yet, or has run half.

A block hands its mixer or feed-forward a ``PendingNorm`` instead of the
normalised rows.  A consumer whose first step is a projection can fold the
norm into that projection's kernel (``fused``); any other consumer calls
``materialize`` and gets the rows from the norm's own kernel.  Either way
``residual`` afterwards holds the stream the block goes on with.

It comes in three states.  *Lazy*: ``x`` and a part's output ``delta`` that is
not added yet; the consumer's kernel takes the sum, the statistics and the
gain itself (up to ``FUSED_MAX_TOKENS`` rows).  *Prepared*: the projection
that produced the part's output has already added it to the stream and left
``scaled`` = bfloat16(stream * gain) and parts of each row's sum of squares
(``ResidualInto.take``); the consumer's kernel multiplies ``scaled`` and
applies 1 / sqrt(mean + eps) to the product, for any number of rows.
*Ready*: the kernel that wrote the stream last ran the norm too; its rows are
there.
"""

from __future__ import annotations

from typing import Optional

import torch


class PendingNorm:
    def __init__(self, norm, x: torch.Tensor, delta: Optional[torch.Tensor], rt):
        self.norm = norm
        self.x = x
        self.delta = delta
        self.rt = rt
        self.residual: Optional[torch.Tensor] = None
        self.rows = x.shape[0]
        self.scaled: Optional[torch.Tensor] = None  # prepared state
        self.ss: Optional[torch.Tensor] = None
        self.parts = 0
        self.ready: Optional[torch.Tensor] = None  # the norm's rows, where whoever wrote the stream last made them

    @classmethod
    def from_rows(cls, norm, residual: torch.Tensor, rows: torch.Tensor, rt) -> "PendingNorm":
        pending = cls(norm, residual, None, rt)
        pending.residual, pending.ready = residual, rows
        return pending

    @classmethod
    def prepared(cls, norm, residual: torch.Tensor, scaled: torch.Tensor, ss: torch.Tensor, parts: int, rt) -> "PendingNorm":
        pending = cls(norm, residual, None, rt)
        pending.residual = residual
        pending.scaled, pending.ss, pending.parts = scaled, ss, parts
        return pending

    def materialize(self) -> torch.Tensor:
        if self.ready is not None:
            return self.ready
        if self.delta is None:
            out = self.norm.forward(self.x, self.rt)
        else:
            out = self.norm.add_forward(self.x, self.delta, self.rt)  # sums into x in place
        self.residual = self.x
        return out

    def can_fuse(self, weight) -> bool:
        """True when ``fused`` may be called with this projection weight."""
        ops = self.rt.ops
        if self.ready is not None:
            return False
        fits = (
            getattr(self.norm, "fusable_rms", False)
            and self.x.dtype == torch.float32
            and isinstance(weight, ops.PackedWeight)
            and self.rt.dtype == torch.bfloat16
        )
        if self.scaled is not None:
            return fits
        return fits and self.rows <= ops.FUSED_MAX_TOKENS and (self.delta is None or self.delta.dtype == torch.bfloat16)

    def fused(self, weight, y: torch.Tensor, epilogue: int, rope=None) -> torch.Tensor:
        """y = epilogue(weight . norm(x + delta)) in one kernel."""
        if self.scaled is not None:
            return self.rt.ops.gemm_scaled(self.scaled, self.ss, self.parts, self.norm.eps, weight, y, epilogue, rope)
        x_out = None
        if self.delta is not None:
            x_out = torch.empty_like(self.x)
        self.rt.ops.gemm_fused(self.x, self.delta, x_out, self.norm.weight, self.norm.eps, weight, y, epilogue, rope)
        self.residual = self.x if x_out is None else x_out
        return y


class ResidualInto:
    """Where the projection that ends a mixer or feed-forward may put its
    result instead of returning it: into the residual stream that ``source``
    (the part's own input) leaves behind, with ``norm``, the norm that comes
    next, prepared in the same kernel."""

    def __init__(self, source: PendingNorm, norm, rt):
        self.source = source
        self.norm = norm
        self.rt = rt

    def can_take(self, x: torch.Tensor, weight) -> bool:
        return getattr(self.norm, "fusable_rms", False) and self._fits(x, weight)

    def _fits(self, x: torch.Tensor, weight) -> bool:
        residual = self.source.residual
        return (
            residual is not None
            and residual.dtype == torch.float32
            and residual.is_contiguous()
            and self.rt.dtype == torch.bfloat16
            and x.dtype == torch.bfloat16
            and isinstance(weight, self.rt.ops.PackedWeight)
            and weight.shape[0] == residual.shape[1]
        )

    def take(self, x: torch.Tensor, weight) -> PendingNorm:
        """residual += x @ weight^T; returns the next norm, prepared."""
        return self.take_by(lambda residual, gain, scaled, ss: self.rt.ops.gemm_residual(x, weight, residual, gain, scaled, ss))

    def take_by(self, write) -> PendingNorm:
        """The same by a kernel of the part's own: ``write(residual, gain,
        scaled, ss)`` adds to the stream and returns how many parts of the
        rows' sums of squares it left in ``ss``."""
        rt, residual = self.rt, self.source.residual
        rows, width = residual.shape
        scaled = rt.empty(rows, width)
        ss = rt.empty(rt.ops.gemm_residual_parts(rows, width), rows, dtype=torch.float32)
        parts = write(residual, self.norm.weight, scaled, ss)
        return PendingNorm.prepared(self.norm, residual, scaled, ss, parts, rt)


class StreamInto(ResidualInto):
    """``ResidualInto`` where what comes next reads the stream as it is (a
    norm of kind ``none``): ``take`` returns the stream with its rows in the
    activation type (``PreparedRows``), which the projection's kernel wrote
    beside its sum."""

    def can_take(self, x: torch.Tensor, weight) -> bool:
        return getattr(self.norm, "ones", None) is not None and self._fits(x, weight)

    def take_by(self, write):
        rt, residual = self.rt, self.source.residual
        rows, width = residual.shape
        plain = rt.empty(rows, width)
        ss = rt.empty(rt.ops.gemm_residual_parts(rows, width), rows, dtype=torch.float32)  # (nobody reads it)
        write(residual, self.norm.ones, plain, ss)
        return PreparedRows(self.norm, residual, plain)

    def take(self, x: torch.Tensor, weight):
        return self.take_by(lambda residual, gain, scaled, ss: self.rt.ops.gemm_residual(x, weight, residual, gain, scaled, ss))


class PreparedStreams:
    """What a block over several residual streams hands the block that comes
    next when it has run that block's first norm already (in the kernel that
    brought its own last output into the streams): the streams ``x``
    [streams, tokens, width] and ``h``, the rows that ``norm`` makes of them."""

    def __init__(self, norm, x: torch.Tensor, h: torch.Tensor):
        self.norm, self.x, self.h = norm, x, h


class PostNormed:
    """A part's output ``y`` whose norm has not run: what is to be added to
    the residual stream is ``norm(y)``.  A layer that norms its sublayers on
    the way out too hands this on as the stream's pending part, so that
    whoever takes the stream next (a block, a pass's entry, the final norm)
    does norm, sum and its own first step in one kernel; anybody else calls
    ``materialize``."""

    def __init__(self, y: torch.Tensor, norm):
        self.y, self.norm = y, norm

    def materialize(self, rt) -> torch.Tensor:
        return self.norm.forward(self.y, rt)


class PreparedRows:
    """A stream ``x`` [tokens, width] with nothing left to add, and ``h``,
    the rows that ``norm`` -- the first norm of the block that takes this --
    makes of it: run already by whoever wrote the stream last."""

    def __init__(self, norm, x: torch.Tensor, h: torch.Tensor):
        self.norm, self.x, self.h = norm, x, h


class TanhInto:
    """``ResidualInto`` for a block whose norms keep no statistics: where the
    projection that ends a mixer or feed-forward may put its result.  The
    stream ``residual`` takes ``post``(product) in, and ``following``, the norm
    on the next sublayer's way in, is run on the sum, all in the projection's
    own kernel.  ``take`` returns the ``PreparedRows`` of ``following``."""

    def __init__(self, residual: torch.Tensor, post, following, rt):
        self.residual, self.post, self.following, self.rt = residual, post, following, rt

    def can_take(self, x, weight) -> bool:
        residual, rt = self.residual, self.rt
        return (
            isinstance(x, torch.Tensor)  # (runs of keys that a decode attention left are added up first)
            and hasattr(self.post, "triple") and hasattr(self.following, "triple")
            and rt.dtype == torch.bfloat16 and x.dtype == torch.bfloat16
            and residual.dtype == torch.float32 and residual.is_contiguous()
            and isinstance(weight, rt.ops.PackedWeight)
            and weight.shape[0] == residual.shape[1] and weight.shape[1] % 8 == 0
            and x.data_ptr() % 16 == 0 and residual.data_ptr() % 16 == 0
            and all(v.data_ptr() % 16 == 0 for v in self.post.triple()[1:] + self.following.triple()[1:])
        )

    def take(self, x: torch.Tensor, weight) -> PreparedRows:
        rt, residual = self.rt, self.residual
        rows, width = residual.shape
        normed = rt.empty(rows, width)
        ss = rt.empty(rt.ops.gemm_residual_parts(rows, width), rows, dtype=torch.float32)
        rt.ops.gemm_residual_tanh(x, weight, residual, self.post.triple(), self.following.triple(), normed, ss)
        return PreparedRows(self.following, residual, normed)
