"""Arrangements: how a layer wires its norms, mixer and feed-forward around the residual stream."""
from __future__ import annotations

import torch

from .. import profiler
from ..kernels import ops
from .registry import build_part, register_part

# A decode step of at most this many tokens leaves its norms to the products around them (the
# products that can do it take no more rows).
# (Links for the products of 17 to 32 rows were tried: with the sums of squares and the residual fetched at
# the end of the stream they cost what the two norm kernels cost at Qwen3-8B sizes, and 6% of the step at
# Qwen3-0.6B sizes.)
LINK_MAX_TOKENS = 16
# Up to this many rows a norm hands its rows on in the matrix cores' order when the reader asks.
TILED_MAX_ROWS = 64


class NormLink:
    """An offer to a branch's last product: add your result into ``residual`` yourself and prepare
    the rows for ``norm``, which then needs no kernel of its own."""

    def __init__(self, residual, norm, tiled: bool = False):
        self.residual, self.norm = residual, norm
        self.gain, self.eps = norm.gain, norm.eps
        self.tiled = tiled           # the reader of the prepared rows takes them in the matrix cores' order


class ResidualStream:
    """The float32 sum that runs through the layers, with at most one branch output
    waiting to be added.  The add is done by the next norm, in the same kernel, or, in
    small decode steps, by the product that made the branch output: then what waits is
    the prepared input of one norm (``later``) and the sum is already up to date."""

    def __init__(self, hidden):
        self.sum = hidden            # [T, hidden] float32
        self.pending = None
        self.later = None            # (NormedLater, the norm it was prepared for)
        self.next_entry_norm = None  # the norm that reads the stream after the current layer, if known
        self.next_entry_tiled = False  # and whether the part behind it reads tiled rows
        self.links_ok = True         # whether norms may be left to products at all (not where every step must run alike)

    @property
    def rows(self) -> int:
        return self.sum.shape[0]

    def link(self, norm, act_dtype, tiled: bool = False):
        """A ``NormLink`` for the branch that is about to run, if ``norm`` is the next reader of the
        stream and can be left to a product.  ``tiled``: the part behind that norm reads tiled rows."""
        if (not self.links_ok or norm is None or not getattr(norm, "linkable", False) or self.pending is not None or self.later is not None
                or act_dtype != torch.bfloat16 or self.sum.shape[0] > LINK_MAX_TOKENS
                or norm.dim != self.sum.shape[1]):
            return None
        return NormLink(self.sum, norm, tiled)

    def push(self, branch, gather: bool = False) -> None:
        """``gather``: a float32 branch may wait beside others (``pending`` is then a list) for a norm that adds them all."""
        if (gather and self.pending is not None and self.later is None and not isinstance(branch, tuple)
                and self._gathers(branch)):
            self.pending = (self.pending if isinstance(self.pending, list) else [self.pending]) + [branch]
            return
        if self.pending is not None or self.later is not None:
            self.flush()
        if isinstance(branch, tuple):        # (NormedLater, norm): the product took a NormLink
            self.later = branch
        else:
            self.pending = branch

    def _gathers(self, branch) -> bool:
        waiting = (self.pending if isinstance(self.pending, list) else [self.pending]) + [branch]
        return (all(y.dtype == torch.float32 for y in waiting)
                and sum(y.shape[0] if y.dim() == 3 else 1 for y in waiting) <= ops.MAX_BRANCH_PARTS)

    def normed(self, norm, out_dtype, rows=None, later_ok: bool = False, tiled: bool = False):
        """The stream through ``norm``.  With ``later_ok`` the caller takes a ``NormedLater`` too, with
        ``tiled`` (a norm that can, up to 64 rows) ``ops.TiledRows``."""
        if self.later is not None:
            later, for_norm = self.later
            self.later = None
            if later_ok and for_norm is norm and rows is None:
                return later
            # prepared for another reader: the sum is complete, norm it the plain way
        if isinstance(self.pending, list):
            if getattr(norm, "accepts_branches", False):
                with profiler.section(profiler.NORM):
                    out = norm.apply_branches(self.sum, self.pending, out_dtype, rows)
                if rows is None:
                    self.pending = None
                return out
            self.flush()
        if self.pending is not None and self.pending.dim() == 3 and not getattr(norm, "accepts_parts", False):
            self.flush()                             # a norm that does not know about parts: they go into the sum first
        with profiler.section(profiler.NORM):
            if (tiled and rows is None and getattr(norm, "can_tile", False) and out_dtype == torch.bfloat16
                    and self.sum.shape[0] <= TILED_MAX_ROWS):
                out = norm.apply(self.sum, self.pending, out_dtype, rows, tiled=True)
            else:
                out = norm.apply(self.sum, self.pending, out_dtype, rows)
        if rows is None:
            self.pending = None      # the kernel wrote sum + pending back
        return out

    def add(self, rows) -> None:
        """``x <- x + rows`` (float32) outside any sublayer: one more branch that waits.  What was prepared from the sum as it was
        is dropped."""
        self.later = self.as_act = self.prepared = None
        self.push(rows, gather=True)

    def flush(self) -> None:
        """Add the waiting branch without a norm (only arrangements that push twice need it)."""
        self.later = None            # its sum is in the stream already
        if self.pending is not None:
            for branch in (self.pending if isinstance(self.pending, list) else (self.pending,)):
                for part in (branch.unbind(0) if branch.dim() == 3 else (branch,)):
                    ops.add_rows(self.sum, part, in_place=True)   # parts in order, each sum in float32
            self.pending = None


def _takes_tiled(part, rows: int) -> bool:
    asks = getattr(part, "takes_tiled_at", None)
    return bool(asks(rows)) if asks else False


@register_part("arrangement", "prenorm")
class PreNormBlock:
    """``r = h + mixer(norm1(h))``, then ``h' = r + ff(norm2(r))``: the norm sits before
    each branch and the branch's output is added to the stream
    (the reference: src/models/qwen3.rs:121-145)."""

    def __init__(self, layer_spec):
        self.mixer_norm = build_part("norm", layer_spec.mixer_norm)
        self.mixer = build_part("mixer", layer_spec.mixer)
        # a layer without a feed-forward names neither it nor its norm: it is the first sublayer alone
        self.feed_forward_norm = self.feed_forward = None
        if "feed_forward" in layer_spec.parts:
            self.feed_forward_norm = build_part("norm", layer_spec.feed_forward_norm)
            self.feed_forward = build_part("feed_forward", layer_spec.feed_forward)

    def parts(self):
        both = (self.mixer_norm, self.mixer, self.feed_forward_norm, self.feed_forward)
        return both if self.feed_forward is not None else both[:2]

    def entry_norm(self):
        """The norm through which this layer first reads the stream."""
        return self.mixer_norm

    def entry_takes_tiled(self, rows: int) -> bool:
        """Whether the part behind that norm reads ``rows`` rows in the matrix cores' order."""
        return _takes_tiled(self.mixer, rows)

    def plain(self, h, ctx, store, page_table):
        """``h`` after this layer, float32 numpy (the plain backend)."""
        r = h + self.mixer.plain(self.mixer_norm.plain(h), ctx, store, page_table)
        if self.feed_forward is None:
            return r
        return r + self.feed_forward.plain(self.feed_forward_norm.plain(r), ctx)

    def forward(self, stream: ResidualStream, ctx, store, page_table, act_dtype) -> None:
        # a part with ``links_norms`` takes a NormedLater as input and a NormLink for its output
        rows = stream.sum.shape[0]
        after_mixer = self.feed_forward_norm if self.feed_forward is not None else stream.next_entry_norm
        if getattr(self.mixer, "links_norms", False):
            h = stream.normed(self.mixer_norm, act_dtype, later_ok=True, tiled=_takes_tiled(self.mixer, rows))
            link = stream.link(after_mixer, act_dtype, _takes_tiled(self.feed_forward, rows) if self.feed_forward is not None
                               else stream.next_entry_tiled)
            stream.push(self.mixer.forward(h, ctx, store, page_table, link=link))
        else:
            h = stream.normed(self.mixer_norm, act_dtype)
            stream.push(self.mixer.forward(h, ctx, store, page_table))
        if self.feed_forward is None:
            return
        if getattr(self.feed_forward, "links_norms", False):
            h = stream.normed(self.feed_forward_norm, act_dtype, later_ok=True,
                              tiled=_takes_tiled(self.feed_forward, rows))
            link = stream.link(stream.next_entry_norm, act_dtype, stream.next_entry_tiled)
            stream.push(self.feed_forward.forward(h, ctx, link=link))
        else:
            h = stream.normed(self.feed_forward_norm, act_dtype)
            stream.push(self.feed_forward.forward(h, ctx))


@register_part("arrangement", "parallel_prenorm")
class ParallelPreNormBlock:
    """``x <- x + (mixer(h) + ff(h))`` with ``h = norm(x)``: one norm, whose rows both sublayers read.  Parts: ``mixer_norm``,
    ``mixer`` and, for a layer that has one, ``feed_forward``.  The results wait as branches of the stream, which the next norm
    adds (``ops.add_branches_rmsnorm``); a feed-forward that sets ``separates`` hands back those of its own that are only added."""

    def __init__(self, layer_spec):
        self.mixer_norm = build_part("norm", layer_spec.mixer_norm)
        self.mixer = build_part("mixer", layer_spec.mixer)
        self.feed_forward = build_part("feed_forward", layer_spec.feed_forward) if "feed_forward" in layer_spec.parts else None

    def parts(self):
        first = (self.mixer_norm, self.mixer)
        return first if self.feed_forward is None else first + (self.feed_forward,)

    def entry_norm(self):
        """The norm through which this layer first reads the stream."""
        return self.mixer_norm

    def forward(self, stream: ResidualStream, ctx, store, page_table, act_dtype) -> None:
        h = stream.normed(self.mixer_norm, act_dtype)
        y = self.mixer.forward(h, ctx, store, page_table)
        if self.feed_forward is None:
            stream.push(y)
            return
        z = (self.feed_forward.forward(h, ctx, separate=True) if getattr(self.feed_forward, "separates", False)
             else self.feed_forward.forward(h, ctx))
        for branch in [y] + (z if isinstance(z, list) else [z]):
            stream.push(branch, gather=True)


@register_part("arrangement", "hyper_prenorm")
class HyperConnectedBlock:
    """The pre-norm layer over a residual kept in several streams (``parts.streams.HyperStream``): each
    sublayer reads the streams through its connection's ``in`` coefficients and its norm, and its output is
    written to all streams through ``mix`` and ``out``.  Parts: ``mixer_norm``, ``mixer``, ``mixer_connection``
    and, for a layer that has a feed-forward, ``feed_forward_norm``, ``feed_forward``, ``feed_forward_connection``."""

    def __init__(self, layer_spec):
        self.mixer_norm = build_part("norm", layer_spec.mixer_norm)
        self.mixer = build_part("mixer", layer_spec.mixer)
        self.mixer_connection = build_part("connection", layer_spec.mixer_connection)
        self.feed_forward_norm = self.feed_forward = self.feed_forward_connection = None
        if "feed_forward" in layer_spec.parts:
            self.feed_forward_norm = build_part("norm", layer_spec.feed_forward_norm)
            self.feed_forward = build_part("feed_forward", layer_spec.feed_forward)
            self.feed_forward_connection = build_part("connection", layer_spec.feed_forward_connection)

    def parts(self):
        first = (self.mixer_norm, self.mixer, self.mixer_connection)
        if self.feed_forward is None:
            return first
        return first + (self.feed_forward_norm, self.feed_forward, self.feed_forward_connection)

    def forward(self, stream, ctx, store, page_table, act_dtype) -> None:
        h = stream.read(self.mixer_connection, self.mixer_norm, act_dtype)
        stream.write(self.mixer.forward(h, ctx, store, page_table), self.mixer_connection)
        if self.feed_forward is not None:
            h = stream.read(self.feed_forward_connection, self.feed_forward_norm, act_dtype)
            stream.write(self.feed_forward.forward(h, ctx), self.feed_forward_connection)
