"""The arrangement with norms on both sides of every sublayer."""
from __future__ import annotations

import torch

from .. import profiler
from ..errors import ConfigError
from ..kernels import ops
from .block import TILED_MAX_ROWS, ResidualStream, _takes_tiled
from .norm import RMSNorm
from .registry import build_part, register_part


@register_part("arrangement", "sandwich")
class SandwichBlock:
    """``x <- x + after1(mixer(before1(x)))``, then ``x <- x + after2(ff(before2(x)))``.  Parts: ``mixer_norm``, ``mixer``,
    ``after_mixer_norm`` and, for a layer with a feed-forward, ``feed_forward_norm``, ``feed_forward`` and
    ``after_feed_forward_norm``; the norms behind a sublayer are of a kind with a gain and optionally a bias.

    One kernel closes a sublayer (``ops.branch_norm_add_norm``): it adds the parts of the sublayer's last product, norms
    them, adds them to the float32 residual and, where the norm that reads the residual next is known and an RMS norm
    (this layer's second one, or the next layer's first), takes that norm of the new residual as well.  Its rows wait on
    the stream (``stream.prepared``) for the reader they were made for."""

    def __init__(self, layer_spec):
        self.mixer_norm = build_part("norm", layer_spec.mixer_norm)
        self.mixer = build_part("mixer", layer_spec.mixer)
        self.after_mixer_norm = build_part("norm", layer_spec.after_mixer_norm)
        self.feed_forward_norm = self.feed_forward = self.after_feed_forward_norm = None
        if "feed_forward" in layer_spec.parts:
            self.feed_forward_norm = build_part("norm", layer_spec.feed_forward_norm)
            self.feed_forward = build_part("feed_forward", layer_spec.feed_forward)
            self.after_feed_forward_norm = build_part("norm", layer_spec.after_feed_forward_norm)

    def parts(self):
        first = (self.mixer_norm, self.mixer, self.after_mixer_norm)
        if self.feed_forward is None:
            return first
        return first + (self.feed_forward_norm, self.feed_forward, self.after_feed_forward_norm)

    def entry_norm(self):
        """The norm through which this layer first reads the stream."""
        return self.mixer_norm

    def entry_takes_tiled(self, rows: int) -> bool:
        return _takes_tiled(self.mixer, rows)

    def _open(self, stream, norm, act_dtype, tiled: bool):
        prepared = getattr(stream, "prepared", None)
        stream.prepared = None
        if prepared is not None and prepared[0] is norm and stream.pending is None and stream.later is None:
            return prepared[1]
        return stream.normed(norm, act_dtype, tiled=tiled)

    def _close(self, stream, y, norm, reader, act_dtype, tiled: bool) -> None:
        if isinstance(y, tuple):
            raise ConfigError("a sublayer with a norm behind it hands back its result, not a link to a norm")
        y = y if isinstance(y, torch.Tensor) else ops.as_rows(y)
        stream.as_act = None                     # a copy of the residual that another arrangement left is out of date
        with profiler.section(profiler.NORM):
            args = (stream.sum, y, norm.gain, getattr(norm, "bias", None), norm.eps, norm.kind, None)
            if isinstance(reader, RMSNorm) and reader.dim == norm.dim:
                tiled = (tiled and act_dtype == torch.bfloat16 and stream.rows <= TILED_MAX_ROWS and norm.dim % 4 == 0
                         and norm.dim <= 8192)
                stream.prepared = (reader, ops.branch_norm_add_norm(*args, reader.gain, reader.eps, act_dtype, tiled))
            else:
                stream.prepared = None
                ops.branch_norm_add(*args)

    def forward(self, stream: ResidualStream, ctx, store, page_table, act_dtype) -> None:
        rows = stream.rows
        h = self._open(stream, self.mixer_norm, act_dtype, _takes_tiled(self.mixer, rows))
        y = self.mixer.forward(h, ctx, store, page_table)
        if self.feed_forward is None:
            self._close(stream, y, self.after_mixer_norm, stream.next_entry_norm, act_dtype, stream.next_entry_tiled)
            return
        self._close(stream, y, self.after_mixer_norm, self.feed_forward_norm, act_dtype, _takes_tiled(self.feed_forward, rows))
        h = self._open(stream, self.feed_forward_norm, act_dtype, _takes_tiled(self.feed_forward, rows))
        self._close(stream, self.feed_forward.forward(h, ctx), self.after_feed_forward_norm, stream.next_entry_norm, act_dtype,
                    stream.next_entry_tiled)
