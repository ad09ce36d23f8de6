"""RMSNorm, fused with the residual add that precedes it."""
from __future__ import annotations

import torch

from ..kernels import ops, plain
from ..weights.loader import BIAS, GAIN, OFFSET, TensorSpec
from .base import Norm
from .registry import register_part


@register_part("norm", "rmsnorm")
class RMSNorm(Norm):
    """``y = x * (1 / sqrt(mean(x^2) + eps)) * w`` over the last axis, statistics in
    float32 (the reference: src/ops/norm.rs:7-32; fused with the add: :35-62).  ``from_one``: the stored weight is the
    gain's distance from one, ``w = 1 + stored``; ``scale``: a constant on the norm's output.  Both go into the float32 gain
    when the weights are bound."""

    accepts_parts = True
    kind = ops.NORM_RMS      # what the kernel that also writes and reads several residual streams calls this norm
    linkable = True          # gain, eps and dim are all a product needs to do this norm itself
    can_tile = True          # hands its rows on in the matrix cores' order when asked (up to 64 rows)

    def __init__(self, dim: int, eps: float, name: str, from_one: bool = False, scale: float = 1.0):
        self.dim, self.eps, self.name, self.from_one, self.scale = dim, eps, name, bool(from_one), float(scale)

    def tensors(self):
        return {self.name: TensorSpec((self.dim,), OFFSET if self.from_one else GAIN)}

    def _gain(self, stored):
        g = 1.0 + stored.to(torch.float32) if self.from_one else stored.to(torch.float32)
        return g if self.scale == 1.0 else g * self.scale

    def bind(self, weights, rt):
        self.rt = rt
        self.gain = rt.place_gain(self._gain(weights[self.name]))

    def bind_plain(self, weights):
        self.gain_plain = self._gain(weights[self.name]).numpy()

    def plain(self, x):
        return plain.rms_norm(x, self.gain_plain, self.eps)

    accepts_branches = True

    def apply_branches(self, residual, branches, out_dtype, rows=None):
        """``apply`` for several float32 branches that wait side by side."""
        return ops.add_branches_rmsnorm(residual, branches, self.gain, self.eps, out_dtype, rows)

    def apply(self, residual, pending, out_dtype, rows=None, tiled=False):
        tiled = tiled and self.dim % 4 == 0 and self.dim <= 8192        # what the vectorised kernel takes
        return ops.add_rmsnorm(residual, pending, self.gain, self.eps, out_dtype, rows, tiled=tiled)


@register_part("norm", "layernorm")
class LayerNorm(Norm):
    """``y = (x - mean) / sqrt(var + eps) * w + b`` over the last axis, ``var`` the mean of the squared deviations,
    statistics in float32; the bias is optional (``bias_name`` None: none).  Fused with the residual add that
    precedes it, and, for a residual kept in several streams, with the streams' write and read
    (``ops.streams_read_norm``)."""

    accepts_parts = True
    kind = ops.NORM_LAYER

    def __init__(self, dim: int, eps: float, name: str, bias_name: str | None = None):
        self.dim, self.eps, self.name, self.bias_name = dim, eps, name, bias_name

    def tensors(self):
        t = {self.name: TensorSpec((self.dim,), GAIN)}
        if self.bias_name:
            t[self.bias_name] = TensorSpec((self.dim,), BIAS)
        return t

    def bind(self, weights, rt):
        self.rt = rt
        self.gain = rt.place_gain(weights[self.name])
        self.bias = rt.place_gain(weights[self.bias_name]) if self.bias_name else None

    def apply(self, residual, pending, out_dtype, rows=None, tiled=False):
        # one stream without coefficients: residual += pending, then the norm
        return ops.streams_read_norm(residual.view(residual.shape[0], 1, self.dim), pending, None, None, None,
                                     self.gain, self.bias, self.eps, self.kind, out_dtype, rows)
