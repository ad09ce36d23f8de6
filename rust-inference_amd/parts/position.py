"""Position encodings."""
from __future__ import annotations

import math

import torch

from ..errors import ConfigError
from .base import PositionEncoding
from .registry import register_part


@register_part("position", "rotate_half")
class RotateHalf(PositionEncoding):
    """Rotary encoding of the "default" kind over the whole head, pairs ``(d, d + dh/2)``.
    ``inv_freq[i] = 1 / theta^(2i / dh)`` in float32 (the reference: src/ops/rope.rs:20);
    the kernel forms the angle ``f32(pos) * inv_freq[i]`` in float32 (:39) and rotates
    ``x'[d] = x[d] cos - x[d+half] sin``, ``x'[d+half] = x[d+half] cos + x[d] sin`` (:73-74).

    ``dims``: only the first ``dims`` elements of a head turn (pairs ``(d, d + dims/2)``), with ``theta^(-2i / dims)`` taken in
    64-bit and rounded once.  ``stretch = {factor, original, fast, slow}`` slows the pairs down for contexts ``factor`` times
    as long as ``original``: with ``i(t) = dims ln(original / (2 pi t)) / (2 ln theta)``, the place of a pair that turns ``t`` times
    in the original context, a pair's frequency runs from its own (``i <= floor(i(fast))``) to ``1/factor`` of it (``i >=
    ceil(i(slow))``), linearly in ``i`` between; and ``amplitude = 0.1 ln(factor) + 1`` multiplies cosine and sine.  ``factor``:
    every pair's frequency is divided by it (linear scaling)."""

    amplitude = 1.0

    def __init__(self, head_dim: int, theta: float, dims: int | None = None, stretch: dict | None = None,
                 factor: float = 1.0):
        if not factor > 0:
            raise ConfigError(f"a rotation's frequencies divided by {factor}")
        self.factor = float(factor)
        if dims is None and self.factor != 1.0:
            dims = head_dim
        if head_dim % 2 and dims is None:
            raise ConfigError(f"head_dim {head_dim} must be even for a rotation in pairs")
        if dims is not None and (dims % 2 or not 2 <= dims <= head_dim):
            raise ConfigError(f"a rotation over {dims} of {head_dim} elements: an even number up to the head size")
        self.head_dim, self.theta, self.dims, self.stretch = head_dim, theta, dims, stretch
        if stretch is not None:
            self.dims = dims or head_dim
            self.amplitude = 0.1 * math.log(stretch["factor"]) + 1.0

    def part_frequencies(self) -> torch.Tensor:
        """The frequencies of a rotation over part of a head, stretched or not (float64)."""
        dims, base = self.dims, float(self.theta)
        i = torch.arange(dims // 2, dtype=torch.float64)
        f = torch.pow(torch.tensor(base, dtype=torch.float64), -2.0 * i / dims)
        f = f / self.factor
        if self.stretch is None:
            return f
        s = self.stretch
        place = lambda turns: dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
        first, last = max(math.floor(place(s["fast"])), 0), min(math.ceil(place(s["slow"])), dims - 1)
        ramp = ((i - first) / max(last - first, 0.001)).clamp(0.0, 1.0)
        return f / s["factor"] * ramp + f * (1.0 - ramp)

    def bind(self, weights, rt):
        self.rt = rt
        if self.dims is not None:
            self.inv_freq = self.part_frequencies().to(torch.float32).to(rt.device).contiguous()
            return
        i = torch.arange(self.head_dim // 2, dtype=torch.float32)
        expo = (2.0 * i) / torch.tensor(float(self.head_dim), dtype=torch.float32)
        theta = torch.tensor(self.theta, dtype=torch.float32)
        self.inv_freq = (1.0 / torch.pow(theta, expo)).to(torch.float32).to(rt.device).contiguous()

    def bind_plain(self, weights):
        from ..kernels import plain
        if self.dims is not None:
            raise ConfigError("a rotation over part of a head, or with stretched frequencies, has no plain form")
        self.inv_freq_plain = plain.rope_inv_freq(self.head_dim, self.theta)

    def plain(self, heads, positions):
        """Rotates ``heads: [tokens, n, head_dim]`` (already normed) by their tokens' positions."""
        from ..kernels import plain
        return plain.rope(heads, positions, self.inv_freq_plain)

    def rotation_table(self):
        return self.inv_freq


@register_part("position", "none")
class NoPosition(PositionEncoding):
    """No position enters the mixer (order then comes from the causal mask alone)."""

    def __init__(self, **_):
        pass

    def bind_plain(self, weights):
        pass

    def plain(self, heads, positions):
        return heads


@register_part("position", "rotate_pairs")
class RotatePairs(PositionEncoding):
    """Rotary encoding over the first ``dims`` elements of a head, in neighbouring pairs: the elements ``(2i, 2i + 1)``
    at position ``p`` turn by the angle ``p * base^(-2i / dims)`` (``i < dims / 2``); what lies behind ``dims`` passes
    unchanged.  The frequencies are rounded to float32 once; angle, sine and cosine are float32 in the kernel.
    ``pairs`` tells the mixer that neighbours turn (not the halves of a head): it then rotates before it norms."""

    pairs = True

    def __init__(self, head_dim: int, dims: int, base: float):
        if dims % 2 or not 0 <= dims <= head_dim:
            raise ConfigError(f"a rotation over {dims} of {head_dim} elements: an even number up to the head size")
        if dims and not base > 0:
            raise ConfigError(f"the rotation's base {base} must be positive")
        self.head_dim, self.dims, self.base = head_dim, dims, float(base)

    def bind(self, weights, rt):
        self.rt = rt
        self.inv_freq = None
        if self.dims:
            i = torch.arange(self.dims // 2, dtype=torch.float64)
            self.inv_freq = torch.pow(torch.tensor(self.base, dtype=torch.float64), -2.0 * i / self.dims) \
                .to(torch.float32).to(rt.device).contiguous()

    def rotation_table(self):
        return self.inv_freq
