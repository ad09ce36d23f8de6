"""The gated delta rule: a mixer that keeps a float32 state per head and the tails of three short convolutions."""
from __future__ import annotations

import torch

from .. import profiler
from ..cache import StateNeed
from ..errors import ConfigError
from ..kernels import ops
from ..weights.loader import BIAS, GAIN, MATRIX, TensorSpec
from .base import Mixer
from .registry import register_part


@register_part("mixer", "delta")
class GatedDeltaRule(Mixer):
    """With ``q = W_q h`` and ``k = W_k h`` (``kv_heads x dim``, shared by ``heads / kv_heads`` value heads each) and
    ``v = W_v h`` (``heads x vdim``): each of q, k and v goes through a causal convolution over time per channel
    (``taps`` taps, the last one the current token's, zeros before a sequence's start) and silu; q and k become unit
    vectors per head, ``x / sqrt(sum x^2 + 1e-6)``, q also times ``dim^(-1/2)``; ``beta = sigmoid(W_b h)`` and
    ``g = exp(-exp(A_log) softplus(W_a h + dt_bias))`` per value head.  Per head and token

        S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q,

    so that the read-out sees the token's own write.  Each head's ``o`` goes through an RMS norm over ``vdim`` (one
    gain for all heads), the heads side by side are multiplied by ``silu(W_g h)`` and projected by ``W_o``.

    Per sequence the mixer keeps two things, in this order: the state ``[heads, dim, vdim]`` and the last ``taps - 1``
    inputs of the convolutions ``[taps - 1, channels]``, both float32 and zero when the sequence starts; a run of a
    layer with this mixer names two cache entries.  Everything after the projections is float32.

    ``names``: checkpoint names of ``q, k, v, g, o, a, b, norm, A_log, dt_bias`` where they are not ``<prefix>q`` and
    so on; the taps of q, k and v are ``<name>.conv``.  q, k, v and g are one product with the row-concatenated
    weight, a and b another whose result is float32.

    ``decay="channel"``: a decay per value head and key channel, through a narrow middle whose width the checkpoint gives
    (unless ``rank`` names it): ``g = exp(-exp(A_log_h) softplus(W_a2 (W_a1 h) + dt_bias))`` with ``dt_bias [heads * dim]``, and
    ``S <- diag(g) S``; the output gate then is ``sigmoid(W_g2 (W_g1 h))``, through a middle of its own.  Names ``a1, a2, g1, g2`` in
    the place of ``a`` and ``g``.  q, k, v, both middles and the logits of beta are one product, both second steps another, with
    the block-diagonal of ``a2`` and ``g2``, whose result is float32.  This form can share one input product with other mixers
    (``in_matrix``, ``heads_from``).
    """

    def __init__(self, hidden: int, heads: int, kv_heads: int, dim: int, vdim: int, taps: int, prefix: str,
                 eps: float = 1e-5, names: dict | None = None, decay: str = "head", rank: int | None = None):
        if decay not in ("head", "channel"):
            raise ConfigError(f"a delta rule's decay {decay!r} is neither 'head' nor 'channel'")
        if heads < 1 or kv_heads < 1 or heads % kv_heads:
            raise ConfigError(f"{heads} delta-rule heads not divisible by {kv_heads} query/key heads")
        if not 1 <= dim <= ops.DELTA_MAX_DIM or vdim < 1:
            raise ConfigError(f"a delta rule with heads of {dim} x {vdim}: the kernels take key heads of 1 to {ops.DELTA_MAX_DIM}")
        if not 1 <= taps <= ops.DELTA_MAX_TAPS:
            raise ConfigError(f"short convolutions of {taps} taps: the kernels take 1 to {ops.DELTA_MAX_TAPS}")
        self.hidden, self.heads, self.kv_heads, self.dim, self.vdim, self.taps = hidden, heads, kv_heads, dim, vdim, taps
        self.prefix, self.eps = prefix, eps
        p = prefix
        self.per_channel, self.rank = decay == "channel", rank
        self.names = {n: p + n for n in ("q", "k", "v", "g", "o", "a", "b", "norm", "A_log", "dt_bias", "a1", "a2", "g1", "g2")}
        self.names.update(names or {})
        self.channels = 2 * kv_heads * dim + heads * vdim

    def tensors(self):
        n, d, hk, hv, h = self.names, self.hidden, self.kv_heads * self.dim, self.heads * self.vdim, self.heads
        if self.per_channel:
            hd = h * self.dim
            return {
                n["q"]: TensorSpec((hk, d), MATRIX), n["k"]: TensorSpec((hk, d), MATRIX), n["v"]: TensorSpec((hv, d), MATRIX),
                n["q"] + ".conv": TensorSpec((hk, self.taps), MATRIX), n["k"] + ".conv": TensorSpec((hk, self.taps), MATRIX),
                n["v"] + ".conv": TensorSpec((hv, self.taps), MATRIX), n["o"]: TensorSpec((d, hv), MATRIX),
                n["a1"]: TensorSpec((self.rank, d), MATRIX), n["a2"]: TensorSpec((hd, self.rank), MATRIX),
                n["g1"]: TensorSpec((self.rank, d), MATRIX), n["g2"]: TensorSpec((hv, self.rank), MATRIX),
                n["b"]: TensorSpec((h, d), MATRIX), n["A_log"]: TensorSpec((h,), BIAS), n["dt_bias"]: TensorSpec((hd,), BIAS),
                n["norm"]: TensorSpec((self.vdim,), GAIN),
            }
        return {
            n["q"]: TensorSpec((hk, d), MATRIX), n["k"]: TensorSpec((hk, d), MATRIX), n["v"]: TensorSpec((hv, d), MATRIX),
            n["q"] + ".conv": TensorSpec((hk, self.taps), MATRIX), n["k"] + ".conv": TensorSpec((hk, self.taps), MATRIX),
            n["v"] + ".conv": TensorSpec((hv, self.taps), MATRIX),
            n["g"]: TensorSpec((hv, d), MATRIX), n["o"]: TensorSpec((d, hv), MATRIX),
            n["a"]: TensorSpec((h, d), MATRIX), n["b"]: TensorSpec((h, d), MATRIX),
            n["A_log"]: TensorSpec((h,), BIAS), n["dt_bias"]: TensorSpec((h,), BIAS),
            n["norm"]: TensorSpec((self.vdim,), GAIN),
        }

    def in_matrix(self, weights):
        """The rows of this mixer's input product (of the form with a decay per channel): q, k, v, the two middles, the logits of
        beta, each group on a multiple of 8 (zero rows between)."""
        n = self.names
        groups = ([weights[n[x]] for x in "qkv"], [weights[n["a1"]], weights[n["g1"]]], [weights[n["b"]]])
        rows = []
        for group in groups:
            rows += group
            rows.append(group[0].new_zeros((-sum(w.shape[0] for w in group) % 8, group[0].shape[1])))
        return torch.cat(rows, 0)

    def out_matrix(self, weights):
        return weights[self.names["o"]]

    def bind_channels(self, weights, rt, alone: bool) -> None:
        n = self.names
        a1, a2, g1, g2 = (weights[n[x]] for x in ("a1", "a2", "g1", "g2"))
        for one, two in (("a1", "a2"), ("g1", "g2")):
            if weights[n[one]].shape[0] != weights[n[two]].shape[1]:
                raise ConfigError(f"{n[one]} has {weights[n[one]].shape[0]} rows, {n[two]} {weights[n[two]].shape[1]} columns")
        ra, rg = a1.shape[0], g1.shape[0]
        self.mid_at, self.mid_width = -(-self.channels // 8) * 8, -(-(ra + rg) // 8) * 8
        self.b_at = self.mid_at + self.mid_width
        second = torch.zeros((a2.shape[0] + g2.shape[0], self.mid_width), dtype=a1.dtype, device=a1.device)
        second[:a2.shape[0], :ra], second[a2.shape[0]:, ra:ra + rg] = a2, g2
        self.w_second = rt.pack(rt.place_matrix(second))
        if alone:
            self.w_in = rt.pack(rt.place_matrix(self.in_matrix(weights)), always=True)

    def bind(self, weights, rt, alone: bool = True):
        """``alone`` False: another part owns the products before and after (mixers side by side)."""
        self.rt = rt
        n = self.names
        if self.per_channel:
            self.bind_channels(weights, rt, alone)
            self.conv_taps = rt.place_gain(torch.cat([weights[n[x] + ".conv"] for x in "qkv"], 0))
            self.a_log, self.dt_bias = rt.place_gain(weights[n["A_log"]]), rt.place_gain(weights[n["dt_bias"]])
            self.gain = rt.place_gain(weights[n["norm"]])
            if alone:
                self.w_o = rt.pack(rt.place_matrix(weights[n["o"]]), parts_ok=True)
            return
        fused = torch.cat([weights[n["q"]], weights[n["k"]], weights[n["v"]], weights[n["g"]]], 0)
        self.w_qkvg = rt.pack(rt.place_matrix(fused), always=True)      # four projections in one
        self.w_ab = rt.pack(rt.place_matrix(torch.cat([weights[n["a"]], weights[n["b"]]], 0)))
        self.conv_taps = rt.place_gain(torch.cat([weights[n[x] + ".conv"] for x in "qkv"], 0))
        self.a_log, self.dt_bias = rt.place_gain(weights[n["A_log"]]), rt.place_gain(weights[n["dt_bias"]])
        self.gain = rt.place_gain(weights[n["norm"]])
        self.w_o = rt.pack(rt.place_matrix(weights[n["o"]]), parts_ok=True)

    def cache_need(self):
        return (StateNeed((self.heads, self.dim, self.vdim), torch.float32),
                StateNeed((self.taps - 1, self.channels), torch.float32))

    def heads_from(self, x, proj, col0: int, ctx, store, page_table):
        """The form with a decay per channel between its two products: ``proj [T, row]`` holds the columns of ``in_matrix`` from
        ``col0`` on; the normed and gated heads, ready for the output product."""
        rt = self.rt
        state, tails = store
        sizes = (self.heads, self.kv_heads, self.dim, self.vdim)
        with profiler.section(profiler.QKV_PROJECTION):
            mid = ops.take_columns(proj, col0 + self.mid_at, self.mid_width)         # [T, a1 | g1]
            z = ops.as_rows(rt.linear_packed(mid, self.w_second, out_dtype=torch.float32))      # [T, decays | gates]
        gate_at = self.heads * self.dim
        one_form = rt.dtype == torch.float32 or rt.invariant
        with profiler.section(profiler.ATTENTION):
            if ctx.is_decode and not one_form and ops.delta_step_fits(self.dim, self.vdim):
                return ops.delta_step_channels(proj, col0, self.conv_taps, tails, z, gate_at, proj, col0 + self.b_at, self.a_log, self.dt_bias,
                                               state, ctx.cu_seqlens, ctx.slots, self.gain, self.eps, *sizes)
            qkv, gates = ops.delta_prepare_channels(proj, col0, self.conv_taps, tails, z, proj, col0 + self.b_at, self.a_log, self.dt_bias,
                                                    ctx.tok_seq, ctx.cu_seqlens, ctx.slots, *sizes)
            o = ops.delta_scan_channels(qkv, gates, state, ctx.cu_seqlens, ctx.slots, *sizes, slices=4 if one_form else 0)
            return ops.head_norm_gate(o, z, gate_at, self.gain, self.eps, self.heads, self.vdim, rt.dtype, ops.GATE_SIGMOID)

    def forward(self, x, ctx, store, page_table):
        rt = self.rt
        if self.per_channel:
            with profiler.section(profiler.QKV_PROJECTION):
                proj = ops.as_rows(rt.linear_packed(x, self.w_in))
            heads = self.heads_from(x, proj, 0, ctx, store, page_table)
            with profiler.section(profiler.OUT_PROJECTION):
                return rt.linear_packed(heads, self.w_o, out_dtype=torch.float32, parts_ok=True)
        state, tails = store
        with profiler.section(profiler.QKV_PROJECTION):
            proj = ops.as_rows(rt.linear_packed(x, self.w_qkvg))          # [T, q | k | v | g]
            ab = rt.linear_packed(x, self.w_ab, out_dtype=torch.float32)
        # float32 and the invariant mode run one form of every kernel whatever the step looks like
        one_form = rt.dtype == torch.float32 or rt.invariant
        if ctx.is_decode and not one_form and ops.delta_step_fits(self.dim, self.vdim):
            # one token a sequence: convolutions, unit norms, gates, the step on the state, norm and gate are one kernel
            with profiler.section(profiler.ATTENTION):
                y = ops.delta_step(proj, 0, self.channels, self.conv_taps, tails, ab, self.a_log, self.dt_bias, state,
                                   ctx.cu_seqlens, ctx.slots, self.gain, self.eps, self.heads, self.kv_heads, self.dim,
                                   self.vdim)
            with profiler.section(profiler.OUT_PROJECTION):
                return rt.linear_packed(y, self.w_o, out_dtype=torch.float32, parts_ok=True)
        with profiler.section(profiler.ATTENTION):
            qkv, gates = ops.delta_prepare(proj, 0, self.conv_taps, tails, ab, self.a_log, self.dt_bias, ctx.tok_seq,
                                           ctx.cu_seqlens, ctx.slots, self.heads, self.kv_heads, self.dim, self.vdim)
            o = ops.delta_scan(qkv, gates, state, ctx.cu_seqlens, ctx.slots, self.heads, self.kv_heads, self.dim,
                               self.vdim, slices=4 if one_form else 0)
            y = ops.gla_norm_gate(o, proj, self.channels, self.gain, self.eps, self.heads, self.vdim)
        with profiler.section(profiler.OUT_PROJECTION):
            return rt.linear_packed(y, self.w_o, out_dtype=torch.float32, parts_ok=True)
