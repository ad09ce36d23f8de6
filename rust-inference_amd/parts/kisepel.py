"""Kisepel as a list of parts.

Embedding: the token's row times a constant.  A layer has one norm, whose rows its mixer and its feed-forward both read, and
both results are added to the residual: ``h = norm(x)``, ``x <- x + mixer(h) + ff(h)``, RMS norms with weights stored as their
distance from one.  The mixer is linear attention with a fixed decay per head, a state-space mixer with a scalar decay per head,
or two mixers side by side, each through an RMS norm over the model's width, half their sum: softmax attention in chunks of the
sequence (per-head q/k RMS norm, rotation in halves over the first part of a head with linearly scaled frequencies, a score
factor) and the gated delta rule (short convolutions over q, k and v, unit q and k, a decay per head and key channel and an
output gate through narrow middles).  The feed-forward is a mixture of silu-gated experts that a table of token ids chooses, with
equal weights, beside an expert every token uses.  A stretch of the layers may run several times in a row with the same weights,
every pass with cache entries of its own and, from the second on, with the embedding's output added first.  Final RMS norm; the
output matrix is the embedding table, and the logits are multiplied by a constant.

Checkpoint names: ``embed``, ``l<i>.norm1``, ``l<i>.mix.*`` (``mix.left.*`` / ``mix.right.*``), ``l<i>.mlp.*``, ``final.norm``.
"""
from __future__ import annotations

from ..config import KisepelConfig, register_architecture
from ..config.kisepel import PairSizes, TableExpertsSizes
from ..config.dagezen import StateSpaceSizes
from .spec import LayerSpec, ModelSpec, PartSpec, Run


def _norm(cfg: KisepelConfig, name: str, scale: float = 1.0) -> PartSpec:
    return PartSpec("rmsnorm", {"dim": cfg.width, "eps": cfg.norm_eps, "name": name, "from_one": True, "scale": scale})


def _mixer(cfg: KisepelConfig, m, p: str):
    """The mixer's part and how many things it keeps per sequence."""
    if isinstance(m, StateSpaceSizes):
        return PartSpec("state_space", {"hidden": cfg.width, "heads": m.heads, "vdim": m.vdim, "state": m.state,
                                        "groups": m.groups, "taps": m.conv, "norm_groups": m.norm_groups, "prefix": p,
                                        "eps": cfg.norm_eps}), 2
    if not isinstance(m, PairSizes):
        return PartSpec("decay_attention", {"hidden": cfg.width, "heads": m.heads, "dim": m.dim, "vdim": m.vdim, "decay": m.decay,
                                            "prefix": p, "eps": cfg.norm_eps, "gate": "sigmoid"}), 1
    a, r = m.left, m.right
    lp, rp = p + "left.", p + "right."
    position = PartSpec("none")
    if a.rot_dims:
        position = PartSpec("rotate_half", {"head_dim": a.dim, "theta": a.rot_base, "dims": a.rot_dims, "factor": a.rot_factor})
    left = PartSpec("attention", {
        "hidden": cfg.width, "heads": a.heads, "kv_heads": a.kv_heads, "head_dim": a.dim, "v_dim": a.vdim, "prefix": lp,
        "qk_norm": True, "eps": cfg.norm_eps, "scale": a.scale, "chunk": a.chunk, "position": position,
        "names": {"q": lp + "q", "k": lp + "k", "v": lp + "v", "o": lp + "o", "q_norm": lp + "q.norm", "k_norm": lp + "k.norm"},
    })
    right = PartSpec("delta", {"hidden": cfg.width, "heads": r.heads, "kv_heads": r.kv_heads, "dim": r.dim, "vdim": r.vdim,
                               "taps": r.conv, "prefix": rp, "eps": cfg.norm_eps, "decay": "channel", "rank": r.rank})
    return PartSpec("parallel", {"mixers": (left, right), "scales": (0.5, 0.5), "norms": (lp + "out", rp + "out"),
                                 "hidden": cfg.width, "eps": cfg.norm_eps}), 3


def _feed_forward(cfg: KisepelConfig, mlp: TableExpertsSizes, p: str) -> PartSpec:
    return PartSpec("routed_experts", {"hidden": cfg.width, "inter": mlp.ff, "experts": mlp.experts, "top": mlp.top, "limit": None,
                                       "prefix": p, "scores": "table", "vocab": cfg.vocab, "shared": mlp.shared_ff,
                                       "shared_gate": False})


def kisepel_spec(cfg: KisepelConfig) -> ModelSpec:
    layers, kept = [], []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        mixer, entries = _mixer(cfg, layer.mixer, p + "mix.")
        parts = {"mixer_norm": _norm(cfg, p + "norm1"), "mixer": mixer}
        if layer.mlp is not None:
            parts["feed_forward"] = _feed_forward(cfg, layer.mlp, p + "mlp.")
        layers.append(LayerSpec("parallel_prenorm", parts))
        kept.append(entries)
    # every run of a layer, a looped one's every pass too, keeps its own keys and values or state
    schedule, at = [], 0
    for i, again in cfg.order():
        n = kept[i]
        schedule.append(Run(layer=i, cache=at if n == 1 else tuple(range(at, at + n)), add_embedding=again))
        at += n
    return ModelSpec(
        architecture=cfg.ARCHITECTURE,
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        embedding=PartSpec("table", {"vocab": cfg.vocab, "dim": cfg.width, "name": "embed", "scale": cfg.embedding_scale}),
        layers=tuple(layers),
        schedule=tuple(schedule),
        # the constant on the logits rides on the last norm's rows: the output matrix is linear in them
        final_norm=_norm(cfg, "final.norm", cfg.logit_scale),
        head=PartSpec("linear", {"vocab": cfg.vocab, "dim": cfg.width, "name": "head", "tied": True}),
        max_positions=cfg.max_positions,
    )


register_architecture("Kisepel", KisepelConfig, kisepel_spec, model_types=("kisepel",))
