"""Notadra as a list of parts.

Embedding: the token's row plus a row for the pair of the token before and the token; the last token is kept per
sequence.  Every layer norms before and after each sublayer, ``x <- x + norm1b(mixer(norm1(x)))``,
``x <- x + norm2b(ff(norm2(x)))``, RMS norms whose stored weight is the gain's distance from one.  The mixer is softmax
attention with biases on q, k and v, a rotation in halves over the first part of a head with stretched frequencies,
scaled and capped scores and a sink of score 0; a layer may read the keys and values of an earlier one, whose cache
entry its run then names.  The feed-forward is a mixture of squared-ReLU experts: sigmoid router, a correction for the
choice alone, groups scored by their two best, weights not renormalized.  Final norm; the output matrix is a tensor of its
own and the logits are scaled.

Checkpoint names: ``embed``, ``bigram``, ``l<i>.norm1`` / ``norm1b`` / ``norm2`` / ``norm2b``, ``l<i>.mix.{q,k,v,o}`` (+ ``.b`` for
q, k and v), ``l<i>.mlp.*``, ``final.norm``, ``head``.
"""
from __future__ import annotations

from ..config import NotadraConfig, register_architecture
from .spec import LayerSpec, ModelSpec, PartSpec, Run


def _norm(cfg: NotadraConfig, name: str, scale: float = 1.0) -> PartSpec:
    return PartSpec("rmsnorm", {"dim": cfg.width, "eps": cfg.norm_eps, "name": name, "from_one": True, "scale": scale})


def _mixer(cfg: NotadraConfig, m, p: str) -> PartSpec:
    position = PartSpec("none")
    if m.rot_dims:
        position = PartSpec("rotate_half", {"head_dim": m.dim, "theta": m.rot_base, "dims": m.rot_dims,
                                            "stretch": None if m.scaling is None else m.scaling.to_dict()})
    return PartSpec("attention", {
        "hidden": cfg.width, "heads": m.heads, "kv_heads": m.kv_heads, "head_dim": m.dim, "v_dim": m.vdim, "prefix": p,
        "qk_norm": False, "eps": cfg.norm_eps, "scale": m.scale, "softcap": m.softcap, "position": position, "qkv_bias": True,
        "sinks": "zero", "reads_kv": m.kv_from is not None,
        "names": {x: p + x for x in ("q", "k", "v", "o")} | {x + "_bias": p + x + ".b" for x in ("q", "k", "v")},
    })


def _feed_forward(cfg: NotadraConfig, mlp, p: str) -> PartSpec:
    return PartSpec("routed_experts", {"hidden": cfg.width, "inter": mlp.ff, "experts": mlp.experts, "top": mlp.top, "limit": None,
                                       "prefix": p, "scores": "sigmoid", "normalize": False, "groups": (mlp.groups, mlp.keep),
                                       "group_score": "best_two", "gated": False, "activation": "relu2"})


def notadra_spec(cfg: NotadraConfig) -> ModelSpec:
    layers, schedule, entry_of, entries = [], [], {}, 0
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        parts = {"mixer_norm": _norm(cfg, p + "norm1"), "mixer": _mixer(cfg, layer.mixer, p + "mix."),
                 "after_mixer_norm": _norm(cfg, p + "norm1b")}
        if layer.mlp is not None:
            parts["feed_forward_norm"] = _norm(cfg, p + "norm2")
            parts["feed_forward"] = _feed_forward(cfg, layer.mlp, p + "mlp.")
            parts["after_feed_forward_norm"] = _norm(cfg, p + "norm2b")
        layers.append(LayerSpec("sandwich", parts))
        if layer.mixer.kv_from is None:
            entry_of[i], entries = entries, entries + 1
        schedule.append(Run(layer=i, cache=entry_of[i if layer.mixer.kv_from is None else layer.mixer.kv_from]))
    embedding = {"vocab": cfg.vocab, "dim": cfg.width, "name": "embed"}
    if cfg.bigram is not None:
        embedding = PartSpec("table_bigram", {**embedding, "bigram_name": "bigram", **cfg.bigram.to_dict()})
    else:
        embedding = PartSpec("table", embedding)
    return ModelSpec(
        architecture=cfg.ARCHITECTURE,
        vocab_size=cfg.vocab,
        hidden_size=cfg.width,
        embedding=embedding,
        embedding_cache=entries if cfg.bigram is not None else None,
        layers=tuple(layers),
        schedule=tuple(schedule),
        # the constant on the logits rides on the last norm's rows: the output matrix is linear in them
        final_norm=_norm(cfg, "final.norm", cfg.logit_scale),
        head=PartSpec("linear", {"vocab": cfg.vocab, "dim": cfg.width, "name": "head", "tied": False}),
        max_positions=cfg.max_positions,
    )


register_architecture("Notadra", NotadraConfig, notadra_spec, model_types=("notadra",))
