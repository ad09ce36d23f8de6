"""The Notadra design without a GPU: configuration, registry, schedule and cache entries, tensor names, and the plain
implementation (tests/plain/notadra_plain.py) against itself and against examples worked out by hand."""
import copy
import math

import numpy as np
import pytest
import torch

from plain import notadra_plain as P


def attention(heads, kv_heads, dim, vdim, scale, cap=8.0, rot_dims=None, base=100.0, stretch=(3.0, 24, 6.0, 0.6), kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if cap:
        m["softcap"] = cap
    if rot_dims != 0:
        m["rot"] = {"dims": dim if rot_dims is None else rot_dims, "base": base}
        if stretch:
            m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), stretch))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def moe(experts, top, ff, groups=None):
    router = {"experts": experts, "top": top}
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": router}


def layer(mixer, mlp):
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def model(layers, vocab=97, width=40, eps=1e-5, logit_scale=1.7, bigram=(53, 29, 11)):
    return {"architecture": "Notadra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale,
            "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}, "layers": layers}


SMALL = model([layer(attention(4, 2, 8, 12, 0.4, rot_dims=4), moe(6, 3, 12, (3, 2))), layer(attention(6, 2, 8, 12, 0.3, cap=5.0, rot_dims=4, kv_from=0), None),
               layer(attention(2, 2, 16, 16, 0.5, stretch=(3.0, 200, 6.0, 0.6)), moe(4, 2, 10))])


def random_weights(cfg, seed=0, std=0.25):
    from rust_inference_amd.config import config_from_dict
    from rust_inference_amd.parts.model import DecoderModel
    from rust_inference_amd.weights.random_init import random_tensors
    arch, typed = config_from_dict(cfg)
    specs = DecoderModel(arch.build_spec(typed)).tensors(for_writing=True)
    return {k: v.to(torch.float64).numpy() for k, v in random_tensors(specs, seed, torch.float32, matrix_std=std).items()}


def test_configuration_reads_back_and_builds_the_parts():
    from rust_inference_amd.cache import KVNeed, StateNeed
    from rust_inference_amd.config import config_from_dict
    from rust_inference_amd.parts.model import DecoderModel
    arch, cfg = config_from_dict(SMALL)
    assert arch.name == "Notadra" and cfg.logit_scale == pytest.approx(1.7) and cfg.bigram.buckets == 53
    assert config_from_dict(cfg.to_dict())[1] == cfg
    spec = arch.build_spec(cfg)
    assert [l.arrangement for l in spec.layers] == ["sandwich"] * 3
    # the second layer reads the first one's entry; the embedding's is behind the layers'
    assert [r.cache for r in spec.schedule] == [0, 0, 1] and spec.embedding_cache == 2 and spec.num_cache_entries == 3
    m = DecoderModel(spec)
    assert m.cache_needs() == [KVNeed(2, 8, None, 12), KVNeed(2, 16), StateNeed((1,), torch.int32)]
    t = m.tensors()
    for n in ("embed", "bigram", "final.norm", "head", "l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l0.mix.q.b", "l0.mix.k", "l0.mix.k.b", "l0.mix.v.b",
              "l0.mix.o", "l0.mlp.router", "l0.mlp.correction", "l0.mlp.e5.up", "l0.mlp.e5.down", "l1.mix.q", "l1.mix.q.b", "l1.mix.o", "l1.norm1b"):
        assert n in t, n
    for n in ("l1.mix.k", "l1.mix.k.b", "l1.mix.v", "l1.mix.v.b", "l1.norm2", "l1.norm2b", "l0.mix.o.b", "l0.mlp.e0.gate", "l0.mlp.router.b"):
        assert n not in t, n
    assert t["bigram"].shape == (54, 40) and t["l0.mix.v.b"].shape == (24,) and t["l1.mix.o"].shape == (40, 72)


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][0].update(type="gla"), "mixer type"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "not divisible"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=10), "head size"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=3), "even"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"), "slow"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(factor=0), "positive"),
    (lambda c: c["layers"][0]["mixer"].update(scale=-1.0), "positive"),
    (lambda c: c["layers"][1]["mixer"].update(kv_from=1), "earlier"),
    (lambda c: c["layers"][1]["mixer"].update(kv_from=2), "earlier"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "of its own"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=0), "whose keys"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "not 'moe'"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "best of"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=4), "groups"),
    (lambda c: c["embedding"]["bigram"].pop("mul_cur"), "mul_cur"),
    (lambda c: c.pop("norm"), "lacks"),
])
def test_configurations_that_are_refused(change, text):
    from rust_inference_amd.config import config_from_dict
    from rust_inference_amd.errors import InferenceError
    cfg = copy.deepcopy(SMALL)
    change(cfg)
    with pytest.raises(InferenceError, match=text):
        config_from_dict(cfg)


def test_absent_keys_mean_not_there():
    from rust_inference_amd.config import config_from_dict
    from rust_inference_amd.parts.model import DecoderModel
    cfg = copy.deepcopy(SMALL)
    cfg.pop("embedding"), cfg.pop("logit_scale")
    m = cfg["layers"][0]["mixer"]
    m.pop("softcap"), m.pop("rot"), m.update(vdim=None)
    cfg["layers"][1]["mixer"].update(vdim=8, softcap=None)
    cfg["layers"][2]["mixer"]["rot"]["scaling"] = None
    arch, typed = config_from_dict(cfg)
    a, b, c = (l.mixer for l in typed.layers)
    assert typed.bigram is None and typed.logit_scale == 1.0 and a.softcap is None and a.rot_dims == 0 and a.vdim == 8 and b.softcap is None
    assert c.scaling is None and c.rot_dims == 16 and typed.layers[2].mlp.groups == 1
    spec = arch.build_spec(typed)
    assert spec.embedding.kind == "table" and spec.embedding_cache is None and "bigram" not in DecoderModel(spec).tensors()


def test_norm_gains_are_distances_from_one():
    from rust_inference_amd.parts import PartSpec, build_part
    from rust_inference_amd.weights.random_init import random_tensor
    part = build_part("norm", PartSpec("rmsnorm", {"dim": 4, "eps": 1e-5, "name": "n", "from_one": True, "scale": 2.0}))
    part.bind_plain({"n": torch.tensor([0.0, -1.0, 0.5, 0.25], dtype=torch.bfloat16)})
    assert part.gain_plain.tolist() == [2.0, 0.0, 3.0, 2.5]
    drawn = random_tensor(0, "n", build_part("norm", PartSpec("rmsnorm", {"dim": 4000, "eps": 1e-5, "name": "n", "from_one": True})).tensors()["n"]
                          .__class__((4000,), "offset"), torch.float32)
    assert abs(drawn.mean()) < 0.01 and abs(drawn.std() - 0.1) < 0.01


def test_the_plain_form_token_by_token_is_the_plain_form_at_once():
    w = random_weights(SMALL, 1)
    rng = np.random.default_rng(0)
    toks = [int(t) for t in rng.integers(0, SMALL["vocab"], 23)]
    whole = P.forward(SMALL, w, toks)
    state, rows = {}, []
    for cut in ([toks[:9]] + [[t] for t in toks[9:15]] + [toks[15:]]):
        rows.append(P.forward(SMALL, w, cut, state))
    assert np.abs(np.concatenate(rows) - whole).max() < 1e-9


def test_every_constant_and_tensor_moves_the_logits():
    w = random_weights(SMALL, 2)
    rng = np.random.default_rng(1)
    toks = [int(t) for t in rng.integers(0, SMALL["vocab"], 60)]
    base = P.forward(SMALL, w, toks)
    for name in w:
        other = dict(w)
        other[name] = w[name] + 0.3 * rng.standard_normal(w[name].shape)
        assert np.abs(P.forward(SMALL, other, toks) - base).max() > 1e-9, name
    for path, value in (("logit_scale", 1.1), ("norm.eps", 0.5), ("embedding.bigram.mul_prev", 3), ("embedding.bigram.mul_cur", 2),
                        ("layers.0.mixer.scale", 0.9), ("layers.0.mixer.softcap", 1.0), ("layers.1.mixer.softcap", 1.0), ("layers.1.mixer.scale", 0.1),
                        ("layers.0.mixer.rot.base", 3.0), ("layers.0.mixer.rot.dims", 8), ("layers.0.mixer.rot.scaling.factor", 2.0),
                        ("layers.0.mixer.rot.scaling.original", 200), ("layers.2.mixer.rot.scaling.fast", 2.0), ("layers.2.mixer.rot.scaling.slow", 0.2),
                        ("layers.0.mlp.router.top", 1), ("layers.0.mlp.router.groups.keep", 3)):
        cfg = copy.deepcopy(SMALL)
        at = cfg
        keys = path.split(".")
        for k in keys[:-1]:
            at = at[int(k)] if isinstance(at, list) else at[k]
        at[keys[-1]] = value
        assert np.abs(P.forward(cfg, w, toks) - base).max() > 1e-9, path


def test_mechanisms_by_hand():
    # the first token reads the table's last row, the next ones the pair's row
    assert P.bigram_rows([5, 6, 2], None, {"buckets": 10, "mul_prev": 3, "mul_cur": 7}) == [10, 7, 2]
    assert P.bigram_rows([6], 5, {"buckets": 10, "mul_prev": 3, "mul_cur": 7}) == [7]
    # halves turn together: (1, 0) in elements 0 and 2 at position 1 with a frequency of 1
    x = np.array([[[1.0, 0.0, 0.0, 0.0, 7.0]]])
    r = P.rotate_half(x, np.array([1.0]), {"dims": 4, "base": 10.0})
    assert np.allclose(r[0, 0], [math.cos(1.0), 0, math.sin(1.0), 0, 7.0])
    # the amplitude stretches what turns and nothing else
    r = P.rotate_half(x, np.array([0.0]), {"dims": 4, "base": 10.0, "scaling": {"factor": math.e, "original": 100, "fast": 8, "slow": 1}})
    assert np.allclose(r[0, 0], [1.1, 0, 0, 0, 7.0])
    # a token alone, score 0: half its value, the other half is the sink's; two equal keys of score 0: a third each
    v = np.array([[[4.0]], [[2.0]]])
    o = P.capped_attention(np.zeros((2, 1, 1)), np.zeros((2, 1, 1)), v, 0, 1.0, 30.0)
    assert np.allclose(o[:, 0, 0], [2.0, 2.0])
    # the cap comes after the scale
    o = P.capped_attention(np.full((1, 1, 1), 8.0), np.full((1, 1, 1), 1.0), v[:1], 0, 0.5, 2.0)
    s = 2.0 * math.tanh(2.0)
    assert np.allclose(o, 4.0 * math.exp(s) / (1 + math.exp(s)))
    # groups by the sum of their two best: {0.9, 0.1} against {0.6, 0.5}; the weights leave the correction out
    z = np.log(np.array([0.9, 0.1, 0.6, 0.5]) / (1 - np.array([0.9, 0.1, 0.6, 0.5])))
    ids, weights, _ = P.route(np.array([[1.0]]), {"router": z[:, None], "correction": np.zeros(4)}, "", {"top": 2, "groups": {"count": 2, "keep": 1}})
    assert ids.tolist() == [[2, 3]] and np.allclose(weights, [[0.6, 0.5]])
    ids, weights, _ = P.route(np.array([[1.0]]), {"router": z[:, None], "correction": np.array([-5.0, -5.0, -9.0, -9.0])}, "",
                              {"top": 2, "groups": {"count": 2, "keep": 1}})
    assert ids.tolist() == [[0, 1]] and np.allclose(weights, [[0.9, 0.1]])
    # squared ReLU
    assert P.expert(np.array([-1.0, 3.0]), {"e0.up": np.eye(2), "e0.down": np.eye(2)}, "", 0).tolist() == [0.0, 9.0]
