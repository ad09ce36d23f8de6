"""The Kisepel design without a GPU: configuration, registry, schedule and cache entries, tensor names, the cache's pages in
chunks, and the plain implementation (tests/plain/kisepel_plain.py) against itself and against examples worked out by hand."""
import copy
import math

import numpy as np
import pytest
import torch

from plain import kisepel_plain as P


def lin(heads, dim, vdim, decay=None):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                                           "decay": decay or [1.0 - 0.5 ** (i + 2) for i in range(heads)]}}


def ssm(heads, vdim, state, groups, conv, norm_groups):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                        "norm_groups": norm_groups}}


def att(heads, kv_heads, dim, vdim, scale, chunk, dims=None, base=1000.0, factor=2.0):
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk is not None:
        out["mask"] = {"size": chunk}
    if dims != 0:
        out["rot"] = {"dims": dims or dim, "base": base, "scaling": {"factor": factor}}
    return out


def rule(heads, kv_heads, dim, vdim, conv, rank=6):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "rank": rank}


def par(left, right):
    return {"type": "parallel", "mixer": {"left": left, "right": right}}


def moe(experts, top, ff, shared):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top},
            "shared": None if shared is None else {"ff": shared}}


def layer(mixer, mlp):
    return {**mixer, "mlp": mlp}


def model(layers, loop=None, vocab=97, width=40, eps=1e-5, embed=3.0, logits=0.4):
    cfg = {"architecture": "Kisepel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed},
           "logit_scale": logits, "layers": layers}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


SMALL = model([layer(ssm(4, 5, 7, 2, 3, 2), moe(4, 2, 12, 9)), layer(par(att(4, 2, 6, 10, 0.4, 5, 4), rule(4, 2, 8, 5, 4)), moe(3, 3, 8, None)),
               layer(lin(3, 6, 4), None), layer(ssm(2, 6, 3, 1, 1, 4), moe(1, 1, 8, 16))], (1, 3, 2))


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
    assert arch.name == "Kisepel" and cfg.embedding_scale == 3.0 and cfg.logit_scale == pytest.approx(0.4)
    assert config_from_dict(cfg.to_dict())[1] == cfg
    spec = arch.build_spec(cfg)
    assert [l.arrangement for l in spec.layers] == ["parallel_prenorm"] * 4
    # the looped layers run twice, each pass with entries of its own; the embedding is added before the second pass alone
    assert [(r.layer, r.cache, r.add_embedding) for r in spec.schedule] == [
        (0, (0, 1), False), (1, (2, 3, 4), False), (2, 5, False), (1, (6, 7, 8), True), (2, 9, False), (3, (10, 11), False)]
    m = DecoderModel(spec)
    needs = m.cache_needs()
    assert needs[0] == StateNeed((4, 7, 5)) and needs[1] == StateNeed((2, 4 * 5 + 2 * 2 * 7))
    assert needs[2] == needs[6] == KVNeed(2, 6, None, 10, None, 5)
    assert needs[3] == StateNeed((4, 8, 5)) and needs[4] == StateNeed((3, 2 * 2 * 8 + 4 * 5)) and needs[5] == StateNeed((3, 6, 4))
    names = set(m.tensors())
    for n in ("embed", "final.norm", "l0.norm1", "l0.mix.in", "l0.mix.conv", "l0.mix.conv.b", "l0.mix.dt_bias", "l0.mix.A_log", "l0.mix.D",
              "l0.mix.norm", "l0.mlp.table", "l0.mlp.e3.gate", "l0.mlp.e0.down", "l0.mlp.shared.up", "l1.mix.left.q", "l1.mix.left.q.norm",
              "l1.mix.left.k.norm", "l1.mix.left.o", "l1.mix.left.out", "l1.mix.right.out", "l1.mix.right.q.conv", "l1.mix.right.v.conv",
              "l1.mix.right.b", "l1.mix.right.a1", "l1.mix.right.a2", "l1.mix.right.g1", "l1.mix.right.g2", "l1.mix.right.dt_bias",
              "l1.mix.right.norm", "l2.mix.g", "l2.mix.norm", "l3.mix.o"):
        assert n in names, n
    for n in ("l0.mlp.router", "l0.mlp.correction", "l0.mlp.shared.sg", "l1.mlp.shared.gate", "l2.mlp.table", "l0.norm2", "l1.mix.right.g",
              "l1.mix.right.a"):
        assert n not in names, n
    shapes = {k: v.shape for k, v in m.tensors().items()}
    assert shapes["l0.mlp.table"] == (97, 2) and shapes["l1.mix.right.a2"] == (32, 6) and shapes["l1.mix.right.dt_bias"] == (32,)
    assert shapes["l1.mix.right.g2"] == (20, 6) and shapes["l1.mix.left.v"] == (20, 40) and shapes["l1.mix.left.o"] == (40, 40)


@pytest.mark.parametrize("change, text", [
    (lambda c: c["layers"][0].update(type="attention"), "mixer type"),
    (lambda c: c["layers"][1]["mixer"]["left"].update(kv_heads=3), "not divisible"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(kv_heads=3), "not divisible"),
    (lambda c: c["layers"][1]["mixer"]["right"].pop("conv"), "lacks conv"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"].update(dims=5), "even"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].update(factor=0.0), "positive"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(size=0), "below 1"),
    (lambda c: c["layers"][2]["mixer"].update(decay=[0.5, 0.5]), "one decay for each"),
    (lambda c: c["layers"][0]["mixer"].update(groups=3), "not divisible"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=5), "5 of 4 experts"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "not 'moe'"),
    (lambda c: c["loop"].update(stop=9), "does not lie inside"),
    (lambda c: c.pop("norm"), "lacks norm"),
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
    cfg = copy.deepcopy(SMALL)
    for key in ("loop", "embedding", "logit_scale"):
        cfg.pop(key)
    left, right = cfg["layers"][1]["mixer"]["left"], cfg["layers"][1]["mixer"]["right"]
    left.pop("mask"), left.pop("rot"), right.pop("rank"), cfg["layers"][0]["mlp"].pop("shared")
    typed = config_from_dict(cfg)[1]
    a = typed.layers[1].mixer.left
    assert a.chunk is None and a.rot_dims == 0 and typed.layers[1].mixer.right.rank is None and typed.layers[0].mlp.shared_ff is None
    assert typed.embedding_scale == 1.0 and typed.logit_scale == 1.0 and typed.order() == [(i, False) for i in range(4)]
    assert config_from_dict(typed.to_dict())[1] == typed
    left["rot"] = {"base": 50.0}
    a = config_from_dict(cfg)[1].layers[1].mixer.left
    assert (a.rot_dims, a.rot_base, a.rot_factor) == (6, 50.0, 1.0)


def test_a_loop_of_no_layers_and_one_that_runs_once():
    from rust_inference_amd.config import config_from_dict
    for loop, runs in (((2, 2, 3), [0, 1, 2, 3]), ((0, 4, 1), [0, 1, 2, 3]), ((0, 1, 3), [0, 0, 0, 1, 2, 3]), ((3, 4, 2), [0, 1, 2, 3, 3])):
        order = config_from_dict({**SMALL, "loop": dict(zip(("start", "stop", "times"), loop))})[1].order()
        assert [i for i, _ in order] == runs
        assert [at for at, (_, again) in enumerate(order) if again] == {(2, 2, 3): [], (0, 4, 1): [], (0, 1, 3): [1, 2], (3, 4, 2): [4]}[loop]


def test_a_random_table_has_different_entries_in_a_row():
    w = random_weights(SMALL, 3)
    for name, experts in (("l0.mlp.table", 4), ("l1.mlp.table", 3), ("l3.mlp.table", 1)):
        table = w[name]
        assert table.min() >= 0 and table.max() < experts and all(len(set(row)) == len(row) for row in table)
    assert len({tuple(r) for r in w["l0.mlp.table"]}) == 12          # every ordered pair of four appears


def test_a_table_that_names_experts_there_are_not_is_refused():
    from rust_inference_amd.errors import ConfigError
    from rust_inference_amd.parts import PartSpec, build_part

    class Place:
        device = "cpu"
        pack = staticmethod(lambda w, **_: w)
        place_matrix = staticmethod(lambda w: w)
    part = build_part("feed_forward", PartSpec("routed_experts", {"hidden": 8, "inter": 8, "experts": 2, "top": 1, "limit": None, "prefix": "m.",
                                                                 "scores": "table", "vocab": 3}))
    w = {n: torch.zeros(s.shape, dtype=torch.int32 if n.endswith("table") else torch.float32) for n, s in part.tensors().items()}
    part.bind(w, Place())
    for bad in (2, -1):
        w["m.table"] = torch.tensor([[0], [1], [bad]], dtype=torch.int32)
        with pytest.raises(ConfigError, match="m.table names experts"):
            part.bind(w, Place())


def test_pages_of_earlier_chunks_go_back():
    from rust_inference_amd.cache import Cache, KVNeed
    from rust_inference_amd.errors import CacheError
    c = Cache([KVNeed(1, 8, chunk=80), KVNeed(1, 8)], 2, 32 * 20, 400, dtype=torch.float32, allocate=False)
    slot = c.acquire()
    pool = c.groups[0].pool
    held = []
    for n in (50, 29, 1, 1, 15, 64, 1, 100):                # lengths 50, 79, 80, 81, 96, 160, 161, 261
        c.reserve([slot], [n])
        c.commit([slot], [n])
        held.append([p for p in range(pool.max_pages_per_slot) if pool.tables[slot][p] >= 0])
    # the next query at position L sees from 80 (L // 80) on; page 2 (64..95) holds the chunk's edge and stays while it is needed
    assert held == [[0, 1], [0, 1, 2], [2], [2], [2], [], [5], [7, 8]]
    assert c.groups[1].pool.tables[slot][:9].min() >= 0
    c.check_consistent()
    c.release(slot)
    assert c.free_pages() == [20, 20]
    with pytest.raises(CacheError, match="window"):
        Cache([KVNeed(1, 8, window=8, chunk=8)], 1, 64, 64, dtype=torch.float32, allocate=False)


def test_attention_parts_that_are_refused():
    from rust_inference_amd.errors import ConfigError
    from rust_inference_amd.parts import PartSpec, build_part
    base = {"hidden": 32, "heads": 2, "kv_heads": 1, "head_dim": 8, "prefix": "a.", "chunk": 16}
    build_part("mixer", PartSpec("attention", base))
    for change, text in (({"window": 5}, "no window beside"), ({"chunk": 0}, "positive number"), ({"gate": "sigmoid"}, "takes no unit norm"),
                         ({"qk_norm": "unit"}, "takes no unit norm")):
        with pytest.raises(ConfigError, match=text):
            build_part("mixer", PartSpec("attention", {**base, **change}))
    with pytest.raises(ConfigError, match="neither 'head' nor 'channel'"):
        build_part("mixer", PartSpec("delta", {"hidden": 32, "heads": 2, "kv_heads": 1, "dim": 8, "vdim": 8, "taps": 2, "prefix": "d.", "decay": "row"}))


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
        if name.endswith("table"):
            if name != "l0.mlp.table":                    # (all experts are chosen there)
                continue
            other[name] = (w[name] + 1) % 4
        else:
            other[name] = w[name] + 0.3 * rng.standard_normal(w[name].shape)
        assert np.abs(P.forward(SMALL, other, toks) - base).max() > 1e-9, name
    for path, value in (("embedding.scale", 1.0), ("logit_scale", 1.0), ("norm.eps", 0.5), ("loop.times", 3), ("loop.start", 0),
                        ("layers.0.mixer.norm_groups", 1), ("layers.0.mlp.router.top", 1), ("layers.1.mixer.left.mask.size", 6),
                        ("layers.1.mixer.left.scale", 1.5), ("layers.1.mixer.left.rot.dims", 6), ("layers.1.mixer.left.rot.base", 3.0),
                        ("layers.1.mixer.left.rot.scaling.factor", 1.0), ("layers.2.mixer.decay.1", 0.1)):
        cfg = copy.deepcopy(SMALL)
        at = cfg
        keys = path.split(".")
        for k in keys[:-1]:
            at = at[int(k)] if isinstance(at, list) else at[k]
        at[int(keys[-1]) if isinstance(at, list) else keys[-1]] = value
        assert np.abs(P.forward(cfg, w, toks) - base).max() > 1e-9, path


def test_mechanisms_by_hand():
    # chunks are counted from position 0: with a size of 2 position 2 sees itself alone, position 3 two keys
    k = np.zeros((4, 1, 1))
    v = np.arange(4.0).reshape(4, 1, 1)
    assert np.allclose(P.attention_core(np.ones((4, 1, 1)), k, v, 0, 2, 1.0)[:, 0, 0], [0.0, 0.5, 2.0, 2.5])
    # halves turn: (1, 0, 7) with two elements turning at frequency 1 / 2
    r = P.rotate_halves(np.array([[[1.0, 0.0, 7.0]]]), np.array([1.0]), 2, 10.0, 2.0)
    assert np.allclose(r[0, 0], [math.cos(0.5), math.sin(0.5), 7.0])
    # the norm's weight is stored around zero
    assert np.allclose(P.norm_from_one(np.array([[3.0, 4.0]]), np.array([0.0, 1.0]), 0.0), np.array([[3.0, 8.0]]) / math.sqrt(12.5))
    # the delta rule: the state forgets first, a key channel at a time, then writes what is missing, then reads
    s = np.array([[[4.0], [8.0]]])
    o = P.delta_walk(np.array([[[1.0, 1.0]]]), np.array([[[1.0, 0.0]]]), np.array([[[5.0]]]), np.array([[0.5]]), np.array([[[0.5, 0.25]]]), s)
    assert np.allclose(s[0, :, 0], [2.0 + 0.5 * (5.0 - 2.0), 2.0]) and np.allclose(o, 5.5)
    # two key heads for four value heads: value heads 2 and 3 read the second
    o = P.delta_walk(np.array([[[1.0], [10.0]]]), np.ones((1, 2, 1)), np.ones((1, 4, 1)), np.ones((1, 4)), np.ones((1, 4, 1)), np.zeros((4, 1, 1)))
    assert np.allclose(o[0, :, 0], [1, 1, 10, 10])
    # a fixed decay: the state after two tokens with k = v = 1 before silu
    m = {"heads": 1, "dim": 1, "vdim": 1, "decay": [0.5]}
    w = {"q": np.eye(1), "k": np.eye(1), "v": np.eye(1), "g": np.zeros((1, 1)), "norm": np.ones(1), "o": np.eye(1)}
    st = {}
    out = P.lightning_mixer(np.ones((2, 1)), w, "", m, 0.0, st)
    a = float(P.silu(1.0))
    assert np.allclose(st["S"], 1.5 * a * a) and np.allclose(out, 0.5)         # the norm of one number, times sigmoid(0)
    # experts by the token's row, equal weights, the shared one added whole
    w = {"table": np.array([[1], [0]]), "e0.gate": np.array([[1.0]]), "e0.up": np.array([[1.0]]), "e0.down": np.array([[1.0]]),
         "e1.gate": np.array([[1.0]]), "e1.up": np.array([[3.0]]), "e1.down": np.array([[1.0]]),
         "shared.gate": np.array([[1.0]]), "shared.up": np.array([[10.0]]), "shared.down": np.array([[1.0]])}
    got = P.table_experts(np.ones((2, 1)), w, "", {"router": {"experts": 2, "top": 1}, "shared": {"ff": 1}}, [0, 1])
    assert np.allclose(got[:, 0], [a * 13, a * 11])
