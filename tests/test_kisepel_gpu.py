"""The Kisepel design through the engine, against the plain implementation (tests/plain/kisepel_plain.py), in
float32 and in bfloat16, for configurations made here with random weights: whole prompts; the last tokens one by
one; prompts in portions down to two tokens; batches of unequal requests one after another, so that slots, pages
and states are used again; long decoding over page borders and from chunk to chunk; keys just inside and just outside
a chunk, made to stand out; a far key among hundreds; states that must survive every cut; the residual after every
layer; the ways through the experts; greedy generation through the library's own entry point with and without graphs;
the trace program and the command line."""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import trace_plans as plans
from helpers import assert_logits_close, read_model_f64, rel_to_max
from plain import kisepel_plain as P
from test_kisepel import att, layer, lin, model, moe, par, rule, ssm

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}

# Every mixer, twice, in another order than usual; heads that are no power of two; three query heads a key head; value heads
# larger and smaller than key heads; chunks shorter than a page and longer than two; three delta heads a key head; convolutions of
# four taps and of one; part of a head turned, and none; one expert of five and all of three; layers without feed-forward or
# shared expert; a loop of three layers that runs three times.
K_A = model([layer(lin(3, 20, 12), moe(5, 1, 24, 40)), layer(par(att(6, 2, 24, 40, 0.2, 19, 16), rule(6, 2, 12, 20, 4)), moe(3, 3, 16, None)),
             layer(ssm(6, 8, 12, 3, 4, 3), None), layer(par(att(4, 4, 40, 8, 0.3, 75, 0), rule(2, 2, 24, 8, 1, rank=9)), None),
             layer(ssm(2, 40, 24, 1, 1, 1), moe(4, 2, 56, 24)), layer(lin(1, 8, 30, [0.9]), moe(2, 2, 8, 8))], (1, 4, 3), vocab=211, width=96, embed=8.0, logits=0.2)
# Sizes the matrix cores like: heads of 64 and 128 elements, a width of 256, chunks of exactly two pages and of three, one key head
# for eight query heads, whole heads turned.
K_B = model([layer(par(att(8, 1, 64, 64, 0.11, 64), rule(4, 2, 64, 64, 4, rank=16)), moe(8, 2, 64, 128)),
             layer(ssm(8, 64, 64, 2, 2, 4), moe(16, 4, 32, 64)),
             layer(par(att(4, 2, 128, 128, 0.09, 96, factor=5.0), rule(2, 1, 128, 64, 3, rank=8)), moe(8, 1, 64, 96)),
             layer(lin(4, 64, 64), None)], (0, 2, 2), vocab=300, width=256, eps=1e-6, embed=9.0, logits=0.05)
# A chunk of exactly one page and one of a single token; a state of one row; one expert; a convolution of five taps; no loop; the
# embedding and the logits as they are.
K_C = model([layer(ssm(3, 16, 1, 3, 5, 3), moe(1, 1, 40, 24)), layer(par(att(4, 2, 32, 32, 0.15, 32), rule(4, 4, 16, 16, 2)), moe(6, 4, 16, 8)),
             layer(par(att(2, 1, 8, 8, 0.5, 1, 2), rule(1, 1, 40, 24, 3)), moe(4, 1, 24, 56)), layer(lin(2, 16, 16), moe(3, 2, 16, 16))],
            vocab=157, width=64, embed=1.0, logits=1.0)
# Sizes that 16-byte loads do not divide: a width of 100, heads of 12, 20 and 7, feed-forwards of 52 and 28, chunks over more than a
# page beside one over everything a test sends, and no chunks at all.
K_D = model([layer(par(att(6, 3, 20, 12, 0.2, 41, 6), rule(3, 3, 7, 12, 4, rank=5)), moe(5, 2, 28, 52)),
             layer(par(att(5, 5, 12, 20, 0.3, 500, 12), rule(5, 1, 20, 7, 3, rank=3)), moe(4, 3, 20, 12)),
             layer(ssm(6, 12, 20, 3, 4, 3), moe(5, 5, 12, 28)), layer(par(att(2, 1, 12, 12, 0.3, None, 8), rule(2, 2, 12, 12, 2, rank=4)), None),
             layer(lin(5, 12, 9), moe(3, 1, 12, None))], (4, 5, 4), vocab=333, width=100, embed=5.0, logits=0.3)
CONFIGS = {"A": K_A, "B": K_B, "C": K_C, "D": K_D}


def sharpen(folder):
    """Random weights as the library draws them, with what small or level values would switch off made to count: the decays and
    their biases, the step sizes, the skip, the convolutions."""
    from safetensors.torch import load_file, save_file
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    g = torch.Generator().manual_seed(len(w))
    draw = lambda like, std, mean=0.0: (mean + std * torch.randn(like.shape, generator=g)).to(like.dtype)
    for name in w:
        if name.endswith((".A_log", ".dt_bias")):
            w[name] = draw(w[name], 0.7, -1.0)
        elif name.endswith(".conv.b"):
            w[name] = draw(w[name], 0.2)
        elif name.endswith(".conv"):
            w[name] = draw(w[name], 0.5)
        elif name.endswith((".b", ".a1", ".g1")):
            w[name] = (w[name].float() * 1.5).to(w[name].dtype)
        elif name.endswith((".a2", ".g2")):
            w[name] = (w[name].float() * 4.0).to(w[name].dtype)
    save_file(w, path)
    return folder


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    from rust_inference_amd.weights import write_random_model
    base = tmp_path_factory.mktemp("kisepel")
    return {name: sharpen(write_random_model(str(base / name), cfg, seed, torch.bfloat16, matrix_std=0.12, gain_std=0.1))
            for seed, (name, cfg) in enumerate(CONFIGS.items())}


_models, _plain, _read = {}, {}, {}


def loaded(folders, name, dtype_name, **kw):
    from rust_inference_amd.parts import load_model
    key = (name, dtype_name, *kw.items())
    if key not in _models:
        _models[key] = load_model(folders[name], DTYPES[dtype_name], **kw)
    return _models[key]


def plain_logits(folder, tokens):
    key = (folder, tuple(tokens))
    if key not in _plain:
        if folder not in _read:
            _read[folder] = read_model_f64(folder)
        _plain[key] = P.forward(*_read[folder], list(tokens))
    return _plain[key]


def requests_for(cfg, prefix, lengths, seed):
    rng = np.random.default_rng(seed)
    return {f"{prefix}{i}": [int(t) for t in rng.integers(0, cfg["vocab"], n)] for i, n in enumerate(lengths)}


def replay(model_, steps):
    from rust_inference_amd.engine.replay import Replayer, engine_for_trace
    engine = engine_for_trace(model_, plans.max_live_tokens(steps))
    player = Replayer(engine)
    outs = {}
    for s in steps:
        logits = player.feed(s)
        if logits is not None:
            outs[s["step"]] = logits.cpu().numpy()
    engine.cache.check_consistent()
    assert engine.cache.slots.free_count == engine.cache.num_slots
    assert all(f == g.pool.num_pages for f, g in zip(engine.cache.free_pages(), engine.cache.groups))
    return plans.collect(steps, lambda i: outs[i], model_.spec.vocab_size)


def against_plain(folder, got, requests, dtype_name, what, bound=None):
    for rid, toks in requests.items():
        want = plain_logits(folder, toks)
        if dtype_name == "float32":
            assert_logits_close(got[rid], want, dtype_name, f"{what}, request {rid}")
            continue
        # the norms (over heads, over parts of a mixer's result) lift a row whose values happen to be small, and the rounding of its
        # 16 bits with them: few positions may lie over the bound, none far over it
        bound = bound or 3e-2
        errs = np.abs(np.asarray(got[rid], dtype=np.float64) - want).max(-1) / np.abs(want).max()
        over = int((errs > bound).sum())
        assert over <= max(1, 0.04 * len(errs)) and errs.max() <= 3 * bound, (
            f"{what}, request {rid}: {over} of {len(errs)} positions differ by more than {bound:.0e} (bfloat16), the worst by {errs.max():.2e}")


def in_portions(requests, sizes):
    """Each request alone, its prompt in portions of the given sizes in turn (the last portion takes what is left)."""
    steps = []
    for rid, toks in requests.items():
        at, i = 0, 0
        while at < len(toks):
            n = min(sizes[i % len(sizes)], len(toks) - at)
            steps.append({"step": len(steps), "entries": [{"id": rid, "tokens": toks[at:at + n], "want": list(range(n))}],
                          "end": [rid] if at + n == len(toks) else []})
            at, i = at + n, i + 1
    return steps


LENGTHS = {"A": [70, 3, 131], "B": [45, 1, 200], "C": [97, 33, 64], "D": [150, 2, 61]}


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompts(folders, name, dtype_name):
    reqs = requests_for(CONFIGS[name], name, LENGTHS[name], 1)
    got = replay(loaded(folders, name, dtype_name), plans.whole(reqs))
    against_plain(folders[name], got, reqs, dtype_name, "whole")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_last_tokens_one_by_one_and_portions(folders, name, dtype_name):
    reqs = requests_for(CONFIGS[name], name, [n + 40 for n in LENGTHS[name]], 2)
    model_ = loaded(folders, name, dtype_name)
    whole = replay(model_, plans.whole(reqs))
    for what, steps in (("last 32 one by one", plans.tail_one_by_one(reqs, 32)),
                        ("portions of 2, 31 and 32", in_portions(reqs, [2, 31, 32])),
                        ("portions of 64, 1 and 7", in_portions(reqs, [64, 1, 7])), ("portions of two", in_portions(reqs, [2]))):
        got = replay(model_, steps)
        against_plain(folders[name], got, reqs, dtype_name, what)
        for rid in reqs:
            err = rel_to_max(got[rid], whole[rid])
            assert err <= (2e-5 if dtype_name == "float32" else 2e-2), f"{rid}, {what}: {err:.2e} against the whole prompt"


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_unequal_batches_one_after_another(folders, name, dtype_name):
    rng = np.random.default_rng(8)
    batches, reqs = [], {}
    for b in range(3):                                       # three batches on one cache: slots, pages and states come back
        batch = {}
        for i in rng.permutation(len(LENGTHS[name])):
            p = LENGTHS[name][i]
            toks = [int(t) for t in rng.integers(0, CONFIGS[name]["vocab"], p + int(rng.integers(0, 14)))]
            batch[f"{name}{b}_{i}"] = (toks, p)
            reqs[f"{name}{b}_{i}"] = toks
        batches.append(batch)
    model_ = loaded(folders, name, dtype_name)
    got = replay(model_, plans.unequal_batches(batches))
    against_plain(folders[name], got, reqs, dtype_name, "unequal batches")
    alone = replay(model_, plans.whole(reqs))
    for rid in reqs:
        err = rel_to_max(got[rid], alone[rid])
        assert err <= (2e-5 if dtype_name == "float32" else 2e-2), f"{rid}: {err:.2e} in a batch against itself alone"


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_long_decoding_from_the_first_tokens(folders, name, dtype_name):
    """Three tokens of prompt, then 200 one by one: over page borders and from chunk to chunk, the pages of earlier chunks
    given back."""
    reqs = requests_for(CONFIGS[name], name, [203], 3)
    got = replay(loaded(folders, name, dtype_name), plans.tail_one_by_one(reqs, 200))
    against_plain(folders[name], got, reqs, dtype_name, "long decoding")


@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_residual_after_every_layer(folders, name):
    """In float32: what the stream holds after every run of a layer, branches that wait included."""
    from rust_inference_amd.engine.replay import Replayer, engine_for_trace
    toks = requests_for(CONFIGS[name], name, [37], 11)[f"{name}0"]
    want = []
    P.forward(*read_model_f64(folders[name]), toks, layers=want)
    model_ = loaded(folders, name, "float32")
    seen, kept = [], {}
    for l in set(model_.layers):
        kept[l] = l.forward

        def watch(stream, *a, _f=l.forward, **k):
            _f(stream, *a, **k)
            x = stream.sum.clone()
            waiting = stream.pending if isinstance(stream.pending, list) else [] if stream.pending is None else [stream.pending]
            for y in waiting:
                x += y.to(torch.float32) if y.dim() == 2 else y.sum(0)
            seen.append(x.cpu().numpy())
        l.forward = watch
    try:
        engine = engine_for_trace(model_, 64)
        Replayer(engine).feed({"step": 0, "entries": [{"id": "a", "tokens": toks, "want": [len(toks) - 1]}], "end": ["a"]})
    finally:
        for l in kept:
            del l.forward
    assert len(seen) == len(want)
    for i, (a, b) in enumerate(zip(seen, want)):
        assert rel_to_max(a, b) < 1e-5, f"layer run {i}"


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_the_ways_through_the_experts_agree(folders, dtype_name):
    """A prompt of 330 tokens (its tokens sorted by expert), the same in portions of 100 (all experts for all tokens) and
    its last tokens one by one, with a second request beside it."""
    reqs = requests_for(K_B, "B", [330, 290], 9)
    model_ = loaded(folders, "B", dtype_name)
    for what, steps in (("whole", plans.whole(reqs)), ("portions of 100", in_portions(reqs, [100])),
                        ("a batch, then one by one", plans.unequal_batches([{rid: (toks, len(toks) - 6) for rid, toks in reqs.items()}]))):
        against_plain(folders["B"], replay(model_, steps), reqs, dtype_name, what)


@pytest.mark.parametrize("name", ["B", "C"])
def test_the_batch_invariant_mode_gives_the_same_bits_in_every_cut(folders, name):
    reqs = requests_for(CONFIGS[name], "i", [70, 9, 101], 12)
    model_ = loaded(folders, name, "bfloat16", invariant=True)
    whole = replay(model_, plans.whole(reqs))
    against_plain(folders[name], whole, reqs, "bfloat16", "whole")
    for what, steps in (("one by one", plans.tail_one_by_one(reqs, 30)), ("portions", in_portions(reqs, [33, 2, 40])),
                        ("a batch", plans.unequal_batches([{rid: (toks, max(1, len(toks) - 5)) for rid, toks in reqs.items()}]))):
        got = replay(model_, steps)
        assert all(np.array_equal(got[rid], whole[rid]) for rid in reqs), what


# ---------------------------------------------------------------- a chunk's edge and a far key, made to show
@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim, vdim", [(16, 16), (64, 64), (24, 40)])
@pytest.mark.parametrize("chunk", [37, 32, 33, 64, 65, 1, 2, 31, 100])
def test_keys_just_inside_and_just_outside_the_chunk(tmp_path_factory, dim, vdim, chunk, dtype_name):
    """One layer whose attention has a scale close to nothing, so that every visible key weighs the same whatever it holds, and
    whose other mixer hardly counts: a key on the wrong side of a chunk's edge changes the sum as much as its neighbour does."""
    from rust_inference_amd.parts import load_model
    from rust_inference_amd.weights import write_random_model
    cfg = model([layer(par(att(2, 1, dim, vdim, 0.002, chunk), rule(1, 1, 8, 8, 2)), None)], vocab=64, width=32, embed=0.3, logits=1.0)
    folder = write_random_model(str(tmp_path_factory.mktemp(f"edge{dim}_{chunk}")), cfg, chunk, torch.bfloat16, matrix_std=0.3)
    from safetensors.torch import load_file, save_file
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    w["l0.mix.right.out"] = w["l0.mix.right.out"] * 0.02
    save_file(w, path)
    rng = np.random.default_rng(chunk)
    toks = [int(t) for t in rng.integers(0, cfg["vocab"], 4 * 32 + 9)]
    want = plain_logits(folder, toks)
    # the plain form itself must tell the edge: chunks one longer, and chunks counted from position 1, change the logits
    least = 2e-2 if dtype_name == "bfloat16" else 1e-3
    other = copy.deepcopy(cfg)
    other["layers"][0]["mixer"]["left"]["mask"]["size"] = chunk + 1
    moved = rel_to_max(P.forward(other, read_model_f64(folder)[1], toks)[chunk:], want[chunk:])
    assert moved > least, f"one more token in a chunk moves the logits by {moved:.1e} only"
    model_ = load_model(folder, DTYPES[dtype_name])
    reqs = {"e": toks}
    for what, steps in (("whole", plans.whole(reqs)), ("one by one", plans.tail_one_by_one(reqs, len(toks) - 1)),
                        ("portions", in_portions(reqs, [chunk + 1, 2, 31])), ("the last 40 one by one", plans.tail_one_by_one(reqs, 40))):
        got = replay(model_, steps)
        assert_logits_close(got["e"], want, dtype_name, f"chunk {chunk}, {what}")
        assert rel_to_max(got["e"], want) < least * 0.75, f"chunk {chunk}, {what}"


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_a_far_key_among_hundreds(tmp_path_factory, dtype_name):
    """Chunks of 730 and a large score scale, so that one key can take the softmax: the last logits must see a token almost 700
    positions back at a page's border; a token of the chunk before must not reach them through the attention."""
    from rust_inference_amd.parts import load_model
    from rust_inference_amd.weights import write_random_model
    cfg = model([layer(par(att(2, 1, 16, 16, 0.9, 730, 4, 10000.0, 8.0), rule(1, 1, 8, 8, 2)), None)], vocab=80, width=32, embed=0.3, logits=1.0)
    folder = write_random_model(str(tmp_path_factory.mktemp("far")), cfg, 3, torch.bfloat16, matrix_std=0.3)
    from safetensors.torch import load_file, save_file
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    w["l0.mix.right.out"] = w["l0.mix.right.out"] * 0.02
    save_file(w, path)
    rng = np.random.default_rng(5)
    toks = [int(t) for t in rng.integers(0, 40, 1450)]
    toks[768] = 77                                             # a token seen nowhere else, at a page's first place
    want = plain_logits(folder, toks)
    cfg_, w_ = read_model_f64(folder)
    other = list(toks)
    other[768] = 78
    assert rel_to_max(P.forward(cfg_, w_, other)[-30:], want[-30:]) > 1e-2, "the far token does not reach the last logits"
    model_ = load_model(folder, DTYPES[dtype_name])
    reqs = {"f": toks}
    for what, steps in (("whole", plans.whole(reqs)), ("the last 40 one by one", plans.tail_one_by_one(reqs, 40)),
                        ("portions", in_portions(reqs, [300, 2, 431]))):
        got = replay(model_, steps)
        assert_logits_close(got["f"], want, dtype_name, f"far key, {what}")


@pytest.mark.parametrize("cuts", [[300], [1] * 40 + [260], [33, 2, 265], [299, 1]])
@pytest.mark.parametrize("kind", ["delta", "lightning", "mamba2"])
def test_states_that_hardly_decay_survive_every_cut(tmp_path_factory, kind, cuts):
    """A recurrence whose decays are close to one keeps the first token for hundreds of steps, in a loop, beside an attention that
    sees at most 20 tokens: a state or a convolution's tail that is lost, reset or carried to the wrong slot or pass at any cut
    changes the last logits."""
    from rust_inference_amd.parts import load_model
    from rust_inference_amd.weights import write_random_model
    mixer = {"delta": par(att(2, 1, 16, 16, 0.2, 20), rule(2, 1, 12, 12, 4)), "lightning": lin(2, 12, 12, [0.9999, 0.999]),
             "mamba2": ssm(2, 12, 8, 1, 4, 1)}[kind]
    cfg = model([layer(mixer, moe(2, 1, 16, 16))], (0, 1, 2), vocab=90, width=48, embed=0.5, logits=1.0)
    folder = write_random_model(str(tmp_path_factory.mktemp("no_decay")), cfg, 5, torch.bfloat16, matrix_std=0.12, gain_std=0.1)
    from safetensors.torch import load_file, save_file
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    for name in w:
        if name.endswith(".A_log"):
            w[name] = torch.full_like(w[name], -7.0)
        if name.endswith("right.b"):
            w[name] = w[name] * 0.1 - 0.02                     # small writes: what the first token left is not overwritten
    save_file(w, path)
    toks = requests_for(cfg, "s", [300], 4)["s0"]
    want = plain_logits(folder, toks)
    other = plain_logits(folder, [toks[0] ^ 1] + toks[1:])
    assert rel_to_max(other[-1], want[-1]) > 2e-4, "the first token does not reach the last logits: the test shows nothing"
    model_ = load_model(folder, torch.float32)
    steps, at = [], 0
    for n in cuts:
        # another request comes and goes between the portions, on the slot next to this one
        steps.append({"step": len(steps), "entries": [{"id": "x", "tokens": toks[at:at + n], "want": list(range(n))}], "end": []})
        steps.append({"step": len(steps), "entries": [{"id": f"o{at}", "tokens": toks[:5], "want": []}], "end": [f"o{at}"]})
        at += n
    steps[-1]["end"].append("x")
    got = replay(model_, steps)
    err = rel_to_max(got["x"], want)
    assert err < 2e-5, f"cuts {cuts[:3]}: {err:.1e}"


@pytest.mark.parametrize("dtype_name, use_graphs", [("float32", False), ("float32", True), ("bfloat16", True)])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_greedy_generation_through_the_entry_point(folders, name, dtype_name, use_graphs):
    from rust_inference_amd import Model
    prompts = list(requests_for(CONFIGS[name], name, [33, 2, 40, 7], 5).values())
    steps = 12
    cfg, w = read_model_f64(folders[name])
    model_ = Model.load(folders[name], dtype=dtype_name, max_batch=3, max_seq_len=128, use_graphs=use_graphs, graph_after=0)
    got = model_.generate(prompts, max_new_tokens=steps).tokens          # four prompts on three slots: a second batch
    for g, p in zip(got, prompts):
        state, toks = {}, list(p)
        rows = P.forward(cfg, w, toks, state)
        for i, a in enumerate(g):
            row = rows[-1]
            b = int(np.argmax(row))
            if a != b:
                top = np.sort(row)
                assert top[-1] - top[-2] < (1e-4 if dtype_name == "float32" else 0.08) * np.abs(row).max(), f"token {i} is {a}, plain says {b}"
                break                                                   # from here on the two follow different texts
            rows = P.forward(cfg, w, [a], state)
    model_.cache.check_consistent()


def test_a_graph_replayed_many_times_is_the_eager_step(folders):
    """Greedy decoding of 150 tokens past pages and chunks, with graphs and without: the same tokens and states."""
    from rust_inference_amd import Model
    prompts = list(requests_for(K_B, "g", [50, 20], 15).values())
    got = [Model.load(folders["B"], dtype="float32", max_batch=2, max_seq_len=256, use_graphs=g, graph_after=0).generate(prompts, max_new_tokens=150).tokens
           for g in (False, True)]
    assert got[0] == got[1] and all(len(x) == 150 for x in got[0])


def test_the_trace_program(folders, tmp_path):
    reqs = requests_for(K_A, "t", [40, 9], 6)
    steps = plans.unequal_batches([{rid: (toks, len(toks) - 4) for rid, toks in reqs.items()}])
    out = str(tmp_path / "out")
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders["A"], "--dtype", "float32",
                           "--out", out, "--max-tokens", str(plans.max_live_tokens(steps))],
                          input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    got = plans.collect(steps, lambda i: np.fromfile(os.path.join(out, f"{i}.f32"), dtype="<f4"), K_A["vocab"])
    against_plain(folders["A"], got, reqs, "float32", "trace program")


def drawn_config(seed):
    """A configuration drawn at random: sizes, head counts, number and order of layers, chunks, constants, loops, with
    feed-forwards and without."""
    rng = np.random.default_rng(9000 + seed)
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers = []
    for _ in range(int(rng.integers(1, 5))):
        experts = pick([1, 2, 4, 7, 16])
        mlp = pick([None, moe(experts, int(rng.integers(1, experts + 1)), pick([8, 24, 56]), pick([None, 8, 40, 96])),
                    moe(experts, min(experts, 2), 16, 24)])
        kind = pick(["lin", "par", "ssm"])
        if kind == "lin":
            heads = pick([1, 2, 3, 5])
            mixer = lin(heads, pick([4, 8, 20, 32, 64, 100]), pick([8, 12, 32, 64, 128]), [float(d) for d in rng.uniform(0.3, 0.9999, heads)])
        elif kind == "par":
            kv, dk = pick([1, 2, 3, 4]), pick([8, 16, 24, 32, 48, 64, 96, 128])
            g, dd = pick([1, 2, 3]), pick([4, 8, 16, 24, 32, 64, 100])
            mixer = par(att(kv * pick([1, 2, 4]), kv, dk, pick([dk, dk, 8, 40, 64]), float(rng.uniform(0.05, 0.4)), pick([None, 1, 7, 31, 32, 33, 50, 100, 150]),
                            pick([0, 2, dk // 2 // 2 * 2, dk]), float(pick([50.0, 10000.0, 1000000.0])), float(pick([1.0, 2.0, 8.0, 0.5]))),
                        rule(g * pick([1, 2, 3]), g, dd, pick([4, 8, 20, 32, 64]), pick([1, 2, 3, 4, 6]), rank=pick([1, 4, 13, 24])))
        else:
            groups = pick([1, 2, 3])
            heads, vdim = groups * pick([1, 2, 3]), pick([8, 16, 32, 64])
            mixer = ssm(heads, vdim, pick([1, 8, 16, 32, 64, 100]), groups, pick([1, 2, 3, 4, 7]),
                        pick([g for g in (1, 2, heads, 2 * heads) if (heads * vdim) % g == 0]))
        layers.append(layer(mixer, mlp))
    start = int(rng.integers(0, len(layers) + 1))
    loop = pick([None, (start, int(rng.integers(start, len(layers) + 1)), pick([1, 2, 3]))])
    return model(layers, loop, vocab=int(rng.integers(50, 400)), width=pick([48, 80, 136, 192]), eps=pick([1e-5, 1e-6, 1e-3]),
                 embed=float(rng.uniform(0.3, 12.0)), logits=float(rng.uniform(0.05, 1.5)))


@pytest.mark.parametrize("seed", range(14))
def test_configurations_drawn_at_random(tmp_path, seed):
    from rust_inference_amd.parts import load_model
    from rust_inference_amd.weights import write_random_model
    cfg = drawn_config(seed)
    folder = sharpen(write_random_model(str(tmp_path / "m"), cfg, seed, torch.bfloat16, matrix_std=0.12, gain_std=0.1))
    rng = np.random.default_rng(seed)
    reqs = {f"r{i}": [int(t) for t in rng.integers(0, cfg["vocab"], n)] for i, n in enumerate((150, 37, 1, 66))}
    batch = {rid: (toks, max(1, len(toks) - 9)) for rid, toks in reqs.items()}
    for dtype_name in ("float32", "bfloat16"):
        model_ = load_model(folder, DTYPES[dtype_name])
        for what, steps in (("whole", plans.whole(reqs)), ("last 32 one by one", plans.tail_one_by_one(reqs, 32)),
                            ("a batch", plans.unequal_batches([batch])), ("portions", in_portions(reqs, [33, 2, 64]))):
            against_plain(folder, replay(model_, steps), reqs, dtype_name, f"configuration {seed}, {what}", 5e-2)


def test_the_command_line_generates_what_the_plain_implementation_does(folders):
    """bin/runner on a Kisepel folder, prompts as token ids: greedy in float32, sections timed, and a seeded temperature
    run that gives the same tokens twice."""
    cfg, w = read_model_f64(folders["A"])
    prompts = list(requests_for(K_A, "c", [9, 14], 8).values())
    want = []
    for p in prompts:
        toks = list(p)
        for _ in range(6):
            toks.append(int(np.argmax(P.forward(cfg, w, toks)[-1])))
        want.append(toks[len(p):])
    base = [sys.executable, os.path.join(ROOT, "bin", "runner"), folders["A"], "--dtype", "float32", "-n", "6"]
    two = subprocess.run(base + ["--prompt-ids", ",".join(map(str, prompts[0])), "--prompt-ids", ",".join(map(str, prompts[1])),
                                 "--profile"], capture_output=True, text=True, timeout=300)
    assert two.returncode == 0, two.stderr[-2000:]
    assert [[int(t) for t in ln.split()] for ln in two.stdout.strip().splitlines()] == want
    assert "section " in two.stderr and "attention" in two.stderr
    drawn = [subprocess.run(base + ["-p", " ".join(map(str, prompts[0])), "--temperature", "0.9", "--top-k", "20", "--seed", "5"],
                            capture_output=True, text=True, timeout=300) for _ in range(2)]
    assert drawn[0].returncode == 0, drawn[0].stderr[-2000:]
    assert drawn[0].stdout == drawn[1].stdout and len(drawn[0].stdout.split()) == 6
