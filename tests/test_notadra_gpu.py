"""The Notadra design through the engine, against the plain implementation (tests/plain/notadra_plain.py), in float32
and in bfloat16, for configurations made here with random weights: whole prompts; the last tokens one by one; prompts in
portions down to two tokens; batches of unequal requests one after another, so that slots, pages and kept tokens are used
again; long decoding over page borders; a far key among hundreds and the sink, made to stand out; layers that read another
layer's keys; the token kept for the pairs through every cut; greedy generation through the library's own entry point with
and without graphs; the trace program and the command line."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import trace_plans as plans
from helpers import assert_logits_close, read_model_f64, rel_to_max
from plain import notadra_plain as P
from test_dagezen_gpu import close_enough, in_portions, replay, requests_for
from test_notadra import attention, layer, model, moe

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}

# Three query heads a key head, value heads larger than key heads, a rotation over part of a head; a layer that reads the
# layer before the last one's keys with more query heads and another cap, then one that reads the first's; a layer without
# a feed-forward; groups of three experts of which one group stays, and no groups.
N_A = model([layer(attention(6, 2, 24, 40, 0.3, rot_dims=8, base=300.0), moe(9, 2, 24, (3, 1))),
             layer(attention(3, 3, 16, 8, 0.35, cap=5.0, base=50.0, stretch=(2.0, 64, 8.0, 0.5)), None),
             layer(attention(12, 2, 24, 40, 0.2, cap=4.0, rot_dims=8, base=300.0, kv_from=0), moe(5, 5, 40)),
             layer(attention(3, 3, 16, 8, 0.25, cap=None, base=50.0, stretch=(2.0, 64, 8.0, 0.5), kv_from=1), moe(8, 3, 16, (4, 2))),
             layer(attention(2, 2, 24, 40, 0.3, cap=9.0, rot_dims=8, base=300.0, kv_from=0), moe(6, 1, 56, (2, 1)))],
            vocab=211, width=96, logit_scale=0.7, bigram=(101, 37, 5))
# Sizes the matrix cores like: heads of 64 with value heads of 96, heads of 128 and 128; one key head for eight query heads;
# no stretched frequencies in one layer; every expert used; the cap hardly acts.
N_B = model([layer(attention(4, 2, 64, 96, 0.125, cap=30.0, rot_dims=32, base=10000.0, stretch=(4.0, 128, 16.0, 1.0)), moe(8, 4, 64, (4, 3))),
             layer(attention(8, 1, 128, 128, 0.1, cap=12.0, base=500000.0, stretch=None), moe(16, 3, 72, (8, 4))),
             layer(attention(8, 1, 128, 128, 0.06, cap=20.0, base=500000.0, stretch=None, kv_from=1), moe(4, 4, 128, (2, 2)))],
            vocab=300, width=128, eps=1e-6, logit_scale=2.5, bigram=(997, 1000003, 17))
# Sizes that 16-byte loads do not divide: a width of 100, heads of 12, 20 and 7, feed-forwards of 52 and 28; one bucket; no
# rotation in one layer; one expert; a multiplier of 0 beside one larger than the table.
N_C = model([layer(attention(5, 5, 12, 20, 0.4, cap=3.0, rot_dims=0), moe(1, 1, 52)), layer(attention(6, 3, 20, 12, 0.3, rot_dims=6, base=20.0), moe(6, 2, 28, (6, 3))),
             layer(attention(3, 1, 7, 9, 0.5, rot_dims=2, base=7.0, kv_from=None), moe(10, 4, 12, (2, 1)))],
            vocab=157, width=100, eps=1e-3, logit_scale=1.0, bigram=(1, 0, 12345))
# One layer that owns its keys and three that read them, heads of 32 (the same sizes as the matrix cores' first kernels).
N_D = model([layer(attention(4, 4, 32, 32, 0.18, cap=15.0, base=1000.0), moe(12, 3, 40, (3, 2)))] +
            [layer(attention(4 * n, 4, 32, 32, 0.18, cap=15.0, base=1000.0, kv_from=0), moe(4 * n, n, 24, (2, 1))) for n in (1, 2, 4)],
            vocab=333, width=136, logit_scale=1.3, bigram=(333, 1, 1))
CONFIGS = {"A": N_A, "B": N_B, "C": N_C, "D": N_D}


def sharpen(folder):
    """Random weights as the library draws them, with the tensors that small or level values would switch off made to
    count: the routers and their corrections (choice scores of either sign), every bias, the gains of the norms."""
    from safetensors.torch import load_file, save_file
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    g = torch.Generator().manual_seed(len(w))
    draw = lambda like, std, mean=0.0: (mean + std * torch.randn(like.shape, generator=g)).to(like.dtype)
    for name in sorted(w):
        if name.endswith(".router"):
            w[name] = (w[name].float() * 1.5).to(w[name].dtype)
        elif name.endswith(".correction"):
            w[name] = draw(w[name], 0.4, -0.5)
        elif name.endswith(".b"):
            w[name] = draw(w[name], 0.4)
        elif name.endswith((".norm1", ".norm1b", ".norm2", ".norm2b", ".norm")):
            w[name] = draw(w[name], 0.25)
        elif name == "bigram":
            w[name] = (w[name].float() * 1.5).to(w[name].dtype)
    save_file(w, path)
    return folder


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    from rust_inference_amd.weights import write_random_model
    base = tmp_path_factory.mktemp("notadra")
    return {name: sharpen(write_random_model(str(base / name), cfg, seed, torch.bfloat16, matrix_std=0.12))
            for seed, (name, cfg) in enumerate(CONFIGS.items())}


_models, _plain, _read, _settled = {}, {}, {}, {}


def loaded(folders, name, dtype_name):
    from rust_inference_amd.parts import load_model
    if (name, dtype_name) not in _models:
        _models[(name, dtype_name)] = load_model(folders[name], DTYPES[dtype_name])
    return _models[(name, dtype_name)]


def plain_logits(folder, tokens):
    key = (folder, tuple(tokens))
    if key not in _plain:
        if folder not in _read:
            _read[folder] = read_model_f64(folder)
        gaps = []
        _plain[key] = P.forward(*_read[folder], list(tokens), gaps=gaps)
        _settled[key] = np.min(gaps, axis=0) if gaps else np.full(len(tokens), np.inf)
    return _plain[key]


def unclear(folder, tokens, dtype_name):
    """The positions at which a router's call is so close (two choice scores, or two groups' scores) that another
    implementation may rightly send the token elsewhere.  A token's other experts reach later tokens through the keys of the
    layers above alone, one among many."""
    plain_logits(folder, tokens)
    return _settled[(folder, tuple(tokens))] < (1e-5 if dtype_name == "float32" else 2e-2)


def near(got, want, dtype_name, what, bound, median=2e-2):
    """float32: every position.  bfloat16: the positions' errors of the largest logit have a median of 2e-2 (or ``median``) at most, and one in
    six at most is over ``bound``: with weights this large a token whose experts were another choice than the plain form's
    shows in the later tokens that look at it."""
    if dtype_name == "float32":
        return close_enough(got, want, dtype_name, what, bound)
    if len(got):
        errs = np.abs(np.asarray(got, dtype=np.float64) - want).max(-1) / np.abs(want).max()
        assert np.median(errs) <= median and (errs > bound).sum() <= max(2, len(errs) / 6), \
            f"{what}: {int((errs > bound).sum())} of {len(errs)} positions differ by more than {bound:.0e}, the median {np.median(errs):.2e}, the worst {errs.max():.2e}"


def against_plain(folder, got, requests, dtype_name, what, bound=5e-2, median=2e-2):
    for rid, toks in requests.items():
        want, skip = plain_logits(folder, toks), unclear(folder, toks, dtype_name)
        if dtype_name == "float32":
            assert skip.sum() <= 1, f"request {rid}: a router's close calls at {int(skip.sum())} positions: choose other tokens"
        near(got[rid][~skip], want[~skip], dtype_name, f"{what}, request {rid}", bound, median)


def among_themselves(folder, got, other, requests, dtype_name, what):
    bound = 2e-5 if dtype_name == "float32" else 5e-2
    for rid, toks in requests.items():
        ok = ~unclear(folder, toks, dtype_name)
        near(got[rid][ok], other[rid][ok].astype(np.float64), dtype_name, f"{rid}: {what}", bound)


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
                        ("portions of 64, 1 and 7", in_portions(reqs, [64, 1, 7]))):
        got = replay(model_, steps)
        against_plain(folders[name], got, reqs, dtype_name, what)
        among_themselves(folders[name], got, whole, reqs, dtype_name, f"{what}, against the whole prompt")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_unequal_batches_one_after_another(folders, name, dtype_name):
    rng = np.random.default_rng(8)
    batches, reqs = [], {}
    for b in range(3):                                       # three batches on one cache: slots, pages and kept tokens come back
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
    among_themselves(folders[name], got, replay(model_, plans.whole(reqs)), reqs, dtype_name, "in a batch against itself alone")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_long_decoding_from_the_first_tokens(folders, name, dtype_name):
    """Three tokens of prompt, then 200 one by one: over page borders."""
    reqs = requests_for(CONFIGS[name], name, [203], 3)
    got = replay(loaded(folders, name, dtype_name), plans.tail_one_by_one(reqs, 200))
    against_plain(folders[name], got, reqs, dtype_name, "long decoding")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_the_ways_through_the_experts_agree(folders, dtype_name):
    """A prompt of 330 tokens (its tokens sorted by expert), the same in portions of 100 (all experts for all tokens) and
    its last tokens one by one (the chosen experts' rows alone), with a second request beside it."""
    reqs = requests_for(N_B, "B", [330, 290], 9)
    model_ = loaded(folders, "B", dtype_name)
    for what, steps in (("whole", plans.whole(reqs)), ("portions of 100", in_portions(reqs, [100])), ("one by one", plans.tail_one_by_one(reqs, 6)),
                        ("a batch, then one by one", plans.unequal_batches([{rid: (toks, len(toks) - 6) for rid, toks in reqs.items()}]))):
        against_plain(folders["B"], replay(model_, steps), reqs, dtype_name, what)


def test_the_stream_of_layers_in_float32(folders):
    """A prompt layer by layer: every layer alone on top of the ones before it, so that a difference names its layer."""
    from rust_inference_amd.engine.replay import engine_for_trace
    from rust_inference_amd.engine.step import StepEntry
    for name in CONFIGS:
        cfg, w = read_model_f64(folders[name])
        toks = requests_for(CONFIGS[name], name, [41], 6)[f"{name}0"]
        layers = []
        P.forward(cfg, w, toks, layers_out=layers)
        model_ = loaded(folders, name, "float32")
        seen = []
        undo = []
        for arrangement in model_.layers:
            run = arrangement.forward

            def watched(stream, *a, _run=run):
                _run(stream, *a)
                seen.append(stream.sum.detach().cpu().numpy().copy())
            arrangement.forward = watched
            undo.append((arrangement, run))
        try:
            engine = engine_for_trace(model_, 64)
            engine.step([StepEntry(engine.cache.acquire(), toks, "last")])
        finally:
            for arrangement, _ in undo:
                del arrangement.forward
        assert len(seen) == len(layers)
        for i, (got, want) in enumerate(zip(seen, layers)):
            assert rel_to_max(got, want) < 1e-5, f"{name}: after layer {i}"


# ---------------------------------------------------------------- made to show
FAR_SCALE = 24.0              # over the head size: a score scale at which one key can take the softmax


def one_layer(tmp_path_factory, tag, mixer, seed, **kw):
    from rust_inference_amd.weights import write_random_model
    cfg = model([layer(mixer, None)], vocab=80, width=32, **kw)
    return cfg, write_random_model(str(tmp_path_factory.mktemp(tag)), cfg, seed, torch.bfloat16, matrix_std=0.3)


def changed(folder, **tensors):
    """The folder with tensors replaced: a function of the stored one each, by name with '_' for '.'."""
    from safetensors.torch import load_file, save_file
    path = os.path.join(folder, "model.safetensors")
    w = load_file(path)
    for name, f in tensors.items():
        name = next(n for n in w if n.replace(".", "_") == name)
        w[name] = f(w[name].float()).to(w[name].dtype).contiguous()
    save_file(w, path)
    return folder


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim, vdim, place, seed", [(16, 24, 64, 7), (64, 88, 63, 3), (64, 64, 31, 3), (128, 144, 0, 3)])
def test_a_far_key_among_hundreds(tmp_path_factory, dim, vdim, place, seed, dtype_name):
    """A score scale at which one key can take the softmax: the last logits must see a token 700 positions back, at a page's
    first or last place or at the sequence's start.  No pairs beside the tokens (one bucket), so that the key alone tells."""
    from rust_inference_amd.parts import load_model
    cfg, folder = one_layer(tmp_path_factory, f"far{dim}_{place}", attention(2, 1, dim, vdim, FAR_SCALE / dim, cap=20.0, rot_dims=8, base=1e6), seed, bigram=(1, 1, 1))
    rng = np.random.default_rng(5)
    toks = [int(t) for t in rng.integers(0, 40, 760)]
    cfg_, w_ = read_model_f64(folder)
    # of the tokens seen nowhere else, the one whose key moves the last logits most against another one's
    rows = {c: P.forward(cfg_, w_, toks[:place] + [c] + toks[place + 1:])[-30:] for c in range(40, 80, 3)}
    loud, quiet = max(((c, d) for c in rows for d in rows if c != d), key=lambda p: rel_to_max(rows[p[1]], rows[p[0]]))
    toks[place] = loud
    want = plain_logits(folder, toks)
    other = toks[:place] + [quiet] + toks[place + 1:]
    assert rel_to_max(P.forward(cfg_, w_, other)[-30:], want[-30:]) > 8e-2, "the far token does not reach the last logits"
    model_ = load_model(folder, DTYPES[dtype_name])
    reqs = {"f": toks}
    for what, steps in (("whole", plans.whole(reqs)), ("the last 40 one by one", plans.tail_one_by_one(reqs, 40)),
                        ("portions", in_portions(reqs, [300, 2, 255]))):
        err = rel_to_max(replay(model_, steps)["f"], want)
        assert err < (1e-4 if dtype_name == "float32" else 4e-2), f"far key, {what}: {err:.2e}"


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim, vdim", [(16, 24), (64, 64), (64, 72)])
def test_the_sink_of_score_zero_at_the_first_tokens(tmp_path_factory, dim, vdim, dtype_name):
    """Scores near zero: the first tokens lose half, a third, a quarter of their weight to the sink, which the norm behind the
    sublayer would hide if the values were all there is; the value's bias is taken out and the residual kept small, and the
    plain form without a sink gives other logits."""
    from rust_inference_amd.parts import load_model
    cfg, folder = one_layer(tmp_path_factory, f"sink{dim}_{vdim}", attention(2, 1, dim, vdim, 0.01, cap=5.0), 4, eps=0.5)
    changed(folder, l0_mix_v=lambda x: x * 0.5, embed=lambda x: x * 0.5, bigram=lambda x: x * 0.5)
    cfg_, w_ = read_model_f64(folder)
    toks = requests_for(cfg, "s", [70], 2)["s0"]
    want = plain_logits(folder, toks)
    real, P.capped_attention = P.capped_attention, None
    try:
        def no_sink(q, keys, vals, start, scale, cap):
            o = real(q, keys, vals, start, scale, cap)
            for i in range(q.shape[0]):
                s = np.stack([keys[:start + i + 1, hd // (q.shape[1] // keys.shape[1])] @ q[i, hd] for hd in range(q.shape[1])]) * scale
                e = np.exp(cap * np.tanh(s / cap)).sum(-1)
                o[i] *= ((1 + e) / e)[:, None]
            return o
        P.capped_attention = no_sink
        without = P.forward(cfg_, w_, toks)
    finally:
        P.capped_attention = real
    moved = np.abs(without - want).max(-1) / np.abs(want).max()
    assert moved[:2].min() > 4e-2, f"the sink does not show at the first tokens: {moved[:2]}"
    model_ = load_model(folder, DTYPES[dtype_name])
    reqs = {"s": toks}
    for what, steps in (("whole", plans.whole(reqs)), ("one by one", plans.tail_one_by_one(reqs, 69)), ("portions", in_portions(reqs, [2, 3]))):
        assert_logits_close(replay(model_, steps)["s"], want, dtype_name, f"sink, {what}")


@pytest.mark.parametrize("cuts", [[90], [1] * 40 + [50], [33, 2, 55], [89, 1], [2] * 45])
def test_the_token_before_survives_every_cut(tmp_path_factory, cuts):
    """Pairs whose rows are as large as the tokens' own; another request comes and goes between the portions, on the slot
    next to this one, and afterwards a request on this one's slot starts with the last row again."""
    from rust_inference_amd.parts import load_model
    cfg, folder = one_layer(tmp_path_factory, "pairs", attention(2, 2, 8, 8, 0.2), 5, bigram=(1009, 83, 1))
    toks = requests_for(cfg, "p", [90], 4)["p0"]
    want = plain_logits(folder, toks)
    other = plain_logits(folder, toks[:49] + [toks[49] ^ 1] + toks[50:])
    assert rel_to_max(other[50], want[50]) > 5e-2, "the token before does not reach the logits: the test shows nothing"
    model_ = load_model(folder, torch.float32)
    steps, at = [], 0
    for n in cuts:
        steps.append({"step": len(steps), "entries": [{"id": "x", "tokens": toks[at:at + n], "want": list(range(n))}], "end": []})
        steps.append({"step": len(steps), "entries": [{"id": f"o{at}", "tokens": toks[5:10], "want": []}], "end": [f"o{at}"]})
        at += n
    steps[-1]["end"].append("x")
    steps.append({"step": len(steps), "entries": [{"id": "y", "tokens": toks[:7], "want": list(range(7))}], "end": ["y"]})
    got = replay(model_, steps)
    assert_logits_close(got["x"], want, "float32", f"cuts {cuts[:3]}")
    assert_logits_close(got["y"], want[:7], "float32", "the slot again")


@pytest.mark.parametrize("dtype_name", ["float32", "bfloat16"])
def test_a_layer_reads_the_keys_of_the_layer_it_names(tmp_path_factory, dtype_name):
    """Three layers with keys of their own and one that reads the second's: with another one's the logits differ."""
    from rust_inference_amd.parts import load_model
    from rust_inference_amd.weights import write_random_model
    mixer = lambda kv_from=None: attention(4, 2, 16, 24, 0.6, cap=6.0, rot_dims=8, kv_from=kv_from)
    cfg = model([layer(mixer(), None)] * 3 + [layer(mixer(1), None)], vocab=80, width=48)
    folder = write_random_model(str(tmp_path_factory.mktemp("shared")), cfg, 6, torch.bfloat16, matrix_std=0.3)
    toks = requests_for(cfg, "k", [80], 7)["k0"]
    want = plain_logits(folder, toks)
    cfg_, w_ = read_model_f64(folder)
    for wrong in (0, 2):
        cfg_["layers"][3]["mixer"]["kv_from"] = wrong
        assert rel_to_max(P.forward(cfg_, w_, toks), want) > 1e-1
    model_ = load_model(folder, DTYPES[dtype_name])
    reqs = {"k": toks}
    for what, steps in (("whole", plans.whole(reqs)), ("one by one", plans.tail_one_by_one(reqs, 50)), ("portions", in_portions(reqs, [31, 2]))):
        err = rel_to_max(replay(model_, steps)["k"], want)
        assert err < (1e-4 if dtype_name == "float32" else 4e-2), f"shared keys, {what}: {err:.2e}"


# ---------------------------------------------------------------- the library's own ways in
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
        toks = list(p)
        for i, a in enumerate(g):
            row = P.forward(cfg, w, toks)[-1]
            b = int(np.argmax(row))
            if a != b:
                top = np.sort(row)
                assert (top[-1] - top[-2] < (1e-4 if dtype_name == "float32" else 0.08) * np.abs(row).max()
                        or unclear(folders[name], toks, dtype_name).any()), f"token {i} is {a}, plain says {b}"
                break                                                   # from here on the two follow different texts
            toks.append(a)
    model_.cache.check_consistent()


def test_the_invariant_mode_gives_the_same_bits_however_a_request_is_cut(folders):
    from rust_inference_amd.parts import load_model
    name = "B"
    model_ = load_model(folders[name], torch.bfloat16, invariant=True)
    reqs = requests_for(CONFIGS[name], name, [70, 33], 11)
    whole = replay(model_, plans.whole(reqs))
    against_plain(folders[name], whole, reqs, "bfloat16", "invariant, whole")
    for steps in (plans.tail_one_by_one(reqs, 20), plans.unequal_batches([{rid: (toks, len(toks) - 5) for rid, toks in reqs.items()}]), in_portions(reqs, [31, 2])):
        got = replay(model_, steps)
        for rid in reqs:
            assert (got[rid] == whole[rid]).all(), rid


def test_the_trace_program(folders, tmp_path):
    reqs = requests_for(N_A, "t", [40, 9], 6)
    steps = plans.unequal_batches([{rid: (toks, len(toks) - 4) for rid, toks in reqs.items()}])
    out = str(tmp_path / "out")
    proc = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folders["A"], "--dtype", "float32",
                           "--out", out, "--max-tokens", str(plans.max_live_tokens(steps))],
                          input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.splitlines() if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    got = plans.collect(steps, lambda i: np.fromfile(os.path.join(out, f"{i}.f32"), dtype="<f4"), N_A["vocab"])
    against_plain(folders["A"], got, reqs, "float32", "trace program")


def drawn_config(seed):
    """A configuration drawn at random: sizes, head counts, number and order of layers, which layers read which one's keys,
    constants, with feed-forwards and without."""
    rng = np.random.default_rng(9000 + seed)
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers = []
    for i in range(int(rng.integers(1, 7))):
        count = pick([1, 2, 3, 4])
        per = pick([1, 2, 3, 5])
        keep = int(rng.integers(1, count + 1))
        mlp = pick([None, 1, 1, 1])
        if mlp is not None:
            mlp = moe(count * per, int(rng.integers(1, min(4, keep * per) + 1)), pick([8, 24, 56, 44]), pick([None, (count, keep)]))
        owners = [j for j, l in enumerate(layers) if l["mixer"].get("kv_from") is None]
        if owners and rng.random() < 0.4:
            j = pick(owners)
            mixer = {**layers[j]["mixer"], "kv_from": j, "scale": float(rng.uniform(0.05, 0.4)), "softcap": float(pick([3.0, 10.0, 40.0]))}
        else:
            kv, dim = pick([1, 2, 3, 4]), pick([8, 12, 16, 32, 40, 64, 72, 128])
            stretch = pick([None, (float(pick([1.5, 2.0, 8.0])), pick([40, 128, 900]), float(pick([4.0, 32.0])), float(pick([0.5, 1.0, 2.0])))])
            mixer = attention(kv * pick([1, 2, 4]), kv, dim, pick([8, 20, 32, 64, 96, 128, 160]), float(rng.uniform(0.05, 0.4)),
                              cap=pick([None, 3.0, 10.0, 30.0]), rot_dims=2 * int(rng.integers(0, dim // 2 + 1)), base=float(pick([50.0, 10000.0, 500000.0])),
                              stretch=stretch)
        layers.append(layer(mixer, mlp))
    buckets = pick([1, 17, 503, 4099])
    return model(layers, vocab=int(rng.integers(50, 400)), width=pick([48, 80, 136, 192]), eps=pick([1e-5, 1e-6, 1e-3]),
                 logit_scale=float(rng.uniform(0.3, 3.0)), bigram=(buckets, int(rng.integers(0, 2000)), int(rng.integers(0, 2000))))


@pytest.mark.parametrize("seed", range(12))
def test_configurations_drawn_at_random(tmp_path, seed):
    from rust_inference_amd.parts import load_model
    from rust_inference_amd.weights import write_random_model
    cfg = drawn_config(seed)
    folder = sharpen(write_random_model(str(tmp_path / "m"), cfg, seed, torch.bfloat16, matrix_std=0.12))
    rng = np.random.default_rng(seed)
    reqs = {f"r{i}": [int(t) for t in rng.integers(0, cfg["vocab"], n)] for i, n in enumerate((150, 37, 1, 66))}
    batch = {rid: (toks, max(1, len(toks) - 9)) for rid, toks in reqs.items()}
    for dtype_name in ("float32", "bfloat16"):
        model_ = load_model(folder, DTYPES[dtype_name])
        for what, steps in (("whole", plans.whole(reqs)), ("last 32 one by one", plans.tail_one_by_one(reqs, 32)),
                            ("a batch", plans.unequal_batches([batch])), ("portions", in_portions(reqs, [33, 2, 64]))):
            got = replay(model_, steps)
            # (scores of ten and more in some of these: a bfloat16 query or key moves a weight by several per cent)
            against_plain(folder, got, reqs, dtype_name, f"configuration {seed}, {what}", 8e-2 if dtype_name == "bfloat16" else 5e-2, 3e-2)


def test_the_command_line_generates_what_the_plain_implementation_does(folders):
    """bin/runner on a Notadra folder, prompts as token ids: greedy in float32, sections timed, and a seeded temperature
    run that gives the same tokens twice."""
    cfg, w = read_model_f64(folders["A"])
    prompts = list(requests_for(N_A, "c", [9, 14], 8).values())
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
