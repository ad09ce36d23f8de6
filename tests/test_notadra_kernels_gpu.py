"""The kernels of the Notadra design alone, each against the plain function of its mechanism
(tests/plain/notadra_plain.py), at sizes that are no power of two and differ from one another.

Like tests/test_kernels_gpu.py these run without a GPU when the environment says RI_TEST_KERNELS=emulated
(tests/test_kernels_emulated.py starts that run): the CPU build of the same sources between guard pages."""
import os

import numpy as np
import pytest
import torch

from plain import notadra_plain as P

EMULATED = os.environ.get("RI_TEST_KERNELS") == "emulated"
pytestmark = [] if EMULATED else pytest.mark.gpu
DEV = "cpu" if EMULATED else "cuda:0"
PAGE = 32


@pytest.fixture(scope="module")
def ops():
    if EMULATED:
        import emulated
        return emulated.ops()
    from rust_inference_amd.kernels import ops
    return ops


@pytest.fixture(autouse=True)
def _guarded_buffers_go_back():
    yield
    if EMULATED:
        import gc
        import emulated
        gc.collect()
        emulated.free_all()


def guarded(x):
    if EMULATED:
        import emulated
        return emulated.tensor(x.contiguous(), "a test's operand")
    return x


def t(a, dtype=torch.float32):
    return guarded(torch.tensor(np.asarray(a), dtype=dtype, device=DEV))


def f64(x):
    return x.detach().to("cpu", torch.float64).numpy()


def close(got, want, rel, what=""):
    want = np.asarray(want, dtype=np.float64)
    err = np.abs(f64(got) - want).max() / max(np.abs(want).max(), 1e-30)
    assert err <= rel, f"{what}: error {err:.3e} of the largest value exceeds {rel:.0e}"


def bf16_round(a):
    return torch.tensor(np.asarray(a)).to(torch.bfloat16).to(torch.float64).numpy()


F32 = 3e-6
BF16_OUT = 7.5e-3


# ---------------------------------------------------------------- the embedding of pairs
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("dim, buckets, mul_prev, mul_cur", [(52, 37, 29, 11), (51, 1, 3, 5), (2052, 101, 2 ** 40 + 13, 999983), (8, 64, 0, 1)])
def test_the_embedding_of_pairs_of_tokens(ops, dtype, dim, buckets, mul_prev, mul_cur):
    """Three sequences on slots of their own, their tokens in steps of 5, 1 and 2, 1, 3, 4: the first token reads the last
    row, the token kept from the step before counts, and a slot that is used again starts afresh."""
    rng = np.random.default_rng(dim)
    vocab = 211
    bigram = {"buckets": buckets, "mul_prev": mul_prev, "mul_cur": mul_cur}
    w = {"embed": bf16_round(rng.normal(size=(vocab, dim))), "bigram": bf16_round(rng.normal(size=(buckets + 1, dim)))}
    table, pairs = t(w["embed"], dtype), t(w["bigram"], dtype)
    last = t(np.full((5, 1), 17), torch.int32)                # what an earlier sequence left
    seqs = {0: (3, rng.integers(0, vocab, 13).tolist()), 1: (0, rng.integers(0, vocab, 9).tolist()), 2: (4, rng.integers(0, vocab, 11).tolist())}
    plain, at = {b: {} for b in seqs}, {b: 0 for b in seqs}
    for step in ({0: 5, 1: 1, 2: 2}, {0: 1, 1: 1, 2: 1}, {2: 3, 0: 4}, {1: 2}, {0: 1, 2: 2}):
        ids, pos, seq, cu, slots, want = [], [], [], [0], [], []
        for i, (b, n) in enumerate(step.items()):
            slot, toks = seqs[b]
            new = toks[at[b]:at[b] + n]
            ids += new
            pos += list(range(at[b], at[b] + n))
            seq += [i] * n
            cu.append(len(ids))
            slots.append(slot)
            want.append(P.embed(new, w, bigram, plain[b]))
            at[b] += n
        got = ops.embed_bigram(table, pairs, t(ids, torch.int32), t(pos, torch.int32), t(seq, torch.int32), t(cu, torch.int32),
                               t(slots, torch.int32), last, mul_prev, mul_cur)
        close(got, np.concatenate(want), 1e-7, f"step {step}")
        for b in step:
            assert int(last[seqs[b][0], 0]) == seqs[b][1][at[b] - 1]
    assert int(last[1, 0]) == 17 and int(last[2, 0]) == 17    # slots no sequence had


# ---------------------------------------------------------------- the norms around a sublayer
@pytest.mark.parametrize("y_dtype, parts", [(torch.float32, 1), (torch.float32, 3), (torch.bfloat16, 1)])
@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("dim", [36, 51, 1028, 2052, 4100, 8192, 8200])
def test_a_norm_behind_a_sublayer_the_sum_and_the_norm_ahead(ops, dim, act, y_dtype, parts):
    rng = np.random.default_rng(dim + parts)
    rows, eps, eps2 = 3, 1e-3, 2e-2
    x, y = rng.normal(size=(rows, dim)), rng.normal(size=(parts, rows, dim)) * 4
    y[:, 1] *= 1e-2                                           # a row whose norm eps shows in
    if y_dtype == torch.bfloat16:
        y = bf16_round(y)
    g1, g2 = rng.normal(size=dim) * 0.3, rng.normal(size=dim) * 0.3
    new = x + P.rms_norm(y.sum(0), g1, eps)
    want = P.rms_norm(new, g2, eps2)
    for tiled in ([False, True] if act == torch.bfloat16 and dim % 4 == 0 and dim <= 8192 else [False]):
        res = t(x)
        got = ops.branch_norm_add_norm(res, t(y if parts > 1 else y[0], y_dtype), t(1 + g1), None, eps, ops.NORM_RMS, None, t(1 + g2), eps2, act, tiled)
        close(res, new, F32, "the residual")
        close(ops.as_rows(got), want, F32 if act == torch.float32 else BF16_OUT, "the next norm")


# ---------------------------------------------------------------- biases, rotation in halves, the cache write
def rot_of(dims, base, factor=None, original=64, fast=8.0, slow=0.5):
    return {"dims": dims, "base": base, "scaling": None if factor is None else {"factor": factor, "original": original, "fast": fast, "slow": slow}}


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads, kv, dim, vdim, rot", [(6, 2, 24, 40, rot_of(16, 100.0, 3.0)), (3, 3, 20, 12, rot_of(10, 1e4)), (4, 1, 64, 88, rot_of(64, 5e5, 8.0)),
                                                       (2, 2, 9, 7, rot_of(0, 1.0)), (5, 5, 136, 16, rot_of(48, 1e3, 1.5)), (2, 1, 130, 130, rot_of(130, 1e4, 2.0))])
@pytest.mark.parametrize("form", ["prompts", "single tokens", "portions", "queries alone", "one queries alone"])
def test_biases_rotation_in_halves_and_the_cache_write(ops, form, heads, kv, dim, vdim, rot, dtype):
    rng = np.random.default_rng(heads * dim)
    lens = [1, 1, 1] if "one" in form or form == "single tokens" else [45, 1, 70]
    starts = [0, 0, 0] if form == "prompts" else [33, 5, 64]
    own = 0 if "alone" in form else kv
    T = sum(lens)
    width = heads * dim + own * (dim + vdim)
    lead = 8                                                  # columns of something else ahead
    proj, bias = rng.normal(size=(T, lead + width)), rng.normal(size=width)
    if dtype == torch.bfloat16:
        proj = bf16_round(proj)
    pos, seq, cu = [], [], [0]
    for b, (n, s) in enumerate(zip(lens, starts)):
        pos += list(range(s, s + n))
        seq += [b] * n
        cu.append(len(pos))
    pages = 17
    table = rng.permutation(pages)[:15].reshape(3, 5)
    kp, vp = t(np.full((pages, kv, PAGE, dim), 7.0), dtype), t(np.full((pages, kv, vdim, PAGE), 7.0), dtype)
    freq, mult = P.frequencies(rot) if rot["dims"] else (None, 1.0)
    turn = (lambda x: P.rotate_half(x, np.array(pos, dtype=np.float64), rot)) if rot["dims"] else (lambda x: x)
    full = proj[:, lead:] + bias
    want_q = turn(full[:, :heads * dim].reshape(T, heads, dim))
    row = t(proj, dtype)
    ops.qk_half_bias_kv_write(row, lead, lead + heads * dim, lead + (heads + own) * dim, t(bias), None if freq is None else t(freq), mult,
                              t(pos, torch.int32), t(seq, torch.int32), t(table, torch.int32), kp, vp, heads, own, dim, vdim,
                              t(cu, torch.int32), max(lens))
    tol = 2e-5 if dtype == torch.float32 else BF16_OUT        # (an angle near 130 in float32: 1e-5)
    close(row[:, :lead], proj[:, :lead], 1e-7, "the columns ahead")
    close(row[:, lead:lead + heads * dim], want_q.reshape(T, -1), tol, "q")
    want_kp, want_vp = np.full(kp.shape, 7.0), np.full(vp.shape, 7.0)
    if own:
        want_k = turn(full[:, heads * dim:(heads + kv) * dim].reshape(T, kv, dim))
        want_v = full[:, (heads + kv) * dim:].reshape(T, kv, vdim)
        for i in range(T):
            page, at = table[seq[i], pos[i] // PAGE], pos[i] % PAGE
            want_kp[page, :, at], want_vp[page, :, :, at] = want_k[i], want_v[i]
    close(kp, want_kp, tol, "the key pages, where nothing was written too")
    close(vp, want_vp, tol, "the value pages")
    if not own:
        assert (f64(kp) == 7.0).all() and (f64(vp) == 7.0).all()


def test_the_stretched_frequencies_by_hand():
    from rust_inference_amd.parts import PartSpec, build_part
    for dims, base, sc in ((48, 3e4, (2.5, 2000, 24.0, 1.5)), (64, 1e6, (4.0, 32768, 32.0, 1.0)), (8, 10.0, (8.0, 4, 40.0, 30.0)), (16, 500.0, (1.0, 100, 3.0, 3.0)),
                           (6, 3.0, (2.0, 100000, 32.0, 0.001))):
        stretch = dict(zip(("factor", "original", "fast", "slow"), sc))
        part = build_part("position", PartSpec("rotate_half", {"head_dim": 64, "theta": base, "dims": dims, "stretch": stretch}))
        freq, mult = P.frequencies({"dims": dims, "base": base, "scaling": stretch})
        assert np.allclose(part.part_frequencies().numpy(), freq, rtol=1e-12) and abs(part.amplitude - mult) < 1e-12
    # the fastest pair keeps its frequency, the slowest turns four times slower
    freq = P.frequencies({"dims": 64, "base": 1e6, "scaling": {"factor": 4.0, "original": 32768, "fast": 32.0, "slow": 1.0}})[0]
    assert freq[0] == 1.0 and np.isclose(freq[31], 1e6 ** (-62 / 64) / 4)


# ---------------------------------------------------------------- attention
def paged_batch(k, v, lens, seed, dtype=torch.bfloat16):
    """Keys and values of several sequences (flat, one after the other) in pages handed out in shuffled order."""
    G, dk, dv = k.shape[1], k.shape[2], v.shape[2]
    width = max(-(-n // PAGE) for n in lens) + 1
    n_pages = sum(-(-n // PAGE) for n in lens) + 2
    order = np.random.default_rng(seed).permutation(n_pages)
    table = np.full((len(lens), width), -1, dtype=np.int32)
    kp = torch.zeros((n_pages, G, PAGE, dk), dtype=dtype)
    vp = torch.zeros((n_pages, G, dv, PAGE), dtype=dtype)
    nxt = at = 0
    for b, n in enumerate(lens):
        for p in range(-(-n // PAGE)):
            table[b, p] = order[nxt]
            nxt += 1
        for j in range(n):
            kp[table[b, j // PAGE], :, j % PAGE] = torch.tensor(k[at + j]).to(dtype)
            vp[table[b, j // PAGE], :, :, j % PAGE] = torch.tensor(v[at + j]).to(dtype)
        at += n
    return guarded(kp.to(DEV)), guarded(vp.to(DEV)), t(table, torch.int32)


def attention_case(rng, lens, heads, kv, dim, vdim, scale, cap, size=1.0):
    T = sum(lens)
    q, k, v = (bf16_round(rng.normal(size=(T, n, d)) * s) for n, d, s in ((heads, dim, size), (kv, dim, size), (kv, vdim, 1.0)))
    cu = np.concatenate([[0], np.cumsum(lens)])
    want = np.concatenate([P.capped_attention(q[a:b], k[a:b], v[a:b], 0, scale, cap).reshape(b - a, -1) for a, b in zip(cu[:-1], cu[1:])])
    return q, k, v, cu, want


def rows_of(lens, cu, tail):
    """The flat rows of the sequences' last ``tail`` tokens (all of them: None), their positions and the new offsets."""
    rows, pos, new_cu = [], [], [0]
    for a, b in zip(cu[:-1], cu[1:]):
        first = a if tail is None else max(a, b - tail)
        rows += list(range(first, b))
        pos += list(range(first - a, b - a))
        new_cu.append(len(rows))
    return rows, pos, new_cu


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads, kv, dim, vdim, cap", [(6, 2, 24, 40, 5.0), (3, 3, 16, 8, None), (4, 1, 20, 12, 2.0)])
def test_generic_attention_with_a_cap_and_a_sink_of_zero(ops, dtype, heads, kv, dim, vdim, cap):
    rng = np.random.default_rng(heads * 10 + dim)
    lens = [75, 1, 40]
    q, k, v, cu, want = attention_case(rng, lens, heads, kv, dim, vdim, 0.31, cap, 1.5)
    kp, vp, table = paged_batch(k, v, lens, dim, dtype)
    rows, pos, _ = rows_of(lens, cu, None)
    seq = np.repeat(np.arange(3), lens)
    got = ops.attention(t(q.reshape(len(rows), -1), dtype), kp, vp, t(pos, torch.int32), t(seq, torch.int32), table, heads, kv, dim, None, 0.31,
                        cap, None, sinks=t(np.zeros(heads)))
    close(got, want, F32 if dtype == torch.float32 else BF16_OUT)
    # a token alone weighs its own value by exp(s) / (1 + exp(s)), not by 1
    s = (q[75] * np.repeat(k[75], heads // kv, 0)).sum(-1) * 0.31
    s = cap * np.tanh(s / cap) if cap else s
    assert np.allclose(want[75].reshape(heads, vdim), np.repeat(v[75], heads // kv, 0) * (1 / (1 + np.exp(-s)))[:, None])


PADDED = [(8, 4, 64, 88), (4, 1, 128, 160), (2, 2, 24, 36), (6, 3, 96, 96), (16, 1, 40, 64), (3, 3, 128, 252), (4, 2, 64, 128), (2, 1, 8, 4), (4, 4, 128, 72)]


@pytest.mark.parametrize("heads, kv, dim, vdim", PADDED)
@pytest.mark.parametrize("form", ["prompts", "single tokens", "portions"])
def test_matrix_core_attention_with_head_sizes_of_their_own(ops, form, heads, kv, dim, vdim):
    """bfloat16, key and value heads of sizes of their own: prompts of unequal lengths, one new token each, the last tokens
    of each as a portion; a cap, a sink of 0; a scale at which a key can stand out."""
    rng = np.random.default_rng(dim + heads)
    lens = [75, 1, 40] if form == "prompts" else [300, 33, 164]
    scale = 2.0 / dim ** 0.5
    q, k, v, cu, want = attention_case(rng, lens, heads, kv, dim, vdim, scale, 6.0)
    kp, vp, table = paged_batch(k, v, lens, dim)
    rows, pos, new_cu = rows_of(lens, cu, {"prompts": None, "single tokens": 1, "portions": 19}[form])
    wide = np.concatenate([np.full((len(rows), 16), 9.0), q[rows].reshape(len(rows), -1), np.full((len(rows), 8), 9.0)], 1)
    kw = {"softcap": 6.0, "sinks": t(np.zeros(heads)), "q_off": 16}
    assert ops.padded_attention_fits(torch.bfloat16, dim, vdim, heads // kv, PAGE, False)
    got = ops.attention_prefill_padded(t(wide, torch.bfloat16), kp, vp, t(new_cu, torch.int32), t(pos, torch.int32), table, len(lens),
                                       int(np.diff(new_cu).max()), heads, kv, None, scale, **kw)
    close(got, want[rows], BF16_OUT, form)
    if form == "single tokens":                               # the same in chunks side by side and their join
        for tiled in (False, True):
            got = ops.attention_decode_padded(t(wide, torch.bfloat16), kp, vp, t(pos, torch.int32), table, len(lens), max(lens), heads, kv,
                                              None, scale, tiled, **kw)
            close(ops.as_rows(got), want[rows], BF16_OUT, "chunks and join")


def test_which_head_sizes_the_padded_kernels_take(ops):
    fits = lambda *a: ops.padded_attention_fits(torch.bfloat16, *a)
    assert fits(64, 88, 4, 32, True) and fits(128, 256, 16, 32, False) and fits(8, 4, 32, 32, False)
    assert not fits(12, 80, 4, 32, True) and not fits(64, 82, 4, 32, True) and not fits(136, 64, 1, 32, False)
    assert not fits(64, 260, 1, 32, False) and not fits(64, 88, 4, 16, True) and not fits(64, 200, 32, 32, False)
    assert not ops.padded_attention_fits(torch.float32, 64, 88, 4, 32, True)


@pytest.mark.parametrize("dim, vdim", [(64, 88), (128, 128)])
def test_one_far_key_and_the_sink_in_thousands_of_keys(ops, dim, vdim):
    """5,000 keys, more chunks than the short join takes at once; one key 4,968 tokens back answers loudly, at a page's
    border; a query that answers to nothing leaves most of its weight to no key only if the sink counts."""
    rng = np.random.default_rng(12)
    T, heads = 5000, 4
    q, k, v = rng.normal(size=(1, heads, dim)) * 0.2, rng.normal(size=(T, 2, dim)) * 0.2, rng.normal(size=(T, 2, vdim))
    q[0, :2, 5] = 5.0
    k[:, :, 6] = -3.0
    q[0, 2:, 6] = 5.0                                         # two heads whose every score is near -15
    k[31, :, 5] = 5.0
    k[32, :, 5] = -5.0
    q, k, v = bf16_round(q), bf16_round(k), bf16_round(v)
    want = P.capped_attention(q, k, v, T - 1, 1.0, 20.0).reshape(1, -1)
    assert np.abs(want[0, :vdim] - v[31, 0]).max() < 0.1 and np.abs(want[0, 2 * vdim:]).max() < 1e-2
    kp, vp, table = paged_batch(k, v, [T], 3)
    row, pos = t(q.reshape(1, -1), torch.bfloat16), t([T - 1], torch.int32)
    if dim == vdim:
        got = ops.attention_decode_bf16(row, kp, vp, t([0, 1], torch.int32), pos, table, 1, T, heads, 2, dim, None, 1.0, softcap=20.0,
                                        sinks=t(np.zeros(heads)))
    else:
        got = ops.attention_decode_padded(row, kp, vp, pos, table, 1, T, heads, 2, None, 1.0, softcap=20.0, sinks=t(np.zeros(heads)))
    close(got, want, BF16_OUT)


@pytest.mark.parametrize("dim, vdim", [(64, 88), (32, 32), (128, 120)])
@pytest.mark.parametrize("wide", [False, True])
def test_single_tokens_of_many_sequences_walk_their_keys_in_runs_with_a_sink(ops, dim, vdim, wide):
    """As many (sequence, kv head) pairs as make the step stream (with eight wavefronts a workgroup or with four); sequences
    of one key to 150, a cap and the sink."""
    from rust_inference_amd.kernels.build import load
    rng = np.random.default_rng(dim)
    units = load().ri_compute_units()
    kv = 8
    seqs = -(-(units * 9 // 10 if wide else 2 * units) // kv)
    heads = 2 * kv
    lens = [int(n) for n in rng.integers(1, 150, seqs)]
    lens[0] = 1
    if not ops.decode_attention_streams(seqs, kv, max(lens)):
        pytest.skip("this machine's size leaves no such step")
    T = sum(lens)
    q, k, v = (bf16_round(rng.normal(size=(T, n, d))) for n, d in ((heads, dim), (kv, dim), (kv, vdim)))
    cu = np.concatenate([[0], np.cumsum(lens)])
    last = cu[1:] - 1
    want = np.concatenate([P.capped_attention(q[b - 1:b], k[a:b], v[a:b], b - 1 - a, 0.2, 5.0).reshape(1, -1) for a, b in zip(cu[:-1], cu[1:])])
    kp, vp, table = paged_batch(k, v, lens, dim)
    row, pos, sinks = t(q[last].reshape(seqs, -1), torch.bfloat16), t(np.array(lens) - 1, torch.int32), t(np.zeros(heads))
    if dim == vdim:
        got = ops.attention_decode_bf16(row, kp, vp, t(np.arange(seqs + 1), torch.int32), pos, table, seqs, max(lens), heads, kv, dim, None, 0.2,
                                        softcap=5.0, sinks=sinks)
    else:
        got = ops.attention_decode_padded(row, kp, vp, pos, table, seqs, max(lens), heads, kv, None, 0.2, softcap=5.0, sinks=sinks)
    close(got, want, BF16_OUT)


# ---------------------------------------------------------------- the router and the experts
def router_case(seed, tokens, experts, spread=1.0):
    rng = np.random.default_rng(seed)
    return rng.normal(size=(tokens, experts)) * spread, rng.normal(size=experts) * 0.6 - 0.3


@pytest.mark.parametrize("experts, top, count, keep", [(15, 4, 5, 3), (12, 5, 4, 2), (8, 1, 8, 3), (10, 5, 2, 1), (70, 7, 10, 4), (6, 6, 1, 1), (9, 3, 3, 3), (4, 2, 2, 1)])
def test_groups_scored_by_their_two_best(ops, experts, top, count, keep):
    """Choice scores below zero (corrections of either sign), groups of one expert, all groups kept."""
    z, corr = router_case(experts, 200, experts)
    ids, weights, gap = P.route(z, {"router": np.eye(experts), "correction": corr}, "", {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}})
    clear = gap > 1e-5
    assert clear.mean() > 0.95
    got_ids, got_w, dense, _ = ops.experts_route_general(t(z), t(corr), experts, experts, top, ops.ROUTE_SIGMOID, False, count, keep, 2)
    assert (got_ids.cpu().numpy()[clear] == ids[clear]).all()
    close(got_w[torch.tensor(clear, device=got_w.device)], weights[clear], F32)
    full = np.zeros((200, experts))
    np.put_along_axis(full, ids, weights, -1)
    close(dense[torch.tensor(clear, device=dense.device)], full[clear], F32)
    if 1 < experts // count and keep < count and count > 2:   # the best one alone would choose otherwise somewhere
        other = ops.experts_route_general(t(z), t(corr), experts, experts, top, ops.ROUTE_SIGMOID, False, count, keep, 1)[0]
        assert (other.cpu().numpy()[clear] != ids[clear]).any()


def test_a_group_of_two_good_experts_beats_a_group_with_the_best_one(ops):
    z = np.array([[3.0, -4.0, 1.5, 1.5, -4.0, -4.0]])
    ids, w, _, _ = ops.experts_route_general(t(z), t(np.zeros(6)), 6, 6, 2, ops.ROUTE_SIGMOID, False, 3, 1, 2)
    assert ids.cpu().tolist() == [[2, 3]]
    # choice scores below zero in every kept group: still those experts, never one of a group that was left out
    ids, w, _, _ = ops.experts_route_general(t(z), t(np.full(6, -9.0)), 6, 6, 2, ops.ROUTE_SIGMOID, False, 3, 1, 2)
    assert ids.cpu().tolist() == [[2, 3]]
    close(w, 1 / (1 + np.exp(-np.array([[1.5, 1.5]]))), F32)


@pytest.mark.parametrize("tokens, experts, top, ff, dim", [(1, 7, 3, 24, 40), (2, 16, 4, 72, 2056), (3, 8, 2, 16, 512), (1, 5, 1, 520, 8)])
def test_few_tokens_read_the_chosen_experts_alone(ops, tokens, experts, top, ff, dim):
    rng = np.random.default_rng(experts)
    w = {"router": rng.normal(size=(experts, dim)), "correction": rng.normal(size=experts)}
    for e in range(experts):
        w[f"e{e}.up"], w[f"e{e}.down"] = bf16_round(rng.normal(size=(ff, dim)) / dim ** 0.5), bf16_round(rng.normal(size=(dim, ff)) / ff ** 0.5)
    x = bf16_round(rng.normal(size=(tokens, dim)))
    router = {"experts": experts, "top": top}
    ids, weights, _ = P.route(x, w, "", router)
    want = P.moe(x, w, "", {"router": router})
    up = np.concatenate([w[f"e{e}.up"] for e in range(experts)])
    down = np.concatenate([w[f"e{e}.down"] for e in range(experts)], 1)
    got = ops.experts_few_tokens_plain(t(x, torch.bfloat16), t(up, torch.bfloat16), t(down, torch.bfloat16), t(ids, torch.int32), t(weights), ff, "relu2")
    close(got, want, 2e-2)


@pytest.mark.parametrize("activation", ["relu2", "gelu_erf", "gelu_tanh"])
@pytest.mark.parametrize("dtype, ff", [(torch.bfloat16, 24), (torch.bfloat16, 2056), (torch.bfloat16, 21), (torch.float32, 24)])
def test_the_experts_activation_with_and_without_weights(ops, dtype, ff, activation):
    rng = np.random.default_rng(ff)
    tokens, experts = 5, 3
    u = bf16_round(rng.normal(size=(tokens, experts * ff)) * 2)
    dense = np.where(rng.random((tokens, experts + 1)) < 0.5, 0.0, rng.random((tokens, experts + 1)))
    from math import erf
    f = {"relu2": lambda z: np.maximum(z, 0) ** 2, "gelu_erf": lambda z: 0.5 * z * (1 + np.vectorize(erf)(z / 2 ** 0.5)),
         "gelu_tanh": lambda z: 0.5 * z * (1 + np.tanh((2 / np.pi) ** 0.5 * (z + 0.044715 * z ** 3)))}[activation]
    tol = 1e-6 if dtype == torch.float32 else 5e-3
    got = ops.experts_activate_plain(t(u, dtype), t(dense), ff, activation)
    close(got, np.repeat(dense[:, :experts], ff, 1) * f(u), tol)
    close(ops.experts_activate_plain(t(u[:, :ff], dtype), None, ff, activation), f(u[:, :ff]), tol)
