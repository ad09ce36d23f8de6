"""The kernels of the Kisepel design alone, each against the plain function of its mechanism
(tests/plain/kisepel_plain.py), at sizes that are no power of two and differ from one another.

Like tests/test_kernels_gpu.py these run without a GPU when the environment says RI_TEST_KERNELS=emulated
(tests/test_kernels_emulated.py starts that run): the CPU build of the same sources between guard pages."""
import os

import numpy as np
import pytest
import torch

from plain import kisepel_plain as P

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


def rounded(a, dtype):
    return bf16_round(a) if dtype == torch.bfloat16 else np.asarray(a)


F32 = 3e-6
BF16_OUT = 7.5e-3


# ---------------------------------------------------------------- q/k norm, scaled rotation in halves, the cache write
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads, kv, dim, vdim, rot, factor", [(6, 2, 24, 40, 16, 3.0), (3, 3, 20, 12, 10, 1.0), (4, 1, 64, 88, 64, 8.0), (2, 2, 9, 7, 0, 1.0),
                                                               (5, 5, 136, 16, 48, 0.5), (2, 1, 130, 130, 130, 2.0), (2, 1, 520, 8, 16, 4.0)])
@pytest.mark.parametrize("form", ["prompts", "single tokens", "portions"])
def test_norm_rotation_in_halves_and_the_cache_write(ops, form, heads, kv, dim, vdim, rot, factor, dtype):
    rng = np.random.default_rng(heads * dim)
    lens = [1, 1, 1] if form == "single tokens" else [45, 1, 70]
    starts = [0, 0, 0] if form == "prompts" else [33, 5, 64]
    T, width, lead, eps = sum(lens), heads * dim + kv * (dim + vdim), 8, 1e-3
    proj = rng.normal(size=(T, lead + width)) * rng.uniform(0.05, 4.0, size=(T, 1))
    proj = rounded(proj, dtype)
    q_gain, k_gain = 1 + 0.3 * rng.normal(size=dim), 1 + 0.3 * rng.normal(size=dim)
    pos, seq, cu = [], [], [0]
    for b, (n, s) in enumerate(zip(lens, starts)):
        pos += list(range(s, s + n))
        seq += [b] * n
        cu.append(len(pos))
    pages, base = 17, 300.0
    table = rng.permutation(pages)[:15].reshape(3, 5)
    kp, vp = t(np.full((pages, kv, PAGE, dim), 7.0), dtype), t(np.full((pages, kv, vdim, PAGE), 7.0), dtype)
    freq = base ** (-2.0 * np.arange(rot // 2) / max(rot, 1)) / factor
    turn = lambda x: P.rotate_halves(x, np.array(pos, dtype=np.float64), rot, base, factor)
    full = proj[:, lead:]
    want_q = turn(P.rms_unit(full[:, :heads * dim].reshape(T, heads, dim), eps) * q_gain)
    want_k = turn(P.rms_unit(full[:, heads * dim:(heads + kv) * dim].reshape(T, kv, dim), eps) * k_gain)
    want_v = full[:, (heads + kv) * dim:].reshape(T, kv, vdim)
    row = t(proj, dtype)
    ops.qk_half_bias_kv_write(row, lead, lead + heads * dim, lead + (heads + kv) * dim, None, t(freq) if rot else None, 1.0,
                              t(pos, torch.int32), t(seq, torch.int32), t(table, torch.int32), kp, vp, heads, kv, dim, vdim,
                              t(cu, torch.int32), max(lens), t(q_gain), t(k_gain), eps)
    tol = 3e-5 if dtype == torch.float32 else BF16_OUT        # (an angle near 130 in float32: 1e-5)
    close(row[:, :lead], proj[:, :lead], 1e-7, "the columns ahead")
    close(row[:, lead:lead + heads * dim], want_q.reshape(T, -1), tol, "q")
    want_kp, want_vp = np.full(kp.shape, 7.0), np.full(vp.shape, 7.0)
    for i in range(T):
        page, at = table[seq[i], pos[i] // PAGE], pos[i] % PAGE
        want_kp[page, :, at], want_vp[page, :, :, at] = want_k[i], want_v[i]
    close(kp, want_kp, tol, "the key pages, where nothing was written too")
    close(vp, want_vp, tol, "the value pages")


def test_the_scaled_frequencies_are_divided():
    from rust_inference_amd.parts import PartSpec, build_part
    part = build_part("position", PartSpec("rotate_half", {"head_dim": 10, "theta": 50.0, "dims": 6, "factor": 4.0}))
    assert np.allclose(part.part_frequencies().numpy(), [0.25, 0.25 * 50.0 ** (-1 / 3), 0.25 * 50.0 ** (-2 / 3)], rtol=1e-14)


# ---------------------------------------------------------------- attention in chunks of the sequence
def paged_batch(k, v, lens, seed, dtype, first_seen=None):
    """Keys and values of several sequences in pages handed out in shuffled order; pages that lie wholly before
    ``first_seen[b]`` are not mapped, and what is in the pool beside is loud."""
    G, dk, dv = k.shape[1], k.shape[2], v.shape[2]
    width = max(-(-n // PAGE) for n in lens) + 1
    n_pages = sum(-(-n // PAGE) for n in lens) + 2
    order = np.random.default_rng(seed).permutation(n_pages)
    table = np.full((len(lens), width), -1, dtype=np.int32)
    kp = torch.full((n_pages, G, PAGE, dk), 3.0, dtype=dtype)
    vp = torch.full((n_pages, G, dv, PAGE), 50.0, dtype=dtype)
    nxt = at = 0
    for b, n in enumerate(lens):
        for p in range((first_seen[b] // PAGE) if first_seen is not None else 0, -(-n // PAGE)):
            table[b, p] = order[nxt]
            nxt += 1
        for j in range(n):
            page = table[b, j // PAGE]
            if page >= 0:
                kp[page, :, j % PAGE] = torch.tensor(k[at + j]).to(dtype)
                vp[page, :, :, j % PAGE] = torch.tensor(v[at + j]).to(dtype)
        at += n
    return guarded(kp.to(DEV)), guarded(vp.to(DEV)), t(table, torch.int32)


def chunk_case(rng, lens, heads, kv, dim, vdim, scale, size, dtype):
    T = sum(lens)
    q, k, v = (rounded(rng.normal(size=(T, n, d)), dtype) for n, d in ((heads, dim), (kv, dim), (kv, vdim)))
    cu = np.concatenate([[0], np.cumsum(lens)])
    want = np.concatenate([P.attention_core(q[a:b], k[a:b], v[a:b], 0, size, scale).reshape(b - a, -1) for a, b in zip(cu[:-1], cu[1:])])
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


CHUNKS = [1, 7, 31, 32, 33, 64, 100, 256, 1000]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads, kv, dim, vdim", [(6, 2, 24, 40), (3, 3, 16, 8), (2, 1, 9, 7)])
@pytest.mark.parametrize("size", CHUNKS)
def test_generic_attention_in_chunks(ops, size, heads, kv, dim, vdim, dtype):
    rng = np.random.default_rng(heads * 10 + size)
    lens = [75, 1, 290] if dim == 24 else [66, 33]
    q, k, v, cu, want = chunk_case(rng, lens, heads, kv, dim, vdim, 0.31, size, dtype)
    for tail in (None, 1):
        rows, pos, new_cu = rows_of(lens, cu, tail)
        if tail is None and dim == 24 and EMULATED:
            rows, pos = rows[::5], pos[::5]
        seen = [pos[a] // size * size for a in new_cu[:-1]] if tail == 1 else None
        kp, vp, table = paged_batch(k, v, lens, dim, dtype, seen)
        seq = np.searchsorted(cu, rows, side="right") - 1
        got = ops.attention(t(q[rows].reshape(len(rows), -1), dtype), kp, vp, t(pos, torch.int32), t(seq, torch.int32), table, heads, kv,
                            dim, None, 0.31, chunk=size)
        close(got, want[rows], F32 if dtype == torch.float32 else BF16_OUT, f"last {tail}")


@pytest.mark.parametrize("heads, kv, dim, vdim", [(4, 2, 64, 64), (8, 1, 128, 128), (6, 3, 96, 96), (4, 2, 24, 40), (2, 2, 32, 32), (3, 1, 72, 200)])
@pytest.mark.parametrize("size", CHUNKS)
@pytest.mark.parametrize("form", ["prompts", "single tokens", "portions"])
def test_matrix_core_attention_in_chunks(ops, form, size, heads, kv, dim, vdim):
    """bfloat16: prompts of unequal lengths, one new token each, the last tokens of each as a portion that crosses a chunk's
    edge; pages before the first token's chunk are not mapped."""
    rng = np.random.default_rng(dim + heads + size)
    lens = [75, 1, 140] if form == "prompts" else [300, 33, 65]
    scale = 2.0 / dim ** 0.5
    q, k, v, cu, want = chunk_case(rng, lens, heads, kv, dim, vdim, scale, size, torch.bfloat16)
    rows, pos, new_cu = rows_of(lens, cu, {"prompts": None, "single tokens": 1, "portions": 19}[form])
    kp, vp, table = paged_batch(k, v, lens, dim, torch.bfloat16, [pos[a] // size * size for a in new_cu[:-1]])
    wide = t(np.concatenate([np.full((len(rows), 16), 9.0), q[rows].reshape(len(rows), -1), np.full((len(rows), 8), 9.0)], 1), torch.bfloat16)
    kw, seqs, most = {"q_off": 16, "chunk": size}, len(lens), int(np.diff(new_cu).max())
    cu_t, pos_t = t(new_cu, torch.int32), t(pos, torch.int32)
    equal = dim == vdim and dim in ops.MFMA_HEAD_DIMS
    if ops.padded_attention_fits(torch.bfloat16, dim, vdim, heads // kv, PAGE, False):
        got = ops.attention_prefill_padded(wide, kp, vp, cu_t, pos_t, table, seqs, most, heads, kv, None, scale, **kw)
        close(got, want[rows], BF16_OUT, form)
    if equal:
        got = ops.attention_prefill_bf16(wide, kp, vp, cu_t, pos_t, table, seqs, most, heads, kv, dim, None, scale, **kw)
        close(got, want[rows], BF16_OUT, form + ", equal heads")
    if form != "single tokens":
        return
    got = ops.attention_decode_padded(wide, kp, vp, pos_t, table, seqs, max(lens), heads, kv, None, scale, **kw)
    close(got, want[rows], BF16_OUT, "chunks of keys and join")
    if equal:
        got = ops.attention_decode_bf16(wide, kp, vp, cu_t, pos_t, table, seqs, max(lens), heads, kv, dim, None, scale, **kw)
        close(got, want[rows], BF16_OUT, "chunks of keys and join, equal heads")


@pytest.mark.parametrize("dim, vdim", [(64, 64), (64, 88)])
@pytest.mark.parametrize("size", [48, 64, 1000])
def test_single_tokens_of_many_sequences_walk_their_chunk_in_runs(ops, size, dim, vdim):
    """As many (sequence, kv head) pairs as make the step stream; sequences of one key to 150."""
    from rust_inference_amd.kernels.build import load
    rng = np.random.default_rng(dim + size)
    kv = 8
    seqs = max(4, -(-2 * load().ri_compute_units() // kv))
    heads = 2 * kv
    lens = [int(n) for n in rng.integers(1, 150, seqs)]
    lens[0], lens[1], lens[2] = 1, 97, 96                     # one past a chunk's edge, and its last token
    if not ops.decode_attention_streams(seqs, kv, max(lens)):
        pytest.skip("this machine's size leaves no such step")
    q, k, v, cu, want = chunk_case(rng, lens, heads, kv, dim, vdim, 0.2, size, torch.bfloat16)
    rows, pos, _ = rows_of(lens, cu, 1)
    kp, vp, table = paged_batch(k, v, lens, dim, torch.bfloat16, [p // size * size for p in pos])
    row, pos_t = t(q[rows].reshape(seqs, -1), torch.bfloat16), t(pos, torch.int32)
    if dim == vdim:
        got = ops.attention_decode_bf16(row, kp, vp, t(np.arange(seqs + 1), torch.int32), pos_t, table, seqs, max(lens), heads, kv, dim, None,
                                        0.2, chunk=size)
    else:
        got = ops.attention_decode_padded(row, kp, vp, pos_t, table, seqs, max(lens), heads, kv, None, 0.2, chunk=size)
    close(got, want[rows], BF16_OUT)


@pytest.mark.parametrize("dim, vdim", [(64, 88), (128, 128)])
def test_one_loud_key_at_a_chunks_edge_among_thousands(ops, dim, vdim):
    """4,000 keys in chunks of 1,500; the first key of the query's chunk answers loudly, the one before it louder still."""
    rng = np.random.default_rng(12)
    T, heads, size = 4000, 4, 1500
    q, k, v = rng.normal(size=(1, heads, dim)) * 0.2, rng.normal(size=(T, 2, dim)) * 0.2, rng.normal(size=(T, 2, vdim))
    q[..., 5] = 5.0
    k[3000, :, 5], k[2999, :, 5] = 5.0, 9.0
    q, k, v = bf16_round(q), bf16_round(k), bf16_round(v)
    want = P.attention_core(q, k, v, T - 1, size, 1.0).reshape(1, -1)
    assert np.abs(want[0, :vdim] - v[3000, 0]).max() < 0.1
    kp, vp, table = paged_batch(k, v, [T], 3, torch.bfloat16)
    row, pos = t(q.reshape(1, -1), torch.bfloat16), t([T - 1], torch.int32)
    if dim == vdim:
        got = ops.attention_decode_bf16(row, kp, vp, t([0, 1], torch.int32), pos, table, 1, T, heads, 2, dim, None, 1.0, chunk=size)
    else:
        got = ops.attention_decode_padded(row, kp, vp, pos, table, 1, T, heads, 2, None, 1.0, chunk=size)
    close(got, want, BF16_OUT)


def test_a_window_and_chunks_are_refused_together(ops):
    from rust_inference_amd.errors import KernelError
    z = t(np.zeros((1, 24)))
    with pytest.raises(KernelError, match="chunks of 4 beside a window of 3"):
        ops.attention(z, t(np.zeros((1, 1, PAGE, 8))), t(np.zeros((1, 1, 8, PAGE))), t([0], torch.int32), t([0], torch.int32),
                      t([[0]], torch.int32), 1, 1, 8, 3, 1.0, chunk=4)


# ---------------------------------------------------------------- the delta rule with a decay per key channel
def delta_case(rng, T, H, G, dk, dv, K, lead):
    """The projection's rows: ``lead`` columns of something else, q, k, v, and behind them H logits of beta."""
    C = 2 * G * dk + H * dv
    return {"C": C, "proj": rng.normal(size=(T, lead + C + H)), "taps": rng.normal(size=(C, K)) * 0.5, "z": rng.normal(size=(T, H * dk + H * dv + 4)),
            "a_log": rng.normal(size=H) * 0.7 - 0.5, "dt_bias": rng.normal(size=H * dk) * 0.7}


def lay_gates(ops, g, beta):
    """[decays | betas | what pads a row]."""
    T, H, dk = g.shape
    return t(np.concatenate([g.reshape(T, -1), beta, np.full((T, ops.delta_gate_row(H, dk) - H * dk - H), 7.0)], 1))


def plain_prepare(c, H, G, dk, dv, lens, tails, lead):
    """q, k, v, gates of the sequences one after the other; ``tails`` are moved on in place."""
    rows, gates, at, C = [], [], 0, c["C"]
    for b, n in enumerate(lens):
        state = {"x": tails[b]}
        y = P.silu(P.short_conv(c["proj"][at:at + n, lead:lead + C], c["taps"], None, state, "x"))
        tails[b] = state["x"]
        q = P.unit(y[:, :G * dk].reshape(n, G, dk)) * dk ** -0.5
        k = P.unit(y[:, G * dk:2 * G * dk].reshape(n, G, dk))
        rows.append(np.concatenate([q.reshape(n, -1), k.reshape(n, -1), y[:, 2 * G * dk:]], 1))
        g = P.decays(c["z"][at:at + n, :H * dk], c["a_log"], c["dt_bias"])
        gates.append(np.concatenate([g.reshape(n, -1), P.sigmoid(c["proj"][at:at + n, lead + C:])], 1))
        at += n
    return np.concatenate(rows), np.concatenate(gates)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, G, dk, dv, K, lens", [(4, 2, 12, 20, 3, (1, 7, 3)), (2, 1, 64, 48, 4, (45, 1)), (3, 3, 5, 70, 1, (2, 18)), (4, 4, 32, 32, 2, (9, 1, 5)),
                                                   (2, 2, 16, 300, 6, (20,)), (1, 1, 256, 4, 4, (3, 2, 1)), (6, 2, 4, 36, 4, (700, 400)), (300, 1, 8, 1, 3, (2,))])
def test_delta_prepare_with_a_decay_per_channel(ops, dtype, H, G, dk, dv, K, lens):
    rng = np.random.default_rng(H * 7 + dk)
    T, lead = sum(lens), 8
    if EMULATED and T > 1000:
        lens, T = (600, 430), 1030
    c = delta_case(rng, T, H, G, dk, dv, K, lead)
    c["proj"] = rounded(c["proj"], dtype)
    slots = [3, 0, 4][:len(lens)]
    tails = rng.normal(size=(5, K - 1, c["C"]))
    plain_tails = [tails[s].copy() for s in slots]
    want_qkv, want_gates = plain_prepare(c, H, G, dk, dv, lens, plain_tails, lead)
    cu, seq = np.concatenate([[0], np.cumsum(lens)]), np.repeat(np.arange(len(lens)), lens)
    dev_tails, proj = t(tails), t(c["proj"], dtype)
    qkv, gates = ops.delta_prepare_channels(proj, lead, t(c["taps"]), dev_tails, t(c["z"]), proj, lead + c["C"], t(c["a_log"]), t(c["dt_bias"]),
                                            t(seq, torch.int32), t(cu, torch.int32), t(slots, torch.int32), H, G, dk, dv)
    close(qkv, want_qkv, F32, "q, k, v")
    assert gates.shape[1] == ops.delta_gate_row(H, dk)
    close(gates[:, :H * dk + H], want_gates, F32, "gates")
    for s, want in zip(slots, plain_tails):
        if K > 1:
            close(dev_tails[s], want, 1e-7, "tail")
    untouched = [s for s in range(5) if s not in slots]
    assert np.array_equal(f64(dev_tails[untouched]), tails[untouched].astype(np.float32).astype(np.float64))


WALKS = [(4, 2, 12, 20, (1, 7, 3)), (2, 1, 64, 48, (45,)), (3, 3, 5, 70, (2, 18)), (2, 2, 100, 33, (17, 1)), (1, 1, 256, 40, (20,)), (2, 1, 130, 64, (9, 24)),
         (6, 6, 8, 8, (40, 3)), (3, 1, 16, 12, (8, 7, 9)), (2, 2, 200, 10, (25,))]


@pytest.mark.parametrize("H, G, dk, dv, lens", WALKS)
@pytest.mark.parametrize("slices", [0, 4, 8, 16])
def test_delta_walk_with_a_decay_per_channel(ops, H, G, dk, dv, lens, slices):
    rng = np.random.default_rng(H * 11 + dk)
    T = sum(lens)
    if slices == 16 and (dk % 4 or H * dv % 4):
        pytest.skip("sixteen slices take heads in 16-byte pieces")
    q, k, v = P.unit(rng.normal(size=(T, G, dk))) * dk ** -0.5, P.unit(rng.normal(size=(T, G, dk))), rng.normal(size=(T, H, dv))
    g, beta = rng.uniform(0.3, 1.0, size=(T, H, dk)), rng.uniform(0.1, 1.0, size=(T, H))
    slots = [2, 0, 3][:len(lens)]
    state = rng.normal(size=(4, H, dk, dv))
    want_state, want, at = state.copy(), [], 0
    for b, n in enumerate(lens):
        want.append(P.delta_walk(q[at:at + n], k[at:at + n], v[at:at + n], beta[at:at + n], g[at:at + n], want_state[slots[b]]))
        at += n
    qkv = np.concatenate([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], 1)
    cu = np.concatenate([[0], np.cumsum(lens)])
    dev_state = t(state)
    got = ops.delta_scan_channels(t(qkv), lay_gates(ops, g, beta), dev_state, t(cu, torch.int32), t(slots, torch.int32),
                                  H, G, dk, dv, slices)
    close(got, np.concatenate(want).reshape(T, -1), 1e-5, "outputs")
    close(dev_state, want_state, 1e-5, "state")


@pytest.mark.parametrize("slices", [4, 8, 16])
def test_the_walk_token_by_token_is_the_walk_in_blocks(ops, slices):
    """The same 37 tokens in one step, and one at a time from the state the step before left: the same bits."""
    rng = np.random.default_rng(5)
    H, G, dk, dv, T = 2, 1, 24, 40, 37
    q, k = P.unit(rng.normal(size=(T, G, dk))) * dk ** -0.5, P.unit(rng.normal(size=(T, G, dk)))
    qkv = np.concatenate([q.reshape(T, -1), k.reshape(T, -1), rng.normal(size=(T, H * dv))], 1)
    gates = lay_gates(ops, rng.uniform(0.3, 1.0, size=(T, H, dk)), rng.uniform(0.1, 1.0, size=(T, H)))
    one, slot = t(np.zeros((2, H, dk, dv))), t([1], torch.int32)
    whole = ops.delta_scan_channels(t(qkv), gates, one, t([0, T], torch.int32), slot, H, G, dk, dv, slices)
    two = t(np.zeros((2, H, dk, dv)))
    rows = [ops.delta_scan_channels(t(qkv[i:i + 1]), t(f64(gates[i:i + 1])), two, t([0, 1], torch.int32), slot, H, G, dk, dv, slices) for i in range(T)]
    assert torch.equal(torch.cat([r.cpu() for r in rows]), whole.cpu()) and torch.equal(one.cpu(), two.cpu())


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, G, dk, dv, K", [(4, 2, 12, 20, 3), (2, 1, 64, 48, 4), (3, 3, 5, 72, 1), (2, 2, 128, 128, 4), (1, 1, 256, 64, 2), (2, 2, 40, 256, 7)])
def test_one_step_of_the_delta_rule_with_a_decay_per_channel(ops, dtype, H, G, dk, dv, K):
    assert ops.delta_step_fits(dk, dv)
    rng = np.random.default_rng(H * 13 + dv)
    B, lead, eps = 3, 16, 1e-4
    c = delta_case(rng, B, H, G, dk, dv, K, lead)
    c["proj"] = rounded(c["proj"], dtype)
    slots = [3, 0, 4]
    tails, state, gain = rng.normal(size=(5, K - 1, c["C"])), rng.normal(size=(5, H, dk, dv)) * 0.3, 1 + 0.1 * rng.normal(size=dv)
    plain_tails = [tails[s].copy() for s in slots]
    qkv, gates = plain_prepare(c, H, G, dk, dv, [1] * B, plain_tails, lead)
    want_state, want = state.copy(), []
    for b in range(B):
        o = P.delta_walk(qkv[b:b + 1, :G * dk].reshape(1, G, dk), qkv[b:b + 1, G * dk:2 * G * dk].reshape(1, G, dk),
                         qkv[b:b + 1, 2 * G * dk:].reshape(1, H, dv), gates[b:b + 1, H * dk:], gates[b:b + 1, :H * dk].reshape(1, H, dk),
                         want_state[slots[b]])
        want.append((P.rms_unit(o[0], eps) * gain).reshape(-1) * P.sigmoid(c["z"][b, H * dk + 4:]))
    proj, z, dev_tails, dev_state = t(c["proj"], dtype), t(c["z"]), t(tails), t(state)
    got = ops.delta_step_channels(proj, lead, t(c["taps"]), dev_tails, z, H * dk + 4, proj, lead + c["C"], t(c["a_log"]), t(c["dt_bias"]), dev_state,
                                  t(np.arange(B + 1), torch.int32), t(slots, torch.int32), t(gain), eps, H, G, dk, dv)
    close(got, np.stack(want), 2e-5 if dtype == torch.float32 else BF16_OUT, "outputs")
    close(dev_state, want_state, 1e-5, "state")
    for s, w in zip(slots, plain_tails):
        if K > 1:
            close(dev_tails[s], w, 1e-7, "tail")


@pytest.mark.parametrize("act, gate_dtype", [(torch.float32, torch.float32), (torch.bfloat16, torch.float32), (torch.bfloat16, torch.bfloat16)])
@pytest.mark.parametrize("heads, vdim", [(3, 64), (5, 20), (2, 7), (1, 512)])
@pytest.mark.parametrize("kind", ["sigmoid", "silu"])
def test_heads_normed_and_gated(ops, kind, heads, vdim, act, gate_dtype):
    rng = np.random.default_rng(vdim)
    T, off = 9, 8
    o, gate, gain = rng.normal(size=(T, heads, vdim)), rounded(rng.normal(size=(T, off + heads * vdim + 8)) * 2, gate_dtype), 1 + 0.2 * rng.normal(size=vdim)
    act_of = P.sigmoid if kind == "sigmoid" else P.silu
    want = (P.rms_unit(o, 1e-3) * gain).reshape(T, -1) * act_of(gate[:, off:off + heads * vdim])
    got = ops.head_norm_gate(t(o.reshape(T, -1)), t(gate, gate_dtype), off, t(gain), 1e-3, heads, vdim, act, ops.GATE_SIGMOID if kind == "sigmoid" else ops.GATE_SILU)
    close(got, want, F32 if act == torch.float32 else BF16_OUT)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("row, col, width, T", [(64, 16, 24, 5), (37, 3, 11, 70), (20, 0, 20, 1), (24, 20, 4, 3)])
def test_columns_taken_out_of_wider_rows(ops, dtype, row, col, width, T):
    x = rounded(np.random.default_rng(row).normal(size=(T, row)), dtype)
    close(ops.take_columns(t(x, dtype), col, width), x[:, col:col + width], 1e-7)


# ---------------------------------------------------------------- sums of branches with their norms
@pytest.mark.parametrize("dim", [36, 51, 1028, 2052, 4100, 8200])
@pytest.mark.parametrize("a_parts, b_parts", [(1, 1), (5, 2), (1, 9)])
def test_two_normed_branches_added(ops, dim, a_parts, b_parts):
    rng = np.random.default_rng(dim + a_parts)
    T, eps = 3, 1e-2
    a, b = rng.normal(size=(a_parts, T, dim)), rng.normal(size=(b_parts, T, dim)) * 3
    a[:, 1] *= 1e-2                                           # a row whose norm eps shows in
    ga, gb, gc = (1 + 0.3 * rng.normal(size=dim) for _ in range(3))
    first = 0.5 * P.rms_unit(a.sum(0), eps) * ga
    both = first + 0.25 * P.rms_unit(b.sum(0), eps) * gb
    lay = lambda y: t(y if y.shape[0] > 1 else y[0])
    close(ops.normed_sum([lay(a)], [t(ga)], [0.5], eps), first, F32, "one")
    close(ops.normed_sum([lay(a), lay(b)], [t(ga), t(gb)], [0.5, 0.25], eps), both, F32, "two")
    c = bf16_round(rng.normal(size=(T, dim)))
    got = ops.normed_sum([lay(a), lay(b), t(c, torch.bfloat16)], [t(ga), t(gb), t(gc)], [0.5, 0.25, 2.0], eps)
    close(got, both + 2.0 * P.rms_unit(c, eps) * gc, F32, "three, one of them bfloat16")


@pytest.mark.parametrize("act", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("dim", [36, 51, 1028, 2052, 4100, 8200])
@pytest.mark.parametrize("parts", [(1,), (1, 3), (2, 12, 1), (30, 1, 1)])
def test_branches_that_wait_and_the_norm(ops, parts, dim, act):
    rng = np.random.default_rng(dim + sum(parts))
    T, eps = 4, 1e-3
    x, ys, gain = rng.normal(size=(T, dim)), [rng.normal(size=(p, T, dim)) for p in parts], 1 + 0.3 * rng.normal(size=dim)
    new = x + sum(y.sum(0) for y in ys)
    branches = [t(y if y.shape[0] > 1 else y[0]) for y in ys]
    res = t(x)
    rows = [2, 0]
    some = ops.add_branches_rmsnorm(res, branches, t(gain), eps, act, t(rows, torch.int32))
    close(res, x, 1e-7, "nothing is written back for chosen rows")
    close(some, P.rms_unit(new[rows], eps) * gain, F32 if act == torch.float32 else BF16_OUT, "chosen rows")
    got = ops.add_branches_rmsnorm(res, branches, t(gain), eps, act)
    close(res, new, F32, "the residual")
    close(got, P.rms_unit(new, eps) * gain, F32 if act == torch.float32 else BF16_OUT, "the norm")


def test_more_parts_than_the_kernel_adds_are_refused(ops):
    from rust_inference_amd.errors import ShapeError
    y = t(np.zeros((ops.MAX_BRANCH_PARTS + 1, 1, 8)))
    with pytest.raises(ShapeError, match="parts of branches"):
        ops.add_branches_rmsnorm(t(np.zeros((1, 8))), [y], t(np.ones(8)), 1e-5, torch.float32)


# ---------------------------------------------------------------- experts by a table
@pytest.mark.parametrize("vocab, experts, top, T", [(40, 7, 3, 9), (11, 1, 1, 4), (300, 130, 70, 5), (64, 4, 4, 70)])
def test_experts_by_a_table_of_token_ids(ops, vocab, experts, top, T):
    rng = np.random.default_rng(vocab)
    table = np.stack([rng.permutation(experts)[:top] for _ in range(vocab)])
    toks = rng.integers(0, vocab, T)
    toks[0] = vocab - 1
    ids, weights, dense = ops.experts_by_table(t(table, torch.int32), t(toks, torch.int32), experts)
    assert np.array_equal(f64(ids), table[toks]) and np.allclose(f64(weights), 1.0 / top, rtol=1e-6)
    want = np.zeros((T, experts))
    for i, tok in enumerate(toks):
        want[i, table[tok]] = 1.0 / top
    close(dense, want, 1e-6)
    assert ops.experts_by_table(t(table, torch.int32), t(toks, torch.int32), experts, dense=False)[2] is None


def test_a_shared_expert_without_a_gate_is_added_as_it_is(ops):
    rng = np.random.default_rng(3)
    for dim in (48, 50):
        routed, shared = rng.normal(size=(3, 5, dim)), rng.normal(size=(2, 5, dim))
        close(ops.experts_finish(t(routed), None, t(shared), None), routed.sum(0) + shared.sum(0), F32)
