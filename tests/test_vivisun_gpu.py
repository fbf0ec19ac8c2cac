"""Vivisun on the GPU against the plain restatement (oracle/vivisun.py, float64): every kernel alone, then the model through the
engine -- whole prompts, token-by-token decoding, portions down to two tokens, unequal batches, reused pages and slots, long
decoding, loops of every shape, greedy generation through the scheduler, the trace replay command.  Small random configurations made
here; sizes are unlike one another and unlike any shipped model.  Unused cache memory is poisoned with NaN so that a read outside a
sequence's own keys or of a stale state shows."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch

import vivisun_util as U
from oracle import vivisun as O

pytestmark = pytest.mark.gpu
DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(scope="module")
def mops():
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    torch.backends.cuda.matmul.allow_tf32 = False
    from aphrodite_engine_amd import mixer_ops
    return mixer_ops


def dev(a, dtype=torch.float32):
    return torch.from_numpy(np.array(a, dtype=np.float32)).to(DEV).to(dtype)


def rounded(a, dtype):
    return U.bf16_round(a).astype(np.float64) if dtype == torch.bfloat16 else np.asarray(a, np.float32).astype(np.float64)


def f32(a):
    return np.asarray(a, np.float32).astype(np.float64)


def tol_of(dtype):
    return 3e-5 if dtype == torch.float32 else 2e-2


def host(t):
    return t.float().cpu().numpy()


def batch_of(segs, tables, slots, block):
    """segs: [(ctx, tokens)] -> StepBatch"""
    from aphrodite_engine_amd.step_batch import StepBatch
    return StepBatch.build([list(t) for _, t in segs], [c for c, _ in segs], tables, slots, block, DEV)


def run_cut(fn, T, cuts, slot=1, block=16, tables=None):
    """Calls fn(batch, lo, hi) for consecutive portions of one sequence of T tokens."""
    at, out = 0, []
    for n in cuts:
        b = batch_of([(at, [0] * n)], [tables or list(range((T + block - 1) // block))], [slot], block)
        out.append(fn(b, at, at + n))
        at += n
    assert at == T
    return host(torch.cat(out))


def seg(b):
    return b.state_slots, b.q_start, b.q_len, b.ctx_len


def poisoned(*shape, dtype):
    return torch.full(shape, float("nan"), dtype=dtype, device=DEV)


# ---------------------------------------------------------------------------------------------------------------------
# the launch between the layers
# ---------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,width", [(7, 8), (7, 72), (5, 75), (3, 1032), (300, 4096), (1, 8200)])
def test_dynamic_tanh_around_the_residual(mops, dtype, T, width):
    rng = np.random.default_rng(width)
    x = f32(rng.standard_normal((T, width)) * np.exp(rng.uniform(-9, 3, (T, width))))           # tiny to saturating
    ya, yb = (rounded(rng.standard_normal((T, width)), dtype) for _ in range(2))
    table, ids = rounded(rng.standard_normal((11, width)), dtype), rng.integers(0, 11, T)
    W = {}
    for n, a in (("n", 0.7), ("m", 2.25)):
        W[n], W[n + ".b"], W[n + ".alpha"] = rounded(rng.standard_normal(width), dtype), rounded(rng.standard_normal(width), dtype), a
    op = {n: (W[n + ".alpha"], dev(W[n], dtype), dev(W[n + ".b"], dtype)) for n in "nm"}
    wide = lambda y: torch.cat([dev(y, dtype), dev(y, dtype)], 1)[:, :width]                    # rows of a longer buffer
    td, idd = dev(table, dtype), torch.from_numpy(ids).to(DEV)
    tol = tol_of(dtype)
    for names in ("n", "nm", ""):
        for a, b, e, fresh in ((ya, None, None, 0), (ya, yb, None, 0), (ya, None, ids, 0), (None, None, ids, 1), (None, yb, ids, 0), (None, None, None, 0)):
            if not names and a is None and b is None and e is None:
                continue
            new = (0 if fresh else x) + (0 if a is None else a) + (0 if b is None else b) + (0 if e is None else table[ids])
            xd = poisoned(T, width, dtype=torch.float32) if fresh else dev(x)
            before = xd.clone()
            outs = mops.residual_tanh_norm(xd, None if a is None else wide(a), None if b is None else dev(b, dtype), None if e is None else td,
                                           None if e is None else idd, [op[n] for n in names], bool(fresh), dtype=dtype)
            np.testing.assert_allclose(host(xd), new, rtol=2e-6, atol=2e-6)
            if a is None and b is None and e is None:
                assert torch.equal(xd, before)
            assert len(outs) == len(names)
            for n, o in zip(names, outs):
                assert o.dtype == dtype
                np.testing.assert_allclose(host(o), O.dynamic_tanh(new, W, n), rtol=tol / 3, atol=tol / 3)


def test_dynamic_tanh_is_exact_in_fp32_near_zero_and_far_out(mops):
    """tanh keeps its relative accuracy for small arguments and ends at exactly +-1."""
    z = np.concatenate([np.logspace(-12, -1, 40), np.linspace(0.1, 12, 80), [30.0, 1e4, 1e30]])
    x = f32(np.concatenate([z, -z]))[None]
    one, zero = torch.ones(x.shape[1], device=DEV), torch.zeros(x.shape[1], device=DEV)
    got = host(mops.residual_tanh_norm(dev(x), norms=[(1.0, one, zero)])[0])
    np.testing.assert_allclose(got, np.tanh(x), rtol=5e-7)
    assert (np.abs(got[np.abs(x) > 20]) == 1).all()


# ---------------------------------------------------------------------------------------------------------------------
# preparation of queries and keys: convolution, norm, rotation, cache write
# ---------------------------------------------------------------------------------------------------------------------
def prep_case(rng, H, G, d, e, taps, dims, dtype, T, eps, base=300.0, scaling=(3.0, 64, 16.0, 2.0)):
    C = (H + G) * d + G * e
    u, w = rounded(rng.standard_normal((T, C)), dtype), rounded(rng.standard_normal((C, taps)) * 0.3, dtype)
    wq, wk = rounded(1 + rng.standard_normal(d), dtype), rounded(1 + rng.standard_normal(d), dtype)
    sc = scaling and dict(zip(("factor", "original", "fast", "slow"), scaling))
    freq, mag = O.frequencies(dims, base, sc) if dims else (np.zeros(0), 1.0)
    y = O.causal_conv(u, w)
    q, k, v = y[:, :H * d].reshape(T, H, d), y[:, H * d:(H + G) * d].reshape(T, G, d), y[:, (H + G) * d:].reshape(T, G, e)
    q, k = (O.rotate_halves(O.rms_norm(z, n, eps), np.arange(T), freq, mag) for z, n in ((q, wq), (k, wk)))
    return u, w, wq, wk, q.reshape(T, -1), k, v


def gqa(H, G, d, e, taps, dims, dtype, eps, w, wq, wk, base=300.0, scaling=(3.0, 64, 16.0, 2.0)):
    from aphrodite_engine_amd.mixers import GroupedQueryAttention, RotaryFrequencies
    rot = RotaryFrequencies(dims, base, *(scaling or ())) if dims else RotaryFrequencies(0, 1.0)
    m = GroupedQueryAttention(H, G, d, e, d ** -0.5, eps, dtype, qk_norm="head", rotary=rot, taps=taps).to(DEV)
    m.conv.data.copy_(dev(w, dtype))
    m.q_norm.data.copy_(dev(wq, dtype))
    m.k_norm.data.copy_(dev(wk, dtype))
    m.finalize(DEV)
    return m


def prepared(m, mops, kc, vc, state, ud, b, lo, hi):
    """The prepared queries of one portion, by the launch (or the two launches) the mixer takes: attention itself is left out."""
    got = []
    m.attn.attend = lambda out, q, *a: got.append(q.clone())
    m.forward_conv(None, ud[lo:hi], None, (kc, vc), state, b)
    return got[0]


# (heads, kv heads, dim, vdim, taps, rotated): fused sizes with whole and odd halves, partial rotation, none; sizes for the two launches
PREP = [(6, 2, 24, 40, 3, 20), (3, 1, 64, 32, 4, 32), (2, 2, 128, 128, 4, 128), (5, 5, 40, 8, 2, 22), (1, 1, 8, 72, 1, 2), (4, 2, 96, 56, 4, 0),
        (2, 1, 272, 16, 3, 200), (3, 1, 20, 28, 4, 12), (2, 1, 32, 16, 6, 16), (3, 3, 25, 7, 2, 10)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", PREP)
def test_convolution_norm_rotation_and_cache_write_cut_anywhere(mops, dtype, case):
    H, G, d, e, taps, dims = case
    rng = np.random.default_rng(d + taps)
    T, block, eps = 61, 16, 1e-2
    u, w, wq, wk, qw, kw, vw = prep_case(rng, H, G, d, e, taps, dims, dtype, T, eps)
    m = gqa(H, G, d, e, taps, dims, dtype, eps, w, wq, wk)
    fused = d % 8 == 0 and e % 8 == 0 and taps <= 4
    assert mops.conv_rotary_supported(d, e, taps) == fused
    C = m.channels
    pad = -C % 8 + 8
    ud = torch.cat([dev(u, dtype), poisoned(T, pad, dtype=dtype)], 1)[:, :C]                    # rows of a wider product
    pages = (T + block - 1) // block
    tol = 2e-4 if dtype == torch.float32 else (3e-2 if fused else 5e-2)                         # two launches round in between
    for cuts in ([T], [1] * T, [2, 1, 1, 9, 2, 3, 43], [40, 1, 1, 1, 2, 16]):
        table = list(rng.permutation(pages + 3)[:pages])
        kc, vc = poisoned(pages + 3, block, G, d, dtype=dtype), poisoned(pages + 3, block, G, e, dtype=dtype)
        state = poisoned(3, taps - 1, C, dtype=dtype)
        got = run_cut(lambda b, lo, hi: prepared(m, mops, kc, vc, state, ud, b, lo, hi), T, cuts, block=block, tables=table)
        np.testing.assert_allclose(got, qw, rtol=tol, atol=tol, err_msg=str(cuts))
        slots = np.array([table[j // block] * block + j % block for j in range(T)])
        kf, vf = host(kc.view(-1, G, d)), host(vc.view(-1, G, e))
        np.testing.assert_allclose(kf[slots], kw, rtol=tol, atol=tol, err_msg=str(cuts))
        np.testing.assert_allclose(vf[slots], vw, rtol=tol, atol=tol, err_msg=str(cuts))
        rest = np.setdiff1d(np.arange(kf.shape[0]), slots)
        assert np.isnan(kf[rest]).all() and np.isnan(vf[rest]).all()                            # no other row was touched
        if taps > 1:                                                                            # the slot holds the last inputs, no other slot was
            np.testing.assert_array_equal(host(state[1]), u[T - taps + 1:].astype(np.float32))
            assert torch.isnan(state[0]).all() and torch.isnan(state[2]).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", [(6, 2, 24, 40, 3, 20), (3, 1, 64, 32, 4, 64), (3, 1, 20, 28, 4, 12)])
def test_preparation_of_unequal_segments_in_one_step_and_a_slot_taken_over(mops, dtype, case):
    H, G, d, e, taps, dims = case
    rng, eps, block = np.random.default_rng(1), 1e-2, 16
    lens = [37, 1, 22]
    _, w, wq, wk = prep_case(rng, H, G, d, e, taps, dims, dtype, 1, eps)[:4]
    m = gqa(H, G, d, e, taps, dims, dtype, eps, w, wq, wk)
    us = [rounded(rng.standard_normal((n, m.channels)), dtype) for n in lens]
    freq, mag = O.frequencies(dims, 300.0, {"factor": 3.0, "original": 64, "fast": 16.0, "slow": 2.0})
    want = [O.rotate_halves(O.rms_norm(O.causal_conv(u, w)[:, :H * d].reshape(-1, H, d), wq, eps), np.arange(len(u)), freq, mag).reshape(len(u), -1)
            for u in us]
    kc, vc = poisoned(9, block, G, d, dtype=dtype), poisoned(9, block, G, e, dtype=dtype)
    state = poisoned(2, taps - 1, m.channels, dtype=dtype)
    # sequence 1 (one token) ends after the first step and sequence 2 takes its slot; single tokens beside portions, then alone
    plan = [[(0, 5), (1, 1)], [(0, 1), (2, 2)], [(2, 1), (0, 1)], [(0, 1), (2, 1)], [(0, 2), (2, 9)], [(0, 20), (2, 1)], [(2, 8), (0, 7)]]
    slot_of, tables = {0: 1, 1: 0, 2: 0}, {0: [4, 0, 7], 1: [2], 2: [5, 3]}
    at, got = [0, 0, 0], [[], [], []]
    for step in plan:
        b = batch_of([(at[i], [0] * n) for i, n in step], [tables[i] for i, _ in step], [slot_of[i] for i, _ in step], block)
        ud = dev(np.concatenate([us[i][at[i]:at[i] + n] for i, n in step]), dtype)
        q, r = host(prepared(m, mops, kc, vc, state, ud, b, 0, ud.shape[0])), 0
        for i, n in step:
            got[i].append(q[r:r + n])
            r += n
            at[i] += n
    tol = 2e-4 if dtype == torch.float32 else 5e-2
    for i in range(3):
        assert at[i] == lens[i]
        np.testing.assert_allclose(np.concatenate(got[i]), want[i], rtol=tol, atol=tol)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layout_rows", [(64, 32), (20, 12)])
def test_magnitude_factor_of_the_rotation_without_convolution(mops, dtype, layout_rows):
    d, dims = layout_rows
    H, G, e, n, ctx, eps = 3, 1, 16, 9, 1003, 1e-2
    rng = np.random.default_rng(d)
    sc = {"factor": 5.0, "original": 128, "fast": 8.0, "slow": 1.0}
    q, k, v = (rounded(rng.standard_normal((n, h, w)) * 0.3, dtype) for h, w in ((H, d), (G, d), (G, e)))
    wq, wk = rounded(1 + rng.standard_normal(d), dtype), rounded(1 + rng.standard_normal(d), dtype)
    freq, mag = O.frequencies(dims, 700.0, sc)
    qw, kw = (O.rotate_halves(O.rms_norm(z, w, eps), np.arange(ctx, ctx + n), freq, mag) for z, w in ((q, wq), (k, wk)))
    kc, vc = poisoned(64, 16, G, d, dtype=dtype), poisoned(64, 16, G, e, dtype=dtype)
    b = batch_of([(ctx, [0] * n)], [list(range(64))], [0], 16)
    got = mops.rotary_qk_norm_kv_write(*(dev(z.reshape(n, -1), dtype) for z in (q, k, v)), kc, vc, b.slot_mapping, b.q_start, b.ctx_len,
                                       b.seq_of_token, dev(freq), dims, mops.ROTARY_HALF, True, eps, q_weight=dev(wq, dtype),
                                       k_weight=dev(wk, dtype), mscale=mag)
    tol = 3e-4 if dtype == torch.float32 else 3e-2
    np.testing.assert_allclose(host(got), qw.reshape(n, -1), rtol=tol, atol=tol)
    np.testing.assert_allclose(host(kc.view(-1, G, d)[b.slot_mapping]), kw, rtol=tol, atol=tol)


# ---------------------------------------------------------------------------------------------------------------------
# latent attention without a rotated part: sinks, a gate per head
# ---------------------------------------------------------------------------------------------------------------------
def latent_oracle(q, c, scale, sink, gate):
    T, H, R = q.shape
    out = np.stack([O.softmax_attention(q[:, a], c, c, scale, None if sink is None else float(sink[a])) for a in range(H)], 1)
    return out if gate is None else out * O.sigmoid(gate)[:, :, None]


def latent_run(mops, q, c, cuts, dtype, scale, sink=None, gate=None, block=16, seed=0):
    T, H, R = q.shape
    rng = np.random.default_rng(seed)
    pages = (T + block - 1) // block
    table = list(rng.permutation(pages + 4)[:pages])
    cache = poisoned(pages + 4, block, R, dtype=dtype)
    qd, cd = dev(q, dtype), dev(c, dtype)
    gd = None if gate is None else torch.cat([dev(gate, dtype)] * 2, 1)[:, :H]
    sk = None if sink is None else dev(sink)

    def part(b, lo, hi):
        cache.view(-1, R)[b.slot_mapping] = cd[lo:hi]
        out = torch.empty(hi - lo, H, R, dtype=dtype, device=DEV)
        mops.latent_attention(out, qd[lo:hi], None, cache, b.block_tables, b.q_start, b.q_len, b.ctx_len, b.seq_of_token, (hi - lo, hi - lo), None,
                              1.0, 0, scale, max_kv_len=hi, sink=sk, gate=None if gd is None else gd[lo:hi])
        return out
    return run_cut(part, T, cuts, block=block, tables=table)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,R", [(3, 64), (5, 96), (2, 128), (16, 192), (4, 256), (1, 384), (8, 512), (3, 40), (2, 77), (1, 650)])
def test_latent_attention_without_a_rotated_part(mops, dtype, H, R):
    rng = np.random.default_rng(R)
    T, scale = 150, 1.5 * R ** -0.5
    assert mops.latent_attention_fast_supported(R, 0, 0, torch.bfloat16) == (R in (64, 96, 128, 192, 256, 384, 512))
    q, c = rounded(rng.standard_normal((T, H, R)), dtype), rounded(rng.standard_normal((T, R)), dtype)
    gate, sink = rounded(rng.standard_normal((T, H)) * 2, dtype), f32(rng.standard_normal(H) + 2)
    tol = 1e-4 if dtype == torch.float32 else 3e-2
    for kw in ({}, {"gate": gate}, {"sink": sink}, {"gate": gate, "sink": sink}):
        want = latent_oracle(q, c, scale, kw.get("sink"), kw.get("gate"))
        for cuts in ([T], [100] + [1] * 50, [2, 62, 1, 33, 2, 50], [37, 64, 49]):
            np.testing.assert_allclose(latent_run(mops, q, c, cuts, dtype, scale, **kw), want, rtol=tol, atol=tol, err_msg=f"{cuts} {sorted(kw)}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("H,R", [(3, 128), (2, 44)])
def test_one_loud_latent_anywhere_is_found(mops, dtype, decoded, H, R):
    """Among 700 quiet rows one carries a component that the queries pick up: the first token, page borders, tile borders, far and near."""
    T, n = 700, 40
    rng = np.random.default_rng(5)
    for loud in (0, 1, 15, 16, 31, 32, 191, 511, 512, T - n - 1, T - n, T - 5):
        q, c = np.zeros((T, H, R)), rounded(rng.standard_normal((T, R)) * 0.05, dtype)
        q[:, :, 0], c[:, 0] = 8.0, 0.0
        c[loud, 0], c[loud, 1] = 3.0, 30.0
        cuts = [T - n] + [1] * n if decoded else [T - n, 23, 17]
        got = latent_run(mops, q, c, cuts, dtype, 1.0, sink=np.full(H, 2.0), seed=loud)
        tail = np.array([O.softmax_attention(q[i:i + 1, 0], c[loud:loud + 1], c[loud:loud + 1], 1.0)[0, 1] for i in range(T - n, T)])
        for i in range(T - n, T):
            assert (abs(got[i, :, 1] - tail[i - T + n]) < 0.6).all() == (i >= loud), (loud, i)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R", [64, 44])
def test_sink_in_closed_form(mops, dtype, R):
    """Equal scores of 0 leave n / (n + e^sink) of the value; the scale does not touch the sink; the sink counts once, also over splits."""
    H, T = 2, 600
    q, c = np.zeros((T, H, R)), np.ones((T, R))
    sink = np.array([2.0, 5.0])
    n = np.arange(1, T + 1)[:, None]
    for cuts in ([T], [550] + [1] * 50, [1, 1, 2, 596]):
        got = latent_run(mops, q, c, cuts, dtype, 7.0, sink=sink)
        np.testing.assert_allclose(got[:, :, 3], n / (n + np.exp(sink)), rtol=1e-2 if dtype == torch.bfloat16 else 1e-5)


def test_decoded_rows_of_unequal_length_in_one_batch(mops):
    """bf16: decoded rows with 1300, 515, 33 and 2 cached latents side by side, key ranges split over workgroups."""
    dtype, block, scale = torch.bfloat16, 16, 0.1
    rng = np.random.default_rng(3)
    lens = [1300, 515, 33, 2]
    for H, R in ((16, 512), (3, 128), (5, 44)):
        cs, tables, nb = [], [], 0
        for n in lens:
            cs.append(rounded(rng.standard_normal((n, R)), dtype))
            pages = (n + block - 1) // block
            tables.append(list(range(nb, nb + pages)))
            nb += pages
        cache = poisoned(nb, block, R, dtype=dtype)
        for c, tb in zip(cs, tables):
            cache.view(-1, R)[torch.tensor([tb[j // block] * block + j % block for j in range(len(c))], device=DEV)] = dev(c, dtype)
        b = batch_of([(n - 1, [0]) for n in lens], tables, [0, 1, 2, 3], block)
        q, gate, sink = rounded(rng.standard_normal((4, H, R)), dtype), rounded(rng.standard_normal((4, H)), dtype), f32(rng.standard_normal(H) + 3)
        out = torch.empty(4, H, R, dtype=dtype, device=DEV)
        mops.latent_attention(out, dev(q, dtype), None, cache, b.block_tables, b.q_start, b.q_len, b.ctx_len, b.seq_of_token, (1, 1), None, 1.0, 0,
                              scale, max_kv_len=max(lens), sink=dev(sink), gate=dev(gate, dtype))
        for r, (n, c) in enumerate(zip(lens, cs)):
            qq = np.zeros((n, H, R))
            qq[-1] = q[r]
            want = [O.softmax_attention(qq[:, a], c, c, scale, float(sink[a]))[-1] * O.sigmoid(gate[r, a]) for a in range(H)]
            np.testing.assert_allclose(host(out[r]), np.stack(want), rtol=3e-2, atol=3e-2, err_msg=f"{H} {R} {n}")


# ---------------------------------------------------------------------------------------------------------------------
# rotary attention as a whole; the activation into joined rows
# ---------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", [(6, 2, 24, 40, 3, 20), (4, 2, 64, 32, 4, 32), (3, 1, 20, 28, 4, 12), (2, 2, 96, 56, 2, 24)])
def test_one_loud_key_far_back_in_prompts_and_decoded(mops, dtype, case):
    """One token of 400 has a key (after convolution, norm and rotation of none of the numbers it uses) that every query points at: the
    output is its value for every later row and for no earlier one -- the first token, page borders, far and near."""
    H, G, d, e, taps, dims = case
    T, n, eps, block = 400, 40, 1e-4, 16
    rng = np.random.default_rng(7)
    C = (H + G) * d + G * e
    w = np.zeros((C, taps))
    w[:, -1] = 1.0                                                       # the convolution passes the current token
    m = gqa(H, G, d, e, taps, dims, dtype, eps, w, np.full(d, 4.0), np.full(d, 4.0))
    at = dims if dims < d else 0                                         # a number that does not rotate
    gate = np.full((T, H * e), 30.0)
    for loud in (0, 1, 15, 16, 127, 128, 255, T - n - 1, T - n, T - 5):
        u = rng.standard_normal((T, C)) * 0.3
        u[:, :H * d].reshape(T, H, d)[:, :, at] = 20.0
        k = u[:, H * d:(H + G) * d].reshape(T, G, d)
        k[:, :, at] = 0.0
        k[loud, :, at] = 20.0
        u[loud, (H + G) * d:] = 5.0
        u = rounded(u, dtype)
        ud, gd = dev(u, dtype), dev(gate, dtype)
        kc, vc, state = poisoned(25, block, G, d, dtype=dtype), poisoned(25, block, G, e, dtype=dtype), poisoned(2, taps - 1, C, dtype=dtype)
        table = list(rng.permutation(25))

        def part(b, lo, hi):
            out = torch.empty(hi - lo, H * e, dtype=dtype, device=DEV)
            m.forward_conv(out, ud[lo:hi], gd[lo:hi], (kc, vc), state, b)
            return out
        for cuts in ([T - n] + [1] * n, [T - n, 23, 17], [T]):
            got = run_cut(part, T, cuts, block=block, tables=table)
            assert np.isfinite(got).all()
            for i in range(T - n, T):
                assert (np.abs(got[i] - 5.0) < 0.2).all() == (i >= loud), (loud, i, cuts)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(40, 88), (33, 21), (7, 8), (16, )])
def test_joined_output_product(mops, dtype, sizes):
    from aphrodite_engine_amd.mixers import JoinedOutput
    rng = np.random.default_rng(sum(sizes))
    T, width = 5, 24
    j = JoinedOutput(list(sizes), width, dtype).to(DEV)
    ws = [rounded(rng.standard_normal((width, n)), dtype) for n in sizes]
    for i, w in enumerate(ws):
        j.weight_of(i).copy_(dev(w, dtype))
    buf, parts = j.buffer(T, dtype, DEV)
    ys = []
    for n, p in zip(sizes, parts):
        gu = rounded(rng.standard_normal((T, 2 * n)), dtype)
        mops.act_and_mul(dev(gu, dtype), mops.ACT_SILU, p)                # written into its place among the rows
        ys.append(O.silu(gu[:, :n]) * gu[:, n:])
        np.testing.assert_allclose(host(p), ys[-1], rtol=tol_of(dtype) / 2, atol=tol_of(dtype) / 2)
    want = sum(y @ w.T for y, w in zip(ys, ws))
    np.testing.assert_allclose(host(j(buf)), want, rtol=tol_of(dtype) * 2, atol=tol_of(dtype) * 4)


# ---------------------------------------------------------------------------------------------------------------------
# the model through the engine
# ---------------------------------------------------------------------------------------------------------------------
A, L = U.attn_layer, U.latent_layer

CONFIGS = {
    # both mixers, layers that differ in everything, layers without a feed-forward, a span in the middle run three times
    "mixed": lambda: U.make_config([L(), A(), L(heads=5, dim=12, vdim=9, kv_rank=33, scale=0.5, mlp=None),
                                    A(heads=3, kv_heads=3, dim=20, vdim=12, conv=5, rot_dims=12, base=50.0, scaling=None, mlp=U.dense(33)),
                                    A(heads=4, kv_heads=1, dim=16, vdim=24, conv=2, rot_dims=16, mlp=None), L(heads=2, dim=8, vdim=32, kv_rank=64)],
                                   loop=(1, 4, 3)),
    # sizes that the matrix-core kernels serve in bfloat16; the last layers loop
    "wide": lambda: U.make_config([A(heads=6, kv_heads=2, dim=64, vdim=32, conv=4, rot_dims=32, base=1e4, scaling=(4.0, 256, 32.0, 1.0)),
                                   L(heads=8, dim=32, vdim=64, kv_rank=128), A(heads=2, kv_heads=2, dim=128, vdim=128, conv=3, rot_dims=128),
                                   L(heads=3, dim=64, vdim=32, kv_rank=192)], width=128, vocab=211, loop=(2, 4, 2), eps=1e-6),
    # one head everywhere, one tap, no loop at all
    "plain": lambda: U.make_config([A(heads=1, kv_heads=1, dim=40, vdim=24, conv=1, rot_dims=40, scaling=None), L(heads=1, dim=24, vdim=40, kv_rank=40)],
                                   width=96),
    # the whole stack loops, two layers, no convolution
    "whole": lambda: U.make_config([L(heads=2, dim=16, vdim=16, kv_rank=24), A(heads=2, kv_heads=1, dim=16, vdim=16, conv=0, rot_dims=8)], width=64,
                                   loop=(0, 2, 4)),
    # the first layer alone loops
    "first": lambda: U.make_config([A(conv=4, mlp=None), L()], loop=(0, 1, 2)),
    # a loop of one pass
    "once": lambda: U.make_config([L(mlp=None), A()], loop=(0, 2, 1)),
}


def assert_close(got, want, dtype, what=""):
    """float32: every position within 2e-4 of the logits' spread.  bfloat16 against the unrounded restatement: within the rounding of a
    few bfloat16 layers, at every position (no router: nothing jumps)."""
    e = U.logit_errors(got, want)
    assert np.isfinite(e).all(), what
    if dtype == torch.float32:
        assert e.max() < 2e-4, (what, float(e.max()), int(e.argmax()))
    else:
        assert np.median(e) < 0.06 and e.max() < 0.25, (what, float(np.median(e)), float(e.max()), int(e.argmax()))


def poison(eng):
    for c in eng.runner.caches:                   # nothing may be read before it is written
        for t in (c if isinstance(c, (tuple, list)) else [c]):
            t.fill_(float("nan"))


def build(tmp_path, name, dtype, seed=0, weights=None, **engine_args):
    from aphrodite_engine_amd.engine import LLMEngine
    cfg = CONFIGS[name]() if isinstance(name, str) else name
    W = weights or U.make_weights(cfg, seed=seed)
    path = U.write_checkpoint(str(tmp_path / f"m-{seed}"), cfg, W)
    args = dict(max_tokens=512, max_num_seqs=4)
    args.update(engine_args)
    eng = LLMEngine.from_pretrained(path, dtype=dtype, device=DEV, **args)
    poison(eng)
    return cfg, W, eng


def prompts(cfg, lens, seed=0):
    rng = np.random.default_rng(seed)
    return [rng.integers(0, cfg["vocab"], n).tolist() for n in lens]


def in_portions(eng, rid, toks, sizes):
    got, a = [], 0
    for n in sizes:
        got.append(eng.run_segments([(rid, toks[a:a + n], list(range(n)))]))
        a += n
    eng.release(rid)
    assert a == len(toks)
    return host(torch.cat(got))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt_and_layer_trace(mops, tmp_path, name, dtype):
    cfg, W, eng = build(tmp_path, name, dtype)
    toks = prompts(cfg, [83])[0]
    trace = []
    want = O.forward(cfg, W, toks, trace)
    model = eng.runner.model
    model.residual_trace = []
    got = host(eng.run_segments([("a", toks, list(range(len(toks))))]))
    assert_close(got, want, dtype)
    assert len(model.residual_trace) == len(trace) == len(O.layer_order(cfg))
    for x, w in zip(model.residual_trace, trace):
        x = host(x)
        assert np.isfinite(x).all()
        if dtype == torch.float32:
            assert np.abs(x - w).max() < 2e-4 * max(1.0, np.abs(w).max() / 10)
    model.residual_trace = None
    eng.release("a")
    again = host(eng.run_segments([("b", toks, list(range(len(toks))))]))               # reused pages and slot
    assert_close(again, want, dtype)
    eng.release("b")
    some = host(eng.run_segments([("c", toks, [80, 3, 41])]))                           # the last layer runs on the wanted rows only
    assert_close(some, want[[80, 3, 41]], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "wide", "whole"])
def test_portions_and_token_by_token_equal_the_whole_prompt(mops, tmp_path, name, dtype):
    cfg, W, eng = build(tmp_path, name, dtype)
    toks = prompts(cfg, [100], seed=1)[0]
    want = O.forward(cfg, W, toks)
    whole = in_portions(eng, "whole", toks, [100])
    for rid, sizes in (("tok", [1] * 100), ("two", [2] * 50), ("mix", [2, 15, 1, 16, 2, 17, 3, 1, 1, 42]), ("tail", [68] + [1] * 32)):
        got = in_portions(eng, rid, toks, sizes)
        assert_close(got, want, dtype, rid)
        # how a prompt is cut changes nothing beyond rounding -- in bfloat16 too
        assert np.quantile(U.logit_errors(got, whole), 0.9) < (2e-4 if dtype == torch.float32 else 0.08), rid


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_unequal_requests_in_one_batch_equal_each_alone(mops, tmp_path, name, dtype):
    cfg, W, eng = build(tmp_path, name, dtype, max_tokens=320)
    ps = prompts(cfg, [90, 1, 23, 47], seed=2)
    want = [O.forward(cfg, W, p) for p in ps]
    # a schedule with portions beside single tokens; request 1 ends early and request 3 takes its pages and slot; request 2 pauses
    plan = [[(0, 2), (1, 1)], [(0, 30), (2, 3)], [(0, 1), (2, 1), (3, 2)], [(0, 1), (2, 17), (3, 16)], [(2, 1), (3, 1), (0, 1)], [(3, 1), (0, 20)],
            [(3, 27), (0, 1), (2, 1)], [(0, 34)]]
    at, got = [0] * 4, [[] for _ in ps]
    for step in plan:
        entries = [(str(i), ps[i][at[i]:at[i] + n], list(range(n))) for i, n in step]
        out = host(eng.run_segments(entries))
        a = 0
        for i, n in step:
            got[i].append(out[a:a + n])
            a += n
            at[i] += n
            if at[i] == len(ps[i]):
                eng.release(str(i))
    for i in range(4):
        assert at[i] == len(ps[i])
        assert_close(np.concatenate(got[i]), want[i], dtype, i)
    assert eng.pages.num_free == eng.pages.total and eng.slots.num_free == 4


@pytest.mark.parametrize("dtype", DTYPES)
def test_pages_and_slots_taken_over_from_a_finished_request(mops, tmp_path, dtype):
    cfg, W, eng = build(tmp_path, "mixed", dtype, max_tokens=64, max_num_seqs=1)
    a, b = prompts(cfg, [60, 50], seed=3)
    eng.run_segments([("a", a, [])])
    with pytest.raises(Exception):
        eng.run_segments([("b", b, [])])             # neither pages nor a slot are left
    eng.requests.pop("b", None)
    eng.release("a")
    # the new request starts with single tokens in the slot the old one left: no convolution and no key may see a's
    assert_close(in_portions(eng, "b", b, [1, 2, 28, 1, 18]), O.forward(cfg, W, b), dtype)


@pytest.mark.parametrize("kind", ["attention", "latent", "convolution"])
def test_a_marker_token_reaches_exactly_the_rows_that_can_see_it(mops, tmp_path, kind):
    """One layer without a feed-forward: a marker token changes every later row through either attention -- in a prompt and decoded --
    and no earlier one; where the values alone remember (no scores, one key), a convolution of 4 taps reaches three tokens on."""
    if kind == "attention":
        layer = A(heads=2, kv_heads=1, dim=16, vdim=16, rot_dims=8, mlp=None, scale=0.2)
    elif kind == "latent":
        layer = L(heads=2, dim=16, vdim=16, kv_rank=24, mlp=None, scale=0.1)
    else:
        layer = A(heads=2, kv_heads=2, dim=16, vdim=16, conv=4, rot_dims=10, mlp=None, scale=0.2)
    cfg = U.make_config([layer], vocab=50, width=32)
    W = U.make_weights(cfg, seed=7)
    toks = [t if t != 7 else 8 for t in prompts(cfg, [400], seed=8)[0]]
    at = 60
    toks[at] = 7                                     # the marker
    other = list(toks)
    other[at] = 9
    if kind == "convolution":                        # keys and values carry the marker only through the oldest tap
        for n in "kv":
            W[f"l0.mix.{n}.conv"][:, 1:] = 0.0
        W["l0.mix.q.conv"][:, :-1] = 0.0
    want = O.forward(cfg, W, toks)
    _, _, eng = build(tmp_path, cfg, torch.float32, weights=W, max_tokens=1024, max_num_seqs=2)
    for rid, sizes in (("whole", [400]), ("decoded", [at - 5] + [1] * (405 - at)), ("twos", [2] * 200)):
        res = [in_portions(eng, rid, t, sizes) for t in (toks, other)]
        assert_close(res[0], want, torch.float32, rid)
        diff = np.abs(res[0] - res[1]).max(-1)
        assert diff[at] > 1e-3 and diff[:at].max() < 1e-6
        if kind == "convolution":
            assert diff[at + 1:at + 3].max() < 1e-6 and diff[at + 3] > 1e-5
        else:
            assert (diff[at:] > 1e-6).mean() > 0.9


def test_every_pass_of_a_loop_has_caches_of_its_own(mops, tmp_path):
    """The keys of one pass are not those of another: a stack whose single layer loops differs from the same layer run once, and equals
    the layer written out with the embedding added in between -- also when decoded."""
    cfg = U.make_config([A(conv=4)], loop=(0, 1, 3))
    W = U.make_weights(cfg, seed=11)
    toks = prompts(cfg, [70], seed=12)[0]
    want = O.forward(cfg, W, toks)
    once = O.forward(dict(cfg, loop=None), W, toks)
    assert np.median(U.logit_errors(want, once)) > 0.1
    _, _, eng = build(tmp_path, cfg, torch.float32, weights=W)
    assert len(eng.runner.caches) == 6 and len({t.data_ptr() for c in eng.runner.caches for t in (c if isinstance(c, tuple) else (c, ))}) == 9
    for sizes in ([70], [1] * 70, [33, 2, 35]):
        assert_close(in_portions(eng, "a", toks, sizes), want, torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(mops, tmp_path, dtype):
    cfg, W, eng = build(tmp_path, "mixed", dtype)
    toks = prompts(cfg, [180], seed=4)[0]
    want = O.forward(cfg, W, toks)
    got = [eng.run_segments([("a", toks[:5], [4])])]
    for t in toks[5:]:
        got.append(eng.run_segments([("a", [t], [0])]))
    assert_close(host(torch.cat(got)), want[4:], dtype)


def test_decoding_behind_a_long_prompt(mops, tmp_path):
    """bf16, matrix-core sizes: 1100 cached tokens, so that the decoded rows' key ranges are split over workgroups."""
    cfg, W, eng = build(tmp_path, "wide", torch.bfloat16, max_tokens=1152)
    toks = prompts(cfg, [1110], seed=6)[0]
    want = O.forward(cfg, W, toks)
    got = [eng.run_segments([("a", toks[:1098], [0, 511, 1097])])] + [eng.run_segments([("a", [t], [0])]) for t in toks[1098:]]
    assert_close(host(torch.cat(got)), want[[0, 511] + list(range(1097, 1110))], torch.bfloat16)


def test_greedy_generation_through_the_scheduler(mops, tmp_path):
    from aphrodite_engine_amd.engine import SamplingParams
    cfg, W, eng = build(tmp_path, "mixed", torch.float32, max_num_seqs=2, max_num_batched_tokens=24, max_tokens=192)
    ps = prompts(cfg, [40, 3, 1, 29], seed=5)
    outs = eng.generate(ps, SamplingParams(max_tokens=8))
    for p, out in zip(ps, outs):
        seq = list(p)
        for _ in range(8):
            seq.append(int(np.argmax(O.forward(cfg, W, seq)[-1])))
        assert out == seq[len(p):]
    assert eng.pages.num_free == eng.pages.total and eng.slots.num_free == 2 and not eng.requests


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_command_on_an_unseen_shape(mops, tmp_path, dtype):
    """bin/trace_run end to end: a checkpoint of sizes no other test uses, a schedule with portions beside single tokens and a
    request that ends, the logits files against the restatement."""
    cfg = U.make_config([A(heads=8, kv_heads=2, dim=32, vdim=64, conv=2, rot_dims=12, base=900.0, scaling=(2.0, 32, 4.0, 1.0)),
                         L(heads=6, dim=48, vdim=24, kv_rank=104, mlp=None), A(heads=5, kv_heads=5, dim=16, vdim=8, conv=4, rot_dims=16, mlp=U.dense(130)),
                         L(heads=4, dim=32, vdim=16, kv_rank=80)], vocab=300, width=104, eps=1e-4, loop=(1, 4, 2))
    W = U.make_weights(cfg, seed=21)
    model_dir = U.write_checkpoint(str(tmp_path / "m"), cfg, W)
    ps = prompts(cfg, [75, 20, 2], seed=9)
    want = [O.forward(cfg, W, p) for p in ps]
    plan = [[(0, 40), (1, 2)], [(0, 1), (1, 1), (2, 2)], [(0, 20), (1, 17)], [(0, 14)]]
    at, lines, rows = [0, 0, 0], [], []
    for n, step in enumerate(plan):
        entries, end, wanted = [], [], []
        for i, k in step:
            w = list(range(0, k, 2)) if k > 2 else list(range(k))
            entries.append({"id": "q%d" % i, "tokens": ps[i][at[i]:at[i] + k], "want": w})
            wanted += [want[i][at[i] + x] for x in w]
            at[i] += k
            if at[i] == len(ps[i]):
                end.append("q%d" % i)
        rows.append(wanted)
        lines.append(json.dumps({"step": n, "entries": entries, "end": end}))
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", model_dir, "--dtype", dtype, "--out", str(out),
                        "--max-tokens", "128"], input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done %d" % n for n in range(len(plan))]
    got = [np.fromfile(str(out / ("%d.f32" % n)), dtype="<f4").reshape(-1, cfg["vocab"]) for n in range(len(plan))]
    assert [g.shape[0] for g in got] == [len(w) for w in rows]
    assert_close(np.concatenate(got), np.stack([z for w in rows for z in w]), torch.float32 if dtype == "float32" else torch.bfloat16)
