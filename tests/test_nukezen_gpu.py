"""Nukezen on the GPU against the plain restatement (oracle/nukezen.py, float64): every kernel alone, then the model through the
engine -- whole prompts, token-by-token decoding, portions down to two tokens, unequal batches, reused pages and slots, long
decoding past every window and chunk, greedy generation through the scheduler, the trace replay command.  Small random
configurations made here; sizes are unlike one another and unlike any shipped model.  Unused cache memory is poisoned with NaN so
that a read outside a sequence's own keys or of a stale state shows."""
import json
import os
import subprocess

import numpy as np
import pytest
import torch

import nukezen_util as U
from oracle import nukezen as O

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
    return torch.from_numpy(np.ascontiguousarray(a, dtype=np.float32)).to(DEV).to(dtype)


def rounded(a, dtype):
    return U.bf16_round(a).astype(np.float64) if dtype == torch.bfloat16 else np.asarray(a, np.float32).astype(np.float64)


def f32(a):
    return np.asarray(a, np.float32).astype(np.float64)


def tol_of(dtype):
    return 3e-5 if dtype == torch.float32 else 2e-2


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
    return torch.cat(out).float().cpu().numpy()


def seg(b):
    return b.state_slots, b.q_start, b.q_len, b.ctx_len


# ---------------------------------------------------------------------------------------------------------------------
# residual, embedding
# ---------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [8, 72, 75, 1032, 4096])
def test_post_norm_residual(mops, dtype, width):
    rng = np.random.default_rng(width)
    T, eps = 7, 1e-3
    x = f32(rng.standard_normal((T, width)))
    y = rounded(rng.standard_normal((T, width)) * 0.05, dtype)                    # small: eps matters
    post, pre = rounded(rng.standard_normal(width), dtype), rounded(rng.standard_normal(width), dtype)
    new = x + O.rms_norm(y, post, eps)
    for yv in (dev(y, dtype), torch.cat([dev(y, dtype), dev(y, dtype)], 1)[:, :width]):     # dense rows, and a view of longer ones
        xd = dev(x)
        got = mops.residual_post_rms_norm(xd, yv, dev(post, dtype), eps=eps)
        np.testing.assert_allclose(xd.cpu().numpy(), new, rtol=2e-5, atol=2e-5)
        np.testing.assert_allclose(got.float().cpu().numpy(), new, rtol=tol_of(dtype), atol=tol_of(dtype))
    xd = dev(x)
    got = mops.residual_post_rms_norm(xd, dev(y, dtype), dev(post, dtype), dev(pre, dtype), eps)
    np.testing.assert_allclose(xd.cpu().numpy(), new, rtol=2e-5, atol=2e-5)
    np.testing.assert_allclose(got.float().cpu().numpy(), O.rms_norm(new, pre, eps), rtol=tol_of(dtype), atol=tol_of(dtype))
    before = xd.clone()                                                            # the norm alone leaves the residual as it is
    got = mops.residual_post_rms_norm(xd, pre=dev(pre, dtype), eps=eps)
    assert torch.equal(xd, before)
    np.testing.assert_allclose(got.float().cpu().numpy(), O.rms_norm(new, pre, eps), rtol=tol_of(dtype), atol=tol_of(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
def test_scaled_embedding_and_its_rounded_copy(mops, dtype):
    rng = np.random.default_rng(0)
    table, ids = rounded(rng.standard_normal((50, 72)), dtype), rng.integers(0, 50, 13)
    copy = torch.empty(13, 72, dtype=dtype, device=DEV)
    x = mops.embed_scale(dev(table, dtype), torch.from_numpy(ids).to(DEV), 5.5, copy=copy)
    np.testing.assert_allclose(x.cpu().numpy(), table[ids] * 5.5, rtol=1e-6)
    assert torch.equal(copy, x.to(dtype))


# ---------------------------------------------------------------------------------------------------------------------
# the recurrences
# ---------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps,channels", [(4, 64), (3, 52), (1, 24), (6, 40), (2, 48)])
def test_short_convolution_with_bias_cut_anywhere(mops, dtype, taps, channels):
    rng = np.random.default_rng(taps)
    T = 45
    u, w, bias = (rounded(rng.standard_normal(s), dtype) for s in ((T, channels), (channels, taps), (channels, )))
    want = O.silu(O.causal_conv(u, w, bias))
    state = torch.full((3, max(taps - 1, 0), channels), float("nan"), dtype=dtype, device=DEV)
    ud, wd, bd = dev(u, dtype), dev(w, dtype), dev(bias, dtype)

    def part(b, lo, hi):
        return mops.short_conv(ud[lo:hi], wd, state, *seg(b), b.seq_of_token, channels, act=1, bias=bd)
    for cuts in ([T], [1] * T, [2, 1, 1, 9, 2, 30], [40, 1, 1, 1, 2]):
        np.testing.assert_allclose(run_cut(part, T, cuts), want, rtol=tol_of(dtype), atol=tol_of(dtype))


SCAN_CUTS = ([90], [1] * 90, [2] * 45, [40, 1, 1, 33, 2, 13], [3, 50, 1, 36])      # both work splits write what the other reads


def delta_inputs(rng, T, H, G, d, e, dtype):
    q, k = rounded(rng.standard_normal((T, G, d)), dtype), rounded(rng.standard_normal((T, G, d)), dtype)
    v, b = rounded(rng.standard_normal((T, H, e)), dtype), rounded(rng.standard_normal((T, H)) * 2, dtype)
    a = rounded(rng.standard_normal((T, H, d)) * 2, dtype)
    return q, k, v, b, a


def delta_oracle(q, k, v, b, a, a_log, dt_bias):
    H, G, d = v.shape[1], q.shape[1], q.shape[2]
    qn, kn = O.unit(q) * d ** -0.5, O.unit(k)
    beta, g = O.sigmoid(b), np.exp(-np.exp(a_log)[None, :, None] * O.softplus(a + dt_bias))
    return np.stack([O.channel_delta_rule(qn[:, h // (H // G)], kn[:, h // (H // G)], v[:, h], beta[:, h], g[:, h]) for h in range(H)], 1)


def delta_run(mops, t, state, b, max_len, H, G, d, a_log, dt_bias):
    return mops.gated_delta_scan(*t, a_log, dt_bias, state, *seg(b), H, G, d ** -0.5, 1e-6, max_q_len=max_len)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,e", [(4, 2, 24, 40), (3, 3, 64, 64), (2, 1, 100, 72), (6, 2, 16, 130), (1, 1, 200, 8), (5, 5, 1, 24)])
def test_channel_delta_rule_in_segments_of_every_size(mops, dtype, H, G, d, e):
    rng = np.random.default_rng(H * 100 + d)
    T = 90
    q, k, v, b, a = delta_inputs(rng, T, H, G, d, e, dtype)
    a_log, dt_bias = f32(np.log(rng.uniform(0.05, 2.0, H))), f32(rng.standard_normal((H, d)) - 1)
    want = delta_oracle(q, k, v, b, a, a_log, dt_bias).reshape(T, H * e)
    t = [dev(z.reshape(T, -1), dtype) for z in (q, k, v, b, a)]
    state = torch.full((3, H, d, e), float("nan"), dtype=torch.float32, device=DEV)       # poison: a first portion must not read it
    la, ld = dev(a_log), dev(dt_bias.reshape(-1))
    for cuts in SCAN_CUTS:
        got = run_cut(lambda bt, lo, hi: delta_run(mops, [z[lo:hi] for z in t], state, bt, hi - lo, H, G, d, la, ld), T, cuts)
        np.testing.assert_allclose(got, want, rtol=2e-4, atol=2e-4)       # inputs are rounded alike on both sides; the recurrence is fp32


def test_channel_delta_decays_every_key_channel_at_its_own_rate(mops):
    """Values written under two orthogonal keys, one key channel that forgets at once and one that never does."""
    d, e = 8, 4
    keys, vals = np.eye(d)[[0, 1, 2, 2]] * 2.0, np.arange(4.0 * e).reshape(4, e) + 1
    q = np.eye(d)[[0, 1, 0, 1]]
    a = np.full((4, d), -60.0)                                   # softplus -> 0: keeps
    a[:, 1] = 60.0                                               # channel 1 forgets
    state = torch.zeros(1, 1, d, e, device=DEV)
    b = batch_of([(0, [0] * 4)], [[0]], [0], 16)
    out = mops.gated_delta_scan(dev(q), dev(keys), dev(vals), dev(np.full((4, 1), 30.0)), dev(a), dev(np.zeros(1)), dev(np.zeros(d)), state,
                                *seg(b), 1, 1, 1.0, 1e-6, max_q_len=4).cpu().numpy()
    np.testing.assert_allclose(out[0], vals[0], atol=1e-4)
    np.testing.assert_allclose(out[1], vals[1], atol=1e-4)       # the current token's write is read before it is forgotten
    np.testing.assert_allclose(out[2], vals[0], atol=1e-4)
    np.testing.assert_allclose(out[3], 0 * vals[0], atol=1e-4)


def ssm_inputs(rng, T, H, G, N, e, dtype):
    return (rounded(rng.standard_normal((T, H, e)), dtype), rounded(rng.standard_normal((T, G, N)), dtype),
            rounded(rng.standard_normal((T, G, N)), dtype), rounded(rng.standard_normal((T, H)) * 2, dtype))


def ssm_oracle(x, B, C, dt, dt_bias, a_log, D):
    H, G = x.shape[1], B.shape[1]
    step = O.softplus(dt + dt_bias)
    return np.stack([O.state_space(x[:, h], B[:, h // (H // G)], C[:, h // (H // G)], step[:, h], a_log[h], D[h]) for h in range(H)], 1)


def ssm_run(mops, t, state, b, max_len, H, G, a_log, dt_bias, D):
    x, B, C, dt = t
    return mops.outer_memory_scan(C, B, x, (state, ), *seg(b), H, mops.MEMORY_STATE_SPACE, gate_i=dt, max_q_len=max_len, qk_heads=G,
                                  a_log=a_log, dt_bias=dt_bias, skip=D)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,N,e", [(6, 3, 20, 12), (4, 1, 64, 64), (3, 3, 100, 72), (8, 2, 16, 130), (1, 1, 200, 8), (2, 1, 128, 64)])
def test_state_space_in_segments_of_every_size(mops, dtype, H, G, N, e):
    rng = np.random.default_rng(H * 100 + N)
    T = 90
    data = ssm_inputs(rng, T, H, G, N, e, dtype)
    a_log, dt_bias, D = f32(np.log(rng.uniform(0.02, 2.0, H))), f32(rng.standard_normal(H) - 1), f32(rng.standard_normal(H))
    want = ssm_oracle(*data, dt_bias, a_log, D).reshape(T, H * e)
    t = [dev(z.reshape(T, -1), dtype) for z in data]
    state = torch.full((3, H, N, e), float("nan"), dtype=torch.float32, device=DEV)
    la, lb, ld = dev(a_log), dev(dt_bias), dev(D)
    for cuts in SCAN_CUTS:
        got = run_cut(lambda bt, lo, hi: ssm_run(mops, [z[lo:hi] for z in t], state, bt, hi - lo, H, G, la, lb, ld), T, cuts)
        np.testing.assert_allclose(got, want, rtol=2e-4, atol=2e-4 * max(1.0, np.abs(want).max() / 4))


@pytest.mark.parametrize("kind", ["delta", "state_space"])
@pytest.mark.parametrize("lens", [[50, 1, 7], [300, 1, 130]])
def test_recurrences_in_a_batch_of_unequal_segments_and_a_slot_taken_over(mops, kind, lens):
    rng = np.random.default_rng(5)
    H, G, d, e, dtype = 4, 2, 32, 48, torch.float32
    make = delta_inputs if kind == "delta" else ssm_inputs
    data = [make(rng, n, H, G, d, e, dtype) for n in lens]
    a_log, skip = f32(np.log(rng.uniform(0.05, 1.0, H))), f32(rng.standard_normal(H))
    dt_bias = f32(rng.standard_normal((H, d) if kind == "delta" else H))
    want = [(delta_oracle(*x, a_log, dt_bias) if kind == "delta" else ssm_oracle(*x, dt_bias, a_log, skip)).reshape(n, H * e)
            for x, n in zip(data, lens)]
    state = torch.full((2, H, d, e), float("nan"), dtype=torch.float32, device=DEV)
    # sequence 1 (one token) ends after the first step and sequence 2 takes its slot
    n0, n2 = lens[0], lens[2]
    plan = [[(0, 20), (1, 1)], [(0, 1), (2, 3)], [(2, 1), (0, n0 - 23)], [(2, n2 - 4), (0, 2)]]
    slot_of, at, got = {0: 1, 1: 0, 2: 0}, [0, 0, 0], [[], [], []]
    for step in plan:
        b = batch_of([(at[i], [0] * n) for i, n in step], [list(range(8))] * len(step), [slot_of[i] for i, _ in step], 64)
        t = [dev(np.concatenate([data[i][j][at[i]:at[i] + n].reshape(n, -1) for i, n in step])) for j in range(len(data[0]))]
        longest = max(n for _, n in step)
        if kind == "delta":
            out = delta_run(mops, t, state, b, longest, H, G, d, dev(a_log), dev(dt_bias.reshape(-1)))
        else:
            out = ssm_run(mops, t, state, b, longest, H, G, dev(a_log), dev(dt_bias), dev(skip))
        r = 0
        for i, n in step:
            got[i].append(out[r:r + n].cpu().numpy())
            r += n
            at[i] += n
    for i in range(3):
        assert at[i] == lens[i]
        np.testing.assert_allclose(np.concatenate(got[i]), want[i], rtol=3e-4, atol=3e-4)


def test_state_space_with_fast_and_slow_decays_over_a_long_prompt(mops):
    """700 tokens, heads that keep everything (a write at the first token is still read at the last) and heads that forget within a
    token, in one launch and cut."""
    H, G, N, e, T = 4, 2, 16, 8, 700
    rng = np.random.default_rng(9)
    x, B, C, dt = ssm_inputs(rng, T, H, G, N, e, torch.float32)
    dt = np.clip(dt, -3, 3)
    x[0] *= 50.0
    a_log, dt_bias, D = f32([-9.0, 4.0, -2.0, 1.0]), f32(np.zeros(H) - 1), f32(np.zeros(H))
    want = ssm_oracle(x, B, C, dt, dt_bias, a_log, D).reshape(T, H * e)
    t = [dev(z.reshape(T, -1)) for z in (x, B, C, dt)]
    state = torch.full((2, H, N, e), float("nan"), dtype=torch.float32, device=DEV)
    scale = np.abs(want).max(0)
    for cuts in ([T], [64, 65, 63, 1, 1, 506], [333, 367]):
        got = run_cut(lambda bt, lo, hi: ssm_run(mops, [z[lo:hi] for z in t], state, bt, hi - lo, H, G, dev(a_log), dev(dt_bias), dev(D)), T, cuts)
        assert (np.abs(got - want) / scale).max() < 1e-4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,parts", [(72, 4), (72, 1), (75, 5), (2048, 2), (96, 96)])
def test_gate_before_the_norm_in_parts(mops, dtype, n, parts):
    rng = np.random.default_rng(n)
    T = 9
    x = f32(rng.standard_normal((T, n)) * 0.01)                                    # small: eps matters
    z, w = rounded(rng.standard_normal((T, n)), dtype), rounded(rng.standard_normal(n), dtype)
    want = O.rms_norm((x * O.silu(z)).reshape(T, parts, -1), None, 1e-5).reshape(T, n) * w * 1.3
    out = torch.empty(T, n + 8, dtype=dtype, device=DEV)[:, :n]
    mops.silu_gate_part_rms_norm(out, dev(x), dev(z, dtype), dev(w, dtype), parts, 1e-5, 1.3)
    np.testing.assert_allclose(out.float().cpu().numpy(), want, rtol=tol_of(dtype), atol=tol_of(dtype) * 3)


# ---------------------------------------------------------------------------------------------------------------------
# preparation of queries and keys
# ---------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,e,dims", [(3, 1, 20, 28, 12), (2, 2, 40, 72, 40), (3, 1, 130, 8, 16), (4, 2, 64, 32, 24), (2, 1, 24, 8, 0)])
def test_head_norm_with_weights_before_the_rotation(mops, dtype, H, G, d, e, dims):
    from aphrodite_engine_amd.mixers import RotaryFrequencies
    rng = np.random.default_rng(d)
    ctx, n, block, eps, base = 1003, 9, 16, 1e-2, 700.0
    q, k, v = (rounded(rng.standard_normal((n, h, w)) * 0.3, dtype) for h, w in ((H, d), (G, d), (G, e)))
    wq, wk = rounded(1 + rng.standard_normal(d), dtype), rounded(1 + rng.standard_normal(d), dtype)
    pos = np.arange(ctx, ctx + n)
    qw, kw = (O.rotate_neighbours(O.rms_norm(z, w, eps), pos, dims, base) for z, w in ((q, wq), (k, wk)))
    pages = (ctx + n + block - 1) // block
    table = list(rng.permutation(pages + 3)[:pages])
    kc = torch.full((pages + 3, block, G, d), float("nan"), dtype=dtype, device=DEV)
    vc = torch.full((pages + 3, block, G, e), float("nan"), dtype=dtype, device=DEV)
    b = batch_of([(ctx, [0] * n)], [table], [0], block)
    rf = RotaryFrequencies(dims, base).to(DEV)
    got = mops.rotary_qk_norm_kv_write(dev(q.reshape(n, -1), dtype), dev(k.reshape(n, -1), dtype), dev(v.reshape(n, -1), dtype), kc, vc,
                                       b.slot_mapping, b.q_start, b.ctx_len, b.seq_of_token, rf.inv_freq, dims, mops.ROTARY_INTERLEAVED,
                                       True, eps, q_weight=dev(wq, dtype), k_weight=dev(wk, dtype))
    tol = 3e-4 if dtype == torch.float32 else 3e-2               # fp32 angles at position 1000
    np.testing.assert_allclose(got.float().cpu().numpy(), qw.reshape(n, -1), rtol=tol, atol=tol)
    slots = b.slot_mapping.cpu().numpy()
    kf, vf = kc.view(-1, G, d).float().cpu().numpy(), vc.view(-1, G, e).float().cpu().numpy()
    np.testing.assert_allclose(kf[slots], kw, rtol=tol, atol=tol)
    np.testing.assert_array_equal(vf[slots], v.astype(np.float32))
    rest = np.setdiff1d(np.arange(kf.shape[0]), slots)
    assert np.isnan(kf[rest]).all() and np.isnan(vf[rest]).all()           # no other row was touched


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,e", [(6, 2, 24, 16), (3, 1, 25, 7), (16, 16, 128, 128), (40, 8, 128, 64), (36, 2, 256, 8), (1, 1, 8, 8)])
def test_norm_over_the_whole_projection_and_cache_write(mops, dtype, H, G, d, e):
    rng = np.random.default_rng(d + H)
    n, block, eps = 5, 16, 1e-2
    q, k, v = (rounded(rng.standard_normal((n, w)) * 0.3, dtype) for w in (H * d, G * d, G * e))
    q[:, :d] *= 4.0                                               # one loud head: the statistic is the row's, not the head's
    wq, wk = rounded(rng.standard_normal(H * d), dtype), rounded(rng.standard_normal(G * d), dtype)
    kc = torch.full((4, block, G, d), float("nan"), dtype=dtype, device=DEV)
    vc = torch.full((4, block, G, e), float("nan"), dtype=dtype, device=DEV)
    b = batch_of([(14, [0] * n)], [[2, 0]], [0], block)
    proj = dev(np.concatenate([q, k, v, np.zeros((n, 8 + (-(q.shape[1] + k.shape[1] + v.shape[1])) % 8))], 1), dtype)    # rows of one product
    nq, nk, nv = H * d, G * d, G * e
    got = mops.qk_row_norm_kv_write(proj[:, :nq], proj[:, nq:nq + nk], proj[:, nq + nk:nq + nk + nv], kc, vc, b.slot_mapping, dev(wq, dtype),
                                    dev(wk, dtype), eps)
    np.testing.assert_allclose(got.float().cpu().numpy(), O.rms_norm(q, wq, eps), rtol=tol_of(dtype), atol=tol_of(dtype))
    slots = b.slot_mapping.cpu().numpy()
    kf, vf = kc.view(-1, nk).float().cpu().numpy(), vc.view(-1, nv).float().cpu().numpy()
    np.testing.assert_allclose(kf[slots], O.rms_norm(k, wk, eps), rtol=tol_of(dtype), atol=tol_of(dtype))
    np.testing.assert_array_equal(vf[slots], v.astype(np.float32))
    rest = np.setdiff1d(np.arange(kf.shape[0]), slots)
    assert np.isnan(kf[rest]).all() and np.isnan(vf[rest]).all()


# ---------------------------------------------------------------------------------------------------------------------
# attention: window, chunks, soft cap, distance bias, sink, gates
# ---------------------------------------------------------------------------------------------------------------------
def attention_oracle(q, k, v, scale, window=0, chunk=0, softcap=0.0, rel=None, far=0, sink=None, gate=None):
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    see, out = O.visible(T, window, chunk), np.zeros((T, H, v.shape[2]))
    dist = np.maximum(np.arange(T)[:, None] - np.arange(T)[None, :], 0)
    row_of = np.array([O.distance_bucket(n, rel.shape[0], far) for n in range(T)]) if rel is not None else None
    for a in range(H):
        bias = rel[row_of[dist], a] if rel is not None else None
        out[:, a] = O.softmax_attention(q[:, a], k[:, a // (H // G)], v[:, a // (H // G)], scale, see, softcap, bias,
                                        None if sink is None else float(sink[a]))
    out = out.reshape(T, -1)
    return out if gate is None else out * O.sigmoid(gate)


def attend(mops, q, k, v, cuts, dtype, scale, block=16, seed=0, rel=None, far=0, gate=None, sink=None, **kw):
    """Runs one sequence cut into portions over shuffled, poisoned pages; returns [T, H * e]."""
    from aphrodite_engine_amd.mixers import DistanceBiasAttention
    T, H, d = q.shape
    G, e = k.shape[1], v.shape[2]
    rng = np.random.default_rng(seed)
    pages = (T + block - 1) // block
    table = list(rng.permutation(pages + 4)[:pages])
    kc = torch.full((pages + 4, block, G, d), float("nan"), dtype=dtype, device=DEV)
    vc = torch.full((pages + 4, block, G, e), float("nan"), dtype=dtype, device=DEV)
    lut = None
    if rel is not None:
        m = DistanceBiasAttention(H, G, d, e, scale, bias_rows=rel.shape[0], bias_far=far).to(DEV)
        m.rel.data.copy_(dev(rel))
        m.finalize()
        lut = m.bias_lut
    qd, kd, vd = dev(q.reshape(T, -1), dtype), dev(k.reshape(T, -1), dtype), dev(v.reshape(T, -1), dtype)
    gd = dev(gate, dtype) if gate is not None else None
    sk = dev(sink) if sink is not None else None

    def part(b, lo, hi):
        mops.paged_kv_write(kc, vc, kd[lo:hi], vd[lo:hi], b.slot_mapping)
        out = torch.empty(hi - lo, H * e, dtype=dtype, device=DEV)
        mops.distance_bias_attention(out, qd[lo:hi], gd[lo:hi] if gd is not None else None, kc, vc, b.block_tables, b.q_start, b.q_len,
                                     b.ctx_len, b.seq_of_token, (hi - lo, hi - lo), H, scale, lut, max_kv_len=hi, sink=sk, **kw)
        return out
    return run_cut(part, T, cuts, block=block, tables=table)


# (heads, kv heads, dim, vdim): odd sizes; matrix-core sizes with 1, 2, 3, 5 and 8 query heads per kv head
SHAPES = [(6, 2, 24, 16), (3, 1, 20, 28), (4, 2, 64, 32), (3, 1, 32, 96), (10, 2, 128, 32), (8, 1, 64, 128), (2, 2, 96, 64), (3, 3, 136, 8)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("mask", [{"window": 17}, {"window": 64}, {"window": 1}, {"window": 500}, {"chunk": 21}, {"chunk": 64}, {"chunk": 1}, {}])
def test_masked_attention_in_portions_and_decoded(mops, dtype, shape, mask):
    H, G, d, e = shape
    rng = np.random.default_rng(d + sum(mask.values()))
    T, scale = 150, d ** -0.5
    q, k, v = (rounded(rng.standard_normal((T, h, w)) * s, dtype) for h, w, s in ((H, d, 2.0), (G, d, 1.0), (G, e, 1.0)))
    gate = rounded(rng.standard_normal((T, H * e)), dtype)
    sink = f32(rng.standard_normal(H))
    rel = f32(rng.standard_normal((11, H)))
    tol = 3e-4 if dtype == torch.float32 else 3e-2
    for kw in ({"gate": gate}, {"sink": sink, "softcap": 2.5, "rel": rel, "far": 40}, {"softcap": 1.5, "gate": gate, "sink": np.zeros(H)}):
        want = attention_oracle(q, k, v, scale, **mask, **kw)
        for cuts in ([T], [100] + [1] * 50, [2, 62, 1, 33, 2, 50], [37, 64, 49]):
            got = attend(mops, q, k, v, cuts, dtype, scale, **mask, **kw)
            np.testing.assert_allclose(got, want, rtol=tol, atol=tol, err_msg=f"{cuts} {sorted(kw)}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("shape", [(3, 1, 20, 28), (4, 2, 64, 32)])
@pytest.mark.parametrize("mask", [{"window": 37}, {"chunk": 49}, {"window": 64}, {"chunk": 64}])
def test_one_loud_key_just_inside_and_just_outside(mops, dtype, decoded, shape, mask):
    """Among 340 quiet keys one carries a component that the queries pick up: a row's output is that key's value exactly while the
    window (the chunk) holds the key -- its edges, page borders, the first token."""
    H, G, d, e = shape
    T, n = 340, 60
    rng = np.random.default_rng(11)
    size = sum(mask.values())
    inside = T - n + 20
    places = [0, 15, 16, 191, T - n - size + 1, T - n - size, T - n - size + 15, T - 5] if "window" in mask else \
        [0, 191, inside // size * size - 1, inside // size * size, inside // size * size + 1, T - 5]
    for loud in sorted({p for p in places if p >= 0}):
        q, k = np.zeros((T, H, d)), rounded(rng.standard_normal((T, G, d)) * 0.05, dtype)
        v = rounded(rng.standard_normal((T, G, e)) * 0.05, dtype)
        q[:, :, 0], k[:, :, 0] = 8.0, 0.0
        k[loud, :, 0], v[loud, :, 0] = 3.0, 30.0
        cuts = [T - n] + [1] * n if decoded else [T - n, 33, 27]
        got = attend(mops, q, k, v, cuts, dtype, 1.0, seed=loud, **mask)
        want = attention_oracle(q, k, v, 1.0, **mask)
        tol = 3e-4 if dtype == torch.float32 else 3e-2
        np.testing.assert_allclose(got[T - n:], want[T - n:], rtol=tol, atol=tol, err_msg=str(loud))
        for i in range(max(loud, T - n), T):
            seen = i - loud < size if "window" in mask else i // size == loud // size
            assert (abs(got[i, 0] - 30.0) < 0.5) == seen, (loud, i)


@pytest.mark.parametrize("dtype", DTYPES)
def test_sink_of_score_zero_and_soft_cap_bounds(mops, dtype):
    """A first token alone with score s leaves e^s / (1 + e^s) of its value; the cap bounds a huge score before the bias is added."""
    H, G, d, e = 2, 1, 64, 32
    q, k, v = np.zeros((3, H, d)), np.zeros((3, G, d)), np.ones((3, G, e))
    q[:, :, 0], k[:, :, 0] = 4.0, 8.0
    for cuts in ([3], [1, 1, 1]):
        got = attend(mops, q * 0, k, v, cuts, dtype, 1.0, sink=np.zeros(H), chunk=2)
        np.testing.assert_allclose(got[:, 0], [1 / 2, 2 / 3, 1 / 2], atol=4e-3)       # the third row starts a chunk: one key
        rel = np.full((4, H), -5.0)
        got = attend(mops, q, k, v, cuts, dtype, 1.0, sink=np.zeros(H), chunk=1, softcap=5.0, rel=rel, far=8)
        np.testing.assert_allclose(got[:, 0], np.full(3, 0.5), atol=4e-3)             # 5 tanh(32 / 5) - 5 = 0


def test_decoded_rows_of_unequal_length_in_one_batch(mops):
    """bf16: decoded rows with 1100, 515 and 3 keys side by side, under masks whose visible ranges are split over workgroups."""
    dtype = torch.bfloat16
    rng = np.random.default_rng(3)
    lens, block, scale = [1100, 515, 3], 16, 0.13
    for H, G, d, e in ((8, 4, 64, 64), (3, 1, 128, 64), (5, 1, 64, 32)):
        for kw in ({"window": 50}, {"window": 600}, {"chunk": 512}, {"chunk": 1050, "softcap": 3.0}, {}):
            seqs, tables, nb = [], [], 0
            for n in lens:
                seqs.append([rounded(rng.standard_normal((n, h, w)), dtype) for h, w in ((H, d), (G, d), (G, e))])
                pages = (n + block - 1) // block
                tables.append(list(range(nb, nb + pages)))
                nb += pages
            kc = torch.full((nb, block, G, d), float("nan"), dtype=dtype, device=DEV)
            vc = torch.full((nb, block, G, e), float("nan"), dtype=dtype, device=DEV)
            for (q, k, v), tb in zip(seqs, tables):
                idx = torch.tensor([tb[j // block] * block + j % block for j in range(len(k))], device=DEV)
                kc.view(-1, G, d)[idx], vc.view(-1, G, e)[idx] = dev(k, dtype), dev(v, dtype)
            b = batch_of([(n - 1, [0]) for n in lens], tables, [0, 1, 2], block)
            sink = f32(rng.standard_normal(H))
            out = torch.empty(3, H * e, dtype=dtype, device=DEV)
            mops.distance_bias_attention(out, dev(np.stack([s[0][-1].reshape(-1) for s in seqs]), dtype), None, kc, vc, b.block_tables, b.q_start,
                                         b.q_len, b.ctx_len, b.seq_of_token, (1, 1), H, scale, None, max_kv_len=max(lens), sink=dev(sink), **kw)
            for r, (q, k, v) in enumerate(seqs):
                n = len(k)
                see = O.visible(n, kw.get("window", 0), kw.get("chunk", 0))[-1:]
                want = [O.softmax_attention(q[-1:, a], k[:, a // (H // G)], v[:, a // (H // G)], scale, see, kw.get("softcap", 0.0), None,
                                            float(sink[a]))[0] for a in range(H)]
                np.testing.assert_allclose(out[r].float().cpu().numpy(), np.concatenate(want), rtol=3e-2, atol=3e-2, err_msg=f"{kw} {r}")


# ---------------------------------------------------------------------------------------------------------------------
# the model through the engine
# ---------------------------------------------------------------------------------------------------------------------
D, A, P = U.delta_layer, U.attn_layer, U.par_layer


def mixed_config():
    """Every mixer kind, layers that differ in everything, layers without a feed-forward, tensors shared within every kind (and by a
    layer that follows another sharer)."""
    ls = [P(mlp=None), D(), A(), P(heads=4, kv_heads=2, dim=16, vdim=8, window=40, rot_dims=16, base=50.0, left_scale=1.4, right_scale=0.5,
                                   s_heads=5, s_vdim=8, state=12, groups=1, norm_groups=1, conv=2), A(heads=2, kv_heads=2, chunk=34, softcap=3.0, mlp=None)]
    ls += [U.same_as(ls, 0), U.same_as(ls, 2), U.same_as(ls, 1), D(heads=3, kv_heads=3, dim=16, vdim=24, conv=1, mlp=None)]
    return U.make_config(ls + [dict(U.same_as(ls, 3), weights_of=3)])


CONFIGS = {
    "mixed": mixed_config,
    # sizes that the matrix-core kernels serve in bfloat16; fewer rotated numbers than the head has
    "wide": lambda: U.make_config([P(heads=6, kv_heads=2, dim=64, vdim=32, window=45, rot_dims=32, s_heads=4, s_vdim=32, state=64, groups=2,
                                     norm_groups=2, conv=3), D(heads=4, kv_heads=4, dim=64, vdim=32, conv=4),
                                   A(heads=5, kv_heads=1, dim=64, vdim=64, chunk=50, softcap=15.0), A(heads=4, kv_heads=4, dim=128, vdim=32, chunk=16)],
                                  width=128, vocab=211, embed_scale=1.0),
    # one head everywhere, one norm group, five taps, scales of 1, windows and chunks longer than anything they see
    "plain": lambda: U.make_config([P(heads=1, kv_heads=1, dim=40, vdim=24, window=4000, rot_dims=40, left_scale=1.0, right_scale=1.0, s_heads=1,
                                      s_vdim=40, state=24, groups=1, norm_groups=1, conv=5), D(heads=1, kv_heads=1, dim=40, vdim=20, conv=5),
                                    A(heads=1, kv_heads=1, dim=32, vdim=32, chunk=4000, bias_max=300)], width=96, embed_scale=9.0),
}


def assert_close(got, want, dtype, what=""):
    """float32: every position within 2e-4 of the logits' spread.  bfloat16 against the unrounded restatement: within the rounding of a
    few bfloat16 layers, at every position (no router: nothing jumps)."""
    e = U.logit_errors(got, want)
    assert np.isfinite(e).all(), what
    if dtype == torch.float32:
        assert e.max() < 2e-4, (what, float(e.max()), int(e.argmax()))
    else:
        assert np.median(e) < 0.04 and e.max() < 0.2, (what, float(np.median(e)), float(e.max()), int(e.argmax()))


def poison(eng):
    for c in eng.runner.caches:                   # nothing may be read before it is written
        for t in (c if isinstance(c, (tuple, list)) else [c]):
            t.fill_(float("nan"))


def build(tmp_path, name, dtype, seed=0, **engine_args):
    from aphrodite_engine_amd.engine import LLMEngine
    cfg = CONFIGS[name]() if isinstance(name, str) else name
    W = U.make_weights(cfg, seed=seed)
    path = U.write_checkpoint(str(tmp_path / f"m-{seed}"), cfg, W)
    args = dict(max_tokens=512, max_num_seqs=4)
    args.update(engine_args)
    eng = LLMEngine.from_pretrained(path, dtype=dtype, device=DEV, **args)
    poison(eng)
    return cfg, W, eng


def prompts(cfg, lens, seed=0):
    rng = np.random.default_rng(seed)
    return [rng.integers(0, cfg["vocab"], n).tolist() for n in lens]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt_and_layer_trace(mops, tmp_path, name, dtype):
    cfg, W, eng = build(tmp_path, name, dtype)
    toks = prompts(cfg, [83])[0]
    trace = []
    want = O.forward(cfg, W, toks, trace)
    model = eng.runner.model
    model.residual_trace = []
    got = eng.run_segments([("a", toks, list(range(len(toks))))]).cpu().numpy()
    assert_close(got, want, dtype)
    assert len(model.residual_trace) == len(trace) == len(cfg["layers"])
    for x, w in zip(model.residual_trace, trace):
        x = x.cpu().numpy()
        assert np.isfinite(x).all()
        if dtype == torch.float32:
            assert np.abs(x - w).max() < 2e-4 * max(1.0, np.abs(w).max() / 10)
    model.residual_trace = None
    eng.release("a")
    again = eng.run_segments([("b", toks, list(range(len(toks))))]).cpu().numpy()      # reused pages and slot
    assert_close(again, want, dtype)
    eng.release("b")
    some = eng.run_segments([("c", toks, [80, 3, 41])]).cpu().numpy()                   # the last layer runs on the wanted rows only
    assert_close(some, want[[80, 3, 41]], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["mixed", "wide"])
def test_portions_and_token_by_token_equal_the_whole_prompt(mops, tmp_path, name, dtype):
    cfg, W, eng = build(tmp_path, name, dtype)
    toks = prompts(cfg, [100], seed=1)[0]
    want = O.forward(cfg, W, toks)
    whole = eng.run_segments([("whole", toks, list(range(100)))]).cpu().numpy()
    eng.release("whole")
    for rid, sizes in (("tok", [1] * 100), ("two", [2] * 50), ("mix", [2, 15, 1, 16, 2, 17, 3, 1, 1, 42]), ("tail", [68] + [1] * 32)):
        got, a = [], 0
        for n in sizes:
            got.append(eng.run_segments([(rid, toks[a:a + n], list(range(n)))]).cpu().numpy())
            a += n
        eng.release(rid)
        assert a == 100
        assert_close(np.concatenate(got), want, dtype, rid)
        # how a prompt is cut changes nothing beyond rounding -- in bfloat16 too
        assert np.quantile(U.logit_errors(np.concatenate(got), whole), 0.9) < (2e-4 if dtype == torch.float32 else 0.05), rid


@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_requests_in_one_batch_equal_each_alone(mops, tmp_path, dtype):
    cfg, W, eng = build(tmp_path, "mixed", dtype, max_tokens=320)
    ps = prompts(cfg, [90, 1, 23, 47], seed=2)
    want = [O.forward(cfg, W, p) for p in ps]
    # a schedule with portions beside single tokens; request 1 ends early and request 3 takes its pages and slot
    plan = [[(0, 2), (1, 1)], [(0, 30), (2, 3)], [(0, 1), (2, 1), (3, 2)], [(0, 1), (2, 17), (3, 16)], [(2, 2), (3, 1), (0, 20)],
            [(3, 28), (0, 1)], [(0, 35)]]
    at, got = [0] * 4, [[] for _ in ps]
    for step in plan:
        entries = [(str(i), ps[i][at[i]:at[i] + n], list(range(n))) for i, n in step]
        out = eng.run_segments(entries).cpu().numpy()
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


def test_pages_and_slots_taken_over_from_a_finished_request(mops, tmp_path):
    cfg, W, eng = build(tmp_path, "plain", torch.float32, max_tokens=64, max_num_seqs=1)
    a, b = prompts(cfg, [60, 50], seed=3)
    eng.run_segments([("a", a, [])])
    with pytest.raises(Exception):
        eng.run_segments([("b", b, [])])             # neither pages nor a slot are left
    eng.requests.pop("b", None)
    eng.release("a")
    # the new request starts with single tokens in the slot the old one left: no state and no convolution may see a's
    got = [eng.run_segments([("b", b[:1], [0])]), eng.run_segments([("b", b[1:3], [0, 1])]), eng.run_segments([("b", b[3:31], list(range(28)))]),
           eng.run_segments([("b", b[31:], list(range(19)))])]
    assert_close(torch.cat(got).cpu().numpy(), O.forward(cfg, W, b), torch.float32)


@pytest.mark.parametrize("kind", ["chunk", "window", "state"])
def test_a_marker_token_is_seen_as_far_as_the_mixer_reaches(mops, tmp_path, kind):
    """One layer without a feed-forward: a marker token changes the rows that can still see it and no others, in a prompt and decoded:
    the rest of its chunk of 64, the next 49 rows of a window of 50, every later row through a state that hardly decays."""
    if kind == "chunk":
        layer = A(heads=2, kv_heads=1, dim=16, vdim=16, chunk=64, mlp=None, scale=2.0)
    elif kind == "window":                          # (right_scale 0: the state space beside it is silent)
        layer = P(heads=2, kv_heads=1, dim=16, vdim=16, window=50, rot_dims=8, mlp=None, scale=1.0, right_scale=0.0)
    else:
        layer = P(heads=2, kv_heads=1, dim=16, vdim=16, window=50, mlp=None, left_scale=0.0)
    cfg = U.make_config([layer], vocab=50, width=32)
    W = U.make_weights(cfg, seed=7)
    if kind == "state":
        W["l0.mix.right.A_log"][:] = -8.0
        W["l0.mix.right.conv"][:, :-1] = 0.0         # no reach through the convolution
    toks = [t if t != 7 else 8 for t in prompts(cfg, [400], seed=8)[0]]
    at = 150 if kind == "chunk" else 60              # chunk 128 .. 191
    toks[at] = 7                                     # the marker
    other = list(toks)
    other[at] = 9
    want = O.forward(cfg, W, toks)
    from aphrodite_engine_amd.engine import LLMEngine
    path = U.write_checkpoint(str(tmp_path / kind), cfg, W)
    eng = LLMEngine.from_pretrained(path, dtype=torch.float32, device=DEV, max_tokens=1024, max_num_seqs=2)
    poison(eng)
    cut = at - 5
    for rid, sizes in (("whole", [400]), ("decoded", [cut] + [1] * (400 - cut))):
        res = []
        for t in (toks, other):
            got, a = [], 0
            for n in sizes:
                got.append(eng.run_segments([(rid, t[a:a + n], list(range(n)))]))
                a += n
            eng.release(rid)
            res.append(torch.cat(got).cpu().numpy())
        assert_close(res[0], want, torch.float32, rid)
        diff = np.abs(res[0] - res[1]).max(-1)
        assert diff[at] > 1e-3 and diff[:at].max() < 1e-6
        end = {"chunk": 192, "window": at + 50, "state": 400}[kind]
        assert (diff[at:end] > 1e-6).mean() > 0.9 and diff[end - 1] > 1e-7
        assert end == 400 or diff[end:].max() < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_past_every_window_and_chunk(mops, tmp_path, dtype):
    cfg, W, eng = build(tmp_path, "mixed", dtype)
    toks = prompts(cfg, [180], seed=4)[0]
    want = O.forward(cfg, W, toks)
    got = [eng.run_segments([("a", toks[:5], [4])])]
    for t in toks[5:]:
        got.append(eng.run_segments([("a", [t], [0])]))
    assert_close(torch.cat(got).cpu().numpy(), want[4:], dtype)


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
    ls = [A(heads=8, kv_heads=2, dim=32, vdim=32, chunk=30, softcap=12.0, bias_max=25), D(heads=6, kv_heads=2, dim=48, vdim=24, conv=2, mlp=None),
          P(heads=4, kv_heads=4, dim=32, vdim=64, window=27, rot_dims=20, base=900.0, s_heads=9, s_vdim=16, state=36, groups=3, norm_groups=12,
            conv=6)]
    cfg = U.make_config(ls + [U.same_as(ls, 1), U.same_as(ls, 0)], vocab=300, width=104, eps=1e-4, embed_scale=2.5)
    W = U.make_weights(cfg, seed=21, decay_rank=17, gate_rank=8, rel_rows=10)
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
                        "--max-tokens", "128"], input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done %d" % n for n in range(len(plan))]
    got = [np.fromfile(str(out / ("%d.f32" % n)), dtype="<f4").reshape(-1, cfg["vocab"]) for n in range(len(plan))]
    assert [g.shape[0] for g in got] == [len(w) for w in rows]
    assert_close(np.concatenate(got), np.stack([z for w in rows for z in w]), torch.float32 if dtype == "float32" else torch.bfloat16)
