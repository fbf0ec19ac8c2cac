"""Nukezen without a GPU: configuration checks, registry, loader (fused input products, the state space's one input tensor cut into
its pieces, sizes that only the tensors' shapes tell, shared layers; surplus / missing / misshapen tensors), cache shapes, and closed
forms of the restatement."""
import numpy as np
import pytest
import torch

import nukezen_util as U
from oracle import nukezen as O

D, A, P = U.delta_layer, U.attn_layer, U.par_layer


def small():
    ls = [D(), P(), A()]
    return U.make_config(ls + [U.same_as(ls, 1), dict(U.same_as(ls, 1), weights_of=3), D(heads=3, kv_heads=1, dim=8, vdim=16, conv=1, mlp=None)])


def shapes_of(W):
    return {k: v.shape for k, v in W.items()}


def load(cfg, W):
    from aphrodite_engine_amd.nukezen import NukezenConfig, NukezenForCausalLM
    m = NukezenForCausalLM(NukezenConfig.from_dict(cfg, shapes_of(W)), torch.float32)
    m.load_weights((k, torch.from_numpy(np.ascontiguousarray(v))) for k, v in W.items())
    return m


def test_registry_and_config_checks():
    from aphrodite_engine_amd import registry
    from aphrodite_engine_amd.nukezen import NukezenConfig
    assert "Nukezen" in registry.supported_architectures()
    cfg = NukezenConfig.from_dict(small(), {})
    assert cfg.owner == [0, 1, 2, 1, 1, 5] and cfg.embed_scale == 3.0 and cfg.eps == 1e-5

    def refuse(change):
        bad = small()
        change(bad["layers"])
        with pytest.raises(ValueError):
            NukezenConfig.from_dict(bad, {})
    refuse(lambda ls: ls[0].update(type="delta"))
    refuse(lambda ls: ls[0].update(mlp={"kind": "moe"}))
    refuse(lambda ls: ls[3].update(weights_of=9))
    refuse(lambda ls: ls[3].update(weights_of=4))                # a ring
    refuse(lambda ls: ls[3].update(weights_of=2))                # another layer's tensors would not fit
    refuse(lambda ls: ls[3].update(mlp=None))
    with pytest.raises(ValueError, match="lacks"):               # inner sizes come from the checkpoint
        cfg.size_from("l0.mix.a1")


def test_loader_places_every_tensor():
    cfg = small()
    W = U.make_weights(cfg, seed=1)
    m = load(cfg, W)
    d0, p1, a2 = m.own["0"].mix, m.own["1"].mix, m.own["2"].mix
    assert sorted(m.own) == ["0", "1", "2", "5"]
    # the delta layer: one input product [q | k | v | g1 | a1 | b | padding], the second halves of the low-rank products
    rows = np.concatenate([W["l0.mix." + n] for n in ("q", "k", "v", "g1", "a1", "b")])
    got = d0.in_proj.weight.numpy()
    np.testing.assert_array_equal(got[:rows.shape[0]], rows)
    assert got.shape[0] % 8 == 0 and not got[rows.shape[0]:].any() and (d0.decay_rank, d0.gate_rank) == (10, 14)
    np.testing.assert_array_equal(d0.a2.weight.numpy(), W["l0.mix.a2"])
    np.testing.assert_array_equal(d0.g2.weight.numpy(), W["l0.mix.g2"])
    np.testing.assert_array_equal(d0.conv.numpy(), np.concatenate([W["l0.mix." + n + ".conv"] for n in ("q", "k", "v")]))
    np.testing.assert_array_equal(d0.dt_bias.numpy(), W["l0.mix.dt_bias"])
    np.testing.assert_array_equal(d0.out_norm.numpy(), W["l0.mix.norm"])
    # the parallel layer: [left q | k | v | g | right x B C | z | dt], biases in front, both output matrices side by side
    R = cfg["layers"][1]["mixer"]["right"]
    inner, src = R["heads"] * R["vdim"], W["l1.mix.right.in"]
    C = inner + 2 * R["groups"] * R["state"]
    left = [W["l1.mix.left." + n] for n in ("q", "k", "v", "g")]
    rows = np.concatenate(left + [src[inner:inner + C], src[:inner], src[inner + C:]])
    got = p1.in_proj.weight.numpy()
    np.testing.assert_array_equal(got[:rows.shape[0]], rows)
    assert not got[rows.shape[0]:].any()
    bias = np.concatenate([W["l1.mix.left." + n + ".b"] for n in ("q", "k", "v")])
    np.testing.assert_array_equal(p1.in_proj.bias.numpy()[:bias.shape[0]], bias)
    assert not p1.in_proj.bias.numpy()[bias.shape[0]:].any()
    np.testing.assert_array_equal(p1.out_proj.weight.numpy(), np.concatenate([W["l1.mix.left.o"], W["l1.mix.right.o"]], 1))
    for key, t in (("conv", p1.ssm.conv), ("conv.b", p1.ssm.conv_bias), ("A_log", p1.ssm.a_log), ("D", p1.ssm.skip), ("dt_bias", p1.ssm.dt_bias),
                   ("norm", p1.ssm.norm)):
        np.testing.assert_array_equal(t.numpy(), W["l1.mix.right." + key])
    np.testing.assert_array_equal(p1.attn.k_norm.numpy(), W["l1.mix.left.k.norm"])
    assert p1.attn.attn.window == 17 and p1.attn.attn.chunk == 0 and p1.attn.attn.sink is None and p1.attn.rotary.dims == 12
    # attention: whole-row norms, the distance table and its look-up by distance
    np.testing.assert_array_equal(a2.in_proj.weight.numpy()[:a2.attn.heads * a2.attn.dim], W["l2.mix.q"])
    np.testing.assert_array_equal(a2.attn.q_norm.numpy(), W["l2.mix.q.norm"])
    rel = W["l2.mix.rel"]
    m.finalize()
    lut = a2.attn.attn.bias_lut.numpy()
    for n in range(60):
        np.testing.assert_array_equal(lut[:, min(n, lut.shape[1] - 1)], rel[O.distance_bucket(n, rel.shape[0], 50)])
    assert a2.attn.attn.chunk == 21 and a2.attn.attn.softcap == 7.0 and a2.attn.attn.sink.tolist() == [0.0] * 6
    # feed-forward; none in the last layer
    np.testing.assert_array_equal(m.own["2"].mlp.gate_up.weight.numpy(), np.concatenate([W["l2.mlp.gate"], W["l2.mlp.up"]]))
    assert m.own["5"].mlp is None
    # caches: every layer its own, also the sharers; one tap keeps no convolution input
    shapes = [[tuple(t.shape) for t in (c if isinstance(c, tuple) else (c, ))] for c in m.make_caches(5, 16, 2, "cpu")]
    delta, par = [[(2, 3, 2 * 2 * 24 + 4 * 40)], [(2, 4, 24, 40)]], [[(5, 16, 1, 20), (5, 16, 1, 28)], [(2, 3, C)], [(2, 6, 20, 12)]]
    assert shapes == delta + par + [[(5, 16, 2, 24), (5, 16, 2, 16)]] + par + par + [[(2, 0, 2 * 8 + 3 * 16)], [(2, 3, 8, 16)]]
    assert len({id(c) for c in m.make_caches(1, 16, 1, "cpu")}) == len(m.specs)


def test_loader_refuses_surplus_missing_and_misshapen_tensors():
    cfg = small()
    W = U.make_weights(cfg, seed=2)
    with pytest.raises(ValueError, match="unexpected"):
        load(cfg, dict(W, **{"l0.mix.extra": W["l0.norm1"]}))
    with pytest.raises(ValueError, match="unexpected"):           # a layer on another's tensors has none
        load(cfg, dict(W, **{"l3.norm1": W["l1.norm1"]}))
    with pytest.raises(ValueError, match="lacks"):
        load(cfg, {k: v for k, v in W.items() if k != "l1.mix.left.q.b"})
    for name in ("l2.mix.k", "l1.mix.right.in", "l0.mix.dt_bias", "l1.mlp.down", "l1.mix.right.o"):
        with pytest.raises(ValueError, match="does not fit"):
            load(cfg, dict(W, **{name: W[name][:-1]}))
    load(cfg, dict(W, **{"l5.norm2": W["l5.norm1"]}))             # the weight of a norm that is never applied


def test_shapes_are_read_from_the_files(tmp_path):
    from aphrodite_engine_amd.loader import load_model, safetensors_shapes
    cfg = small()
    W = U.make_weights(cfg, seed=3, decay_rank=5, gate_rank=9, rel_rows=20)
    path = U.write_checkpoint(str(tmp_path / "m"), cfg, W)
    assert safetensors_shapes(path) == shapes_of(W)
    m = load_model(path, dtype=torch.float32, device="cpu")
    assert m.own["0"].mix.decay_rank == 5 and m.own["5"].mix.gate_rank == 14 and m.own["2"].mix.attn.attn.rel.shape[0] == 24
    np.testing.assert_array_equal(m.own["5"].mix.g2.weight.numpy(), W["l5.mix.g2"])


def test_restatement_closed_forms():
    rng = np.random.default_rng(0)
    # the rotation of neighbours keeps lengths and makes scores depend on the distance only
    x, y = rng.standard_normal((1, 1, 12)), rng.standard_normal((1, 1, 12))
    r = lambda z, p: O.rotate_neighbours(z, [p], 8, 100.0)
    assert abs((r(x, 5) * r(y, 2)).sum() - (r(x, 105) * r(y, 102)).sum()) < 1e-9
    np.testing.assert_allclose(np.linalg.norm(r(x, 7)), np.linalg.norm(x))
    np.testing.assert_array_equal(r(x, 7)[..., 8:], x[..., 8:])
    # masks
    w, c = O.visible(9, window=3), O.visible(9, chunk=4)
    assert w[5].tolist() == [False] * 3 + [True] * 3 + [False] * 3 and w[1].sum() == 2
    assert c[5].tolist() == [False] * 4 + [True] * 2 + [False] * 3 and c[4].sum() == 1 and c[3].sum() == 4
    np.testing.assert_array_equal(O.visible(9, window=1), np.eye(9, dtype=bool))
    np.testing.assert_array_equal(O.visible(9, window=9), O.visible(9, chunk=20))
    # buckets: exact, then widening, then the last row
    assert [O.distance_bucket(n, 8, 32) for n in (0, 3, 4, 5, 6, 7, 11, 12, 18, 20, 31, 32, 500)] == [0, 3, 4, 4, 4, 5, 5, 6, 6, 7, 7, 7, 7]
    # soft cap before the bias, a sink of score 0
    q, k, v = rng.standard_normal((9, 4)), rng.standard_normal((9, 4)), rng.standard_normal((9, 3))
    s = 2.0 * np.tanh((k[:5] @ q[4]) * 3.0 / 2.0) + 0.7
    p = np.exp(s) / (1.0 + np.exp(s).sum())
    np.testing.assert_allclose(O.softmax_attention(q, k, v, 3.0, O.visible(9), 2.0, np.full((9, 9), 0.7), 0.0)[4], p @ v[:5])
    # the state space with a decay of 1 and unit steps is a running sum; D passes the input on
    B, C, xv = np.ones((4, 1)), np.ones((4, 1)), np.arange(4.0)[:, None]
    np.testing.assert_allclose(O.state_space(xv, B, C, np.ones(4), -800.0, 0.5)[:, 0], [0.0, 1.5, 4.0, 7.5])
    # the delta rule: no decay stores the last value per key; a channel that decays forgets its own row only
    keys, vals = np.eye(4)[[0, 1, 0]], rng.standard_normal((3, 2))
    out = O.channel_delta_rule(np.eye(4)[[0, 0, 0]], keys, vals, np.ones(3), np.ones((3, 4)))
    np.testing.assert_allclose(out, vals[[0, 0, 2]], atol=1e-12)
    g = np.ones((3, 4))
    g[2, 1] = 0.0
    out = O.channel_delta_rule(np.eye(4)[[0, 1, 1]], keys, vals, np.ones(3), g)
    np.testing.assert_allclose(out, [vals[0], vals[1], 0 * vals[0]], atol=1e-12)
    # convolution: the last column is the current token's tap
    u, wc = rng.standard_normal((5, 2)), np.array([[0.0, 0.0, 1.0], [1.0, 0.0, 0.0]])
    y = O.causal_conv(u, wc, np.array([0.0, 2.0]))
    np.testing.assert_allclose(y[:, 0], u[:, 0])
    np.testing.assert_allclose(y[:, 1], np.concatenate([[0, 0], u[:3, 1]]) + 2.0)


def test_a_shared_layer_is_the_same_function_twice():
    ls = [P(), A(mlp=None)]
    cfg = U.make_config(ls + [U.same_as(ls, 0)])
    W = U.make_weights(cfg, seed=4)
    plain = {k: v for k, v in cfg.items() if k != "layers"}
    twice = dict(plain, layers=ls + [dict(ls[0])])
    W2 = dict(W, **{k.replace("l0.", "l2.", 1): v for k, v in W.items() if k.startswith("l0.")})
    toks = [3, 9, 27, 81, 5, 5, 9]
    np.testing.assert_allclose(O.forward(cfg, W, toks), O.forward(twice, W2, toks))
