"""Small random Nukezen checkpoints for the tests: a config dict, numpy weights named as in a checkpoint, and a writer of
config.json + model.safetensors.  Sizes are deliberately unlike one another (dim != vdim, head counts that differ, fewer rotated
numbers than the head has, a width that is no power of two, layers that differ in everything) so that a swapped size or a constant
taken from the wrong layer shows."""
import numpy as np

from fatudra_util import bf16_round, logit_errors  # noqa: F401
from fekotar_util import assert_logits, write_checkpoint  # noqa: F401


def dense(ff=88):
    return {"kind": "dense", "ff": ff}


def delta_layer(heads=4, kv_heads=2, dim=24, vdim=40, conv=4, mlp="default"):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": dense() if mlp == "default" else mlp}


def attn_layer(heads=6, kv_heads=2, dim=24, vdim=16, chunk=21, softcap=7.0, bias_max=50, scale=None, mlp="default"):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk},
                                           "softcap": softcap, "bias_max": bias_max, "scale": scale if scale is not None else dim ** -0.5},
            "mlp": dense() if mlp == "default" else mlp}


def par_layer(heads=3, kv_heads=1, dim=20, vdim=28, window=17, rot_dims=12, base=3000.0, scale=None, left_scale=0.7, right_scale=1.3,
              s_heads=6, s_vdim=12, state=20, groups=3, norm_groups=4, conv=4, mlp="default"):
    return {"type": "parallel", "mlp": dense() if mlp == "default" else mlp,
            "mixer": {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
                               "rot": {"base": base, "dims": rot_dims}, "scale": scale if scale is not None else dim ** -0.5},
                      "right": {"heads": s_heads, "vdim": s_vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv},
                      "left_scale": left_scale, "right_scale": right_scale}}


def same_as(layers, j):
    """A layer on layer j's tensors."""
    return dict(layers[j], weights_of=j)


def make_config(layers, vocab=131, width=72, eps=1e-5, embed_scale=3.0):
    return {"architecture": "Nukezen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale},
            "layers": layers}


def make_weights(cfg, seed=0, round_bf16=True, decay_rank=10, gate_rank=14, rel_rows=12):
    """``decay_rank``, ``gate_rank``, ``rel_rows``: the sizes that only the tensors' shapes tell (layer i adds i to each rank, 2 i to
    the table)."""
    rng = np.random.default_rng(seed)
    W, width = {}, cfg["width"]

    def mat(o, i, gain=1.0):
        return rng.standard_normal((o, i)) * gain / np.sqrt(i)

    def vec(k, mean=1.0, std=0.2):
        return mean + std * rng.standard_normal(k)

    g = 1.0 / cfg["embedding"]["scale"]            # the residual a mixer reads is not normed: keep the projections' outputs near 1
    W["embed"] = rng.standard_normal((cfg["vocab"], width))
    W["final.norm"] = vec(width)
    for i, lc in enumerate(cfg["layers"]):
        if lc.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", lc["mixer"]
        W[p + "norm1"] = vec(width)
        if lc["mlp"] is not None:
            W[p + "norm2"] = vec(width)
            ff = lc["mlp"]["ff"]
            W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"] = mat(ff, width, 2 * g), mat(ff, width, 2 * g), mat(width, ff)
        if lc["type"] == "channel_delta":
            H, G, d, e, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            for nm, rows in (("q", G * d), ("k", G * d), ("v", H * e)):
                W[p + "mix." + nm] = mat(rows, width, 2 * g)
                W[p + "mix." + nm + ".conv"] = rng.standard_normal((rows, taps)) * 0.6
            ra, rg = decay_rank + i, gate_rank + i
            W[p + "mix.b"], W[p + "mix.a1"], W[p + "mix.a2"] = mat(H, width, 2 * g), mat(ra, width, g), mat(H * d, ra, 2.0)
            W[p + "mix.g1"], W[p + "mix.g2"] = mat(rg, width, g), mat(H * e, rg, 2.0)
            W[p + "mix.A_log"], W[p + "mix.dt_bias"] = np.log(rng.uniform(0.1, 2.0, H)), vec(H * d, -1.0, 1.5)
            W[p + "mix.norm"], W[p + "mix.o"] = vec(e), mat(width, H * e)
        elif lc["type"] == "attention":
            H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            W[p + "mix.q"], W[p + "mix.k"], W[p + "mix.v"] = mat(H * d, width, g), mat(G * d, width, g), mat(G * e, width, g)
            W[p + "mix.q.norm"], W[p + "mix.k.norm"] = vec(H * d, 2.0, 0.5), vec(G * d, 2.0, 0.5)
            W[p + "mix.rel"], W[p + "mix.o"] = rng.standard_normal((rel_rows + 2 * i, H)) * 1.5, mat(width, H * e)
        else:
            L, R = m["left"], m["right"]
            H, G, d, e = L["heads"], L["kv_heads"], L["dim"], L["vdim"]
            q = p + "mix.left."
            for nm, rows in (("q", H * d), ("k", G * d), ("v", G * e)):
                W[q + nm], W[q + nm + ".b"] = mat(rows, width, g), vec(rows, 0.0, 0.5)
            W[q + "q.norm"], W[q + "k.norm"] = vec(d, 1.5, 0.4), vec(d, 1.5, 0.4)
            W[q + "g"], W[q + "o"] = mat(H * e, width, 2 * g), mat(width, H * e)
            H, e, N, G = R["heads"], R["vdim"], R["state"], R["groups"]
            q, C = p + "mix.right.", H * e + 2 * G * N
            W[q + "in"] = mat(H * e + C + H, width, 1.5 * g)
            W[q + "conv"], W[q + "conv.b"] = rng.standard_normal((C, R["conv"])) * 0.6, vec(C, 0.0, 0.3)
            W[q + "dt_bias"], W[q + "A_log"], W[q + "D"] = vec(H, -1.0, 1.0), np.log(rng.uniform(0.05, 2.0, H)), vec(H, 1.0, 0.5)
            W[q + "norm"], W[q + "o"] = vec(H * e), mat(width, H * e)
    if round_bf16:
        W = {k: bf16_round(v) for k, v in W.items()}
    return {k: np.asarray(v, np.float32) for k, v in W.items()}
