"""Small random Vivisun checkpoints for the tests: a config dict, numpy weights named as in a checkpoint, and a writer of
config.json + model.safetensors.  Sizes are deliberately unlike one another (dim != vdim, head counts that differ, fewer rotated
numbers than the head has, a width that is no power of two, layers that differ in everything) so that a swapped size or a constant
taken from the wrong layer shows."""
import numpy as np

from fatudra_util import bf16_round, logit_errors  # noqa: F401
from fekotar_util import write_checkpoint  # noqa: F401


def dense(ff=88):
    return {"kind": "dense", "ff": ff}


def attn_layer(heads=6, kv_heads=2, dim=24, vdim=40, conv=3, rot_dims=20, base=3000.0, scaling=(3.0, 64, 16.0, 2.0), scale=None,
               mlp="default"):
    rot = {"base": base, "dims": rot_dims}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": rot, "scale": scale if scale is not None else dim ** -0.5}
    if conv:
        m["conv"] = conv
    return {"type": "attention", "mixer": m, "mlp": dense() if mlp == "default" else mlp}


def latent_layer(heads=3, dim=20, vdim=28, kv_rank=44, scale=None, mlp="default"):
    return {"type": "latent_attention", "mlp": dense() if mlp == "default" else mlp,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale if scale is not None else dim ** -0.5}}


def make_config(layers, vocab=131, width=72, eps=1e-3, loop=None):
    """``loop``: (start, stop, times) or None."""
    c = {"architecture": "Vivisun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    return c


def make_weights(cfg, seed=0, round_bf16=True):
    rng = np.random.default_rng(seed)
    W, width = {}, cfg["width"]

    def mat(o, i, gain=1.0):
        return rng.standard_normal((o, i)) * gain / np.sqrt(i)

    def vec(k, mean=1.0, std=0.2):
        return mean + std * rng.standard_normal(k)

    def norm(name):
        W[name], W[name + ".b"], W[name + ".alpha"] = vec(width), vec(width, 0.0, 0.3), np.asarray(rng.uniform(0.3, 0.8))

    W["embed"], W["head"] = rng.standard_normal((cfg["vocab"], width)), mat(cfg["vocab"], width)
    norm("final.norm")
    for i, lc in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lc["mixer"]
        H, d, e = m["heads"], m["dim"], m["vdim"]
        norm(p + "norm1")
        if lc["mlp"] is not None:
            norm(p + "norm2")
            ff = lc["mlp"]["ff"]
            W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"] = mat(ff, width, 2.0), mat(ff, width, 2.0), mat(width, ff)
        W[p + "mix.q"], W[p + "mix.o"] = mat(H * d, width, 2.0), mat(width, H * e, 2.0)
        if lc["type"] == "attention":
            G = m["kv_heads"]
            W[p + "mix.k"], W[p + "mix.v"], W[p + "mix.g"] = mat(G * d, width, 2.0), mat(G * e, width, 2.0), mat(H * e, width, 2.0)
            W[p + "mix.q.norm"], W[p + "mix.k.norm"] = vec(d, 1.5, 0.4), vec(d, 1.5, 0.4)
            if m.get("conv"):
                for n, rows in (("q", H * d), ("k", G * d), ("v", G * e)):
                    W[p + "mix." + n + ".conv"] = rng.standard_normal((rows, m["conv"])) * 0.6
        else:
            R = m["kv_rank"]
            W[p + "mix.dkv"], W[p + "mix.dkv.norm"] = mat(R, width, 2.0), vec(R)
            W[p + "mix.uk"], W[p + "mix.uv"] = mat(H * d, R, 1.5), mat(H * e, R, 1.5)
            W[p + "mix.sink"], W[p + "mix.g"] = vec(H, 1.5, 1.0), mat(H, width, 2.0)
    if round_bf16:
        W = {k: bf16_round(v) for k, v in W.items()}
    return {k: np.asarray(v, np.float32) for k, v in W.items()}
