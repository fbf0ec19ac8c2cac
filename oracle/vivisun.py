"""Plain, slow restatement of the Vivisun decoder, one function per mechanism (test infrastructure only: nothing under
aphrodite_engine_amd/ imports this, and this imports nothing from there).  float64 numpy, no cache: every call recomputes a whole
sequence; the attentions materialise the whole score matrix and every head's keys and values.

Notation: x [T, W] is the residual of one sequence, positions 0 .. T-1.  Weights come as a dict name -> array, named as in the
checkpoint; the configuration is the checkpoint's config.json as a dict."""
import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis."""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def dynamic_tanh(x, W, name):
    """tanh(alpha x) w + b: elementwise, no statistic of the row."""
    return np.tanh(float(W[name + ".alpha"]) * x) * W[name] + W[name + ".b"]


def causal_conv(u, w):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_{t - taps + 1 + j}, zeros before the sequence."""
    taps = w.shape[1]
    pad = np.concatenate([np.zeros((taps - 1, u.shape[1])), u], 0)
    return sum(pad[j:j + u.shape[0]] * w[:, j] for j in range(taps))


# ---- rotation -------------------------------------------------------------------------------------------------------------
def frequencies(dims, base, scaling=None):
    """(f_i for i < dims / 2, factor on cos and sin).  Scaling: numbers that turn often over the original length keep their
    frequency, numbers that turn seldom are slowed by the factor, a ramp over i joins the two."""
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    if not scaling:
        return f, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])

    def index_that_turns(times):
        return dims * math.log(original / (2.0 * math.pi * times)) / (2.0 * math.log(base))
    lo = max(math.floor(index_that_turns(float(scaling["fast"]))), 0)
    hi = min(math.ceil(index_that_turns(float(scaling["slow"]))), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate_halves(x, positions, freq, mag):
    """x [T, heads, n]: number i of a head turns with number i + len(freq), i < len(freq); the rest passes."""
    half = len(freq)
    a = np.asarray(positions, np.float64)[:, None] * freq
    cos, sin = np.cos(a)[:, None, :] * mag, np.sin(a)[:, None, :] * mag
    out = x.copy()
    u, v = x[..., :half], x[..., half:2 * half]
    out[..., :half], out[..., half:2 * half] = u * cos - v * sin, v * cos + u * sin
    return out


# ---- attention ------------------------------------------------------------------------------------------------------------
def softmax_attention(q, k, v, scale, sink=None):
    """One head, causal: q, k [T, d], v [T, e].  ``sink``: a score without key or value that joins the denominator."""
    T = q.shape[0]
    s = np.where(np.tril(np.ones((T, T), bool)), (q @ k.T) * scale, -np.inf)
    m = s.max(-1, keepdims=True)
    if sink is not None:
        m = np.maximum(m, sink)
    p = np.exp(s - m)
    den = p.sum(-1, keepdims=True)
    if sink is not None:
        den = den + np.exp(sink - m)
    return (p / den) @ v


def attention(h, W, p, mc, eps):
    T = h.shape[0]
    H, G, d, e = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    q, k, v = (causal_conv(h @ W[p + n].T, W[p + n + ".conv"]) if mc.get("conv") else h @ W[p + n].T for n in ("q", "k", "v"))
    q = rms_norm(q.reshape(T, H, d), W[p + "q.norm"], eps)
    k = rms_norm(k.reshape(T, G, d), W[p + "k.norm"], eps)
    v = v.reshape(T, G, e)
    rot = mc["rot"]
    freq, mag = frequencies(int(rot["dims"]), float(rot["base"]), rot.get("scaling"))
    q, k = (rotate_halves(z, np.arange(T), freq, mag) for z in (q, k))
    out = np.zeros((T, H, e))
    for a in range(H):
        out[:, a] = softmax_attention(q[:, a], k[:, a // (H // G)], v[:, a // (H // G)], mc["scale"])
    return (out.reshape(T, H * e) * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def latent_attention(h, W, p, mc, eps):
    T = h.shape[0]
    H, d, e = mc["heads"], mc["dim"], mc["vdim"]
    q = (h @ W[p + "q"].T).reshape(T, H, d)
    c = rms_norm(h @ W[p + "dkv"].T, W[p + "dkv.norm"], eps)
    k, v = (c @ W[p + "uk"].T).reshape(T, H, d), (c @ W[p + "uv"].T).reshape(T, H, e)
    gate = sigmoid(h @ W[p + "g"].T)
    out = np.zeros((T, H, e))
    for a in range(H):
        out[:, a] = softmax_attention(q[:, a], k[:, a], v[:, a], mc["scale"], float(W[p + "sink"][a])) * gate[:, a:a + 1]
    return out.reshape(T, H * e) @ W[p + "o"].T


MIXERS = {"attention": attention, "latent_attention": latent_attention}


def dense_ff(h, W, p):
    return (silu(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


# ---- the stack ------------------------------------------------------------------------------------------------------------
def layer_order(cfg):
    """[(layer, whether the embedding output joins x ahead of it)] in the order of running."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b = int(loop["start"]), int(loop["stop"])
    runs = [(i, False) for i in range(a)]
    for t in range(int(loop["times"])):
        runs += [(i, t > 0 and i == a) for i in range(a, b)]
    return runs + [(i, False) for i in range(b, n)]


def forward(cfg, W, tokens, trace=None):
    """Logits [T, vocab] of one sequence; ``trace`` (a list) receives the residual after every layer run."""
    eps = cfg["norm"]["eps"]
    W = {n: np.asarray(t, np.float64) for n, t in W.items()}
    x = start = W["embed"][np.asarray(tokens)]
    for i, again in layer_order(cfg):
        lc, p = cfg["layers"][i], f"l{i}."
        if again:
            x = x + start
        y = MIXERS[lc["type"]](dynamic_tanh(x, W, p + "norm1"), W, p + "mix.", lc["mixer"], eps)
        if lc.get("mlp") is not None:
            y = y + dense_ff(dynamic_tanh(x, W, p + "norm2"), W, p + "mlp.")
        x = x + y
        if trace is not None:
            trace.append(x.copy())
    return dynamic_tanh(x, W, "final.norm") @ W["head"].T
