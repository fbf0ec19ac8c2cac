"""Plain, slow restatement of the Nukezen decoder, one function per mechanism (test infrastructure only: nothing under
aphrodite_engine_amd/ imports this, and this imports nothing from there).  float64 numpy, no cache: every call recomputes a whole
sequence; the recurrences go token by token, the attentions materialise the whole score matrix.

Notation: x [T, W] is the residual of one sequence, positions 0 .. T-1.  Weights come as a dict name -> array, named as in the
checkpoint; the configuration is the checkpoint's config.json as a dict."""
import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def rms_norm(x, w, eps):
    """x / sqrt(mean(x^2) + eps) * w over the last axis (w None: no weight)."""
    y = x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)
    return y if w is None else y * w


def unit(x, eps=1e-6):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + eps)


# ---- what the attentions have in common ----------------------------------------------------------------------------------
def rotate_neighbours(x, positions, dims, base):
    """x [T, heads, n]: numbers (2 i, 2 i + 1) of a head, i < dims / 2, turn by position * base^(-2 i / dims)."""
    a = np.asarray(positions, np.float64)[:, None] * np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    cos, sin = np.cos(a)[:, None, :], np.sin(a)[:, None, :]
    out = x.copy()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2], out[..., 1:dims:2] = u * cos - v * sin, v * cos + u * sin
    return out


def visible(T, window=0, chunk=0):
    """bool [T, T]: row i sees j <= i; with a window only i - j < window, with chunks only j of its own chunk."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    see = j <= i
    if window:
        see &= i - j < window
    if chunk:
        see &= i // chunk == j // chunk
    return see


def distance_bucket(n, rows, far):
    """Row of a distance table: exact up to rows / 2, then widening geometrically until `far`, capped at the last row."""
    half = rows // 2
    if n < half:
        return n
    return min(rows - 1, half + math.floor(math.log(n / half) / math.log(far / half) * (rows - half)))


def softmax_attention(q, k, v, scale, see, cap=0.0, bias=None, sink=None):
    """One head: q, k [T, d], v [T, e], see bool [T, T].  scores s = q k^T scale, then cap * tanh(s / cap), then + bias [T, T];
    `sink`: a score without key or value that joins the denominator."""
    s = (q @ k.T) * scale
    if cap:
        s = cap * np.tanh(s / cap)
    if bias is not None:
        s = s + bias
    s = np.where(see, s, -np.inf)
    m = s.max(-1, keepdims=True)
    if sink is not None:
        m = np.maximum(m, sink)
    p = np.exp(s - m)
    den = p.sum(-1, keepdims=True)
    if sink is not None:
        den = den + np.exp(sink - m)
    return (p / den) @ v


# ---- mixer "attention": whole-row q / k norm, soft cap, distance table, chunks, a sink of score 0 --------------------------
def attention(h, W, p, mc, eps):
    T = h.shape[0]
    H, G, d, e = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    q = rms_norm(h @ W[p + "q"].T, W[p + "q.norm"], eps).reshape(T, H, d)
    k = rms_norm(h @ W[p + "k"].T, W[p + "k.norm"], eps).reshape(T, G, d)
    v = (h @ W[p + "v"].T).reshape(T, G, e)
    rel = W[p + "rel"]
    dist = np.arange(T)[:, None] - np.arange(T)[None, :]
    row_of = np.array([distance_bucket(n, rel.shape[0], mc["bias_max"]) for n in range(T)])
    see = visible(T, chunk=int(mc["mask"]["size"]))
    out = np.zeros((T, H, e))
    for a in range(H):
        g = a // (H // G)
        bias = rel[row_of[np.maximum(dist, 0)], a]
        out[:, a] = softmax_attention(q[:, a], k[:, g], v[:, g], mc["scale"], see, mc["softcap"], bias, sink=0.0)
    return out.reshape(T, H * e) @ W[p + "o"].T


# ---- mixer "parallel", left: biased projections, per-head norm before the rotation, window, elementwise gate ----------------
def window_attention(h, W, p, mc, eps):
    T = h.shape[0]
    H, G, d, e = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    q, k, v = (h @ W[p + n].T + W[p + n + ".b"] for n in ("q", "k", "v"))
    q = rms_norm(q.reshape(T, H, d), W[p + "q.norm"], eps)
    k = rms_norm(k.reshape(T, G, d), W[p + "k.norm"], eps)
    v = v.reshape(T, G, e)
    pos, rot = np.arange(T), mc["rot"]
    q, k = (rotate_neighbours(z, pos, int(rot["dims"]), rot["base"]) for z in (q, k))
    see = visible(T, window=int(mc["mask"]["size"]))
    out = np.zeros((T, H, e))
    for a in range(H):
        g = a // (H // G)
        out[:, a] = softmax_attention(q[:, a], k[:, g], v[:, g], mc["scale"], see)
    return (out.reshape(T, H * e) * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


# ---- recurrences -----------------------------------------------------------------------------------------------------------
def causal_conv(u, w, b=None):
    """u [T, C], w [C, taps]: y_t = sum_j w[:, j] u_{t - taps + 1 + j} (+ b), zeros before the sequence."""
    T, taps = u.shape[0], w.shape[1]
    pad = np.concatenate([np.zeros((taps - 1, u.shape[1])), u], 0)
    y = sum(pad[j:j + T] * w[:, j] for j in range(taps))
    return y if b is None else y + b


def state_space(x, B, C, dt, a_log, D):
    """One head: x [T, e], B, C [T, N], dt [T].  S <- exp(-exp(a_log) dt) S + dt B x^T;  y = S^T C + D x."""
    S = np.zeros((B.shape[1], x.shape[1]))
    y = np.zeros_like(x)
    for t in range(x.shape[0]):
        S = math.exp(-math.exp(a_log) * dt[t]) * S + dt[t] * np.outer(B[t], x[t])
        y[t] = S.T @ C[t] + D * x[t]
    return y


def state_space_mixer(h, W, p, mc, eps):
    T = h.shape[0]
    H, e, N, G = mc["heads"], mc["vdim"], mc["state"], mc["groups"]
    inner = H * e
    proj = h @ W[p + "in"].T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * G * N], proj[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, W[p + "conv"], W[p + "conv.b"]))
    x = xbc[:, :inner].reshape(T, H, e)
    B, C = xbc[:, inner:inner + G * N].reshape(T, G, N), xbc[:, inner + G * N:].reshape(T, G, N)
    dt = softplus(dt + W[p + "dt_bias"])
    y = np.zeros((T, H, e))
    for a in range(H):
        g = a // (H // G)
        y[:, a] = state_space(x[:, a], B[:, g], C[:, g], dt[:, a], float(W[p + "A_log"][a]), float(W[p + "D"][a]))
    y = y.reshape(T, inner) * silu(z)
    parts = mc["norm_groups"]
    y = rms_norm(y.reshape(T, parts, inner // parts), None, eps).reshape(T, inner) * W[p + "norm"]
    return y @ W[p + "o"].T


def channel_delta_rule(q, k, v, beta, g):
    """One head: q, k, g [T, d], v [T, e], beta [T].  S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q."""
    S = np.zeros((q.shape[1], v.shape[1]))
    out = np.zeros_like(v)
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + np.outer(k[t], u)
        out[t] = S.T @ q[t]
    return out


def channel_delta_mixer(h, W, p, mc, eps):
    T = h.shape[0]
    H, G, d, e = mc["heads"], mc["kv_heads"], mc["dim"], mc["vdim"]
    q, k, v = (silu(causal_conv(h @ W[p + n].T, W[p + n + ".conv"])) for n in ("q", "k", "v"))
    q, k = unit(q.reshape(T, G, d)) * d ** -0.5, unit(k.reshape(T, G, d))
    v = v.reshape(T, H, e)
    beta = sigmoid(h @ W[p + "b"].T)
    a = ((h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]).reshape(T, H, d)
    g = np.exp(-np.exp(W[p + "A_log"])[None, :, None] * softplus(a))
    out = np.zeros((T, H, e))
    for n in range(H):
        j = n // (H // G)
        out[:, n] = channel_delta_rule(q[:, j], k[:, j], v[:, n], beta[:, n], g[:, n])
    gate = sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T)
    return (rms_norm(out, W[p + "norm"], eps).reshape(T, H * e) * gate) @ W[p + "o"].T


# ---- the stack -------------------------------------------------------------------------------------------------------------
def parallel_mixer(h, W, p, mc, eps):
    return (mc["left_scale"] * window_attention(h, W, p + "left.", mc["left"], eps)
            + mc["right_scale"] * state_space_mixer(h, W, p + "right.", mc["right"], eps))


def dense_ff(h, W, p):
    return (gelu_tanh(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


MIXERS = {"channel_delta": channel_delta_mixer, "parallel": parallel_mixer, "attention": attention}


def forward(cfg, W, tokens, trace=None):
    """Logits [T, vocab] of one sequence; ``trace`` (a list) receives the residual after every layer."""
    eps = cfg["norm"]["eps"]
    W = {n: np.asarray(t, np.float64) for n, t in W.items()}
    x = W["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    for i, lc in enumerate(cfg["layers"]):
        src = i
        while cfg["layers"][src].get("weights_of") is not None:
            src = cfg["layers"][src]["weights_of"]
        p = f"l{src}."
        x = x + rms_norm(MIXERS[lc["type"]](x, W, p + "mix.", lc["mixer"], eps), W[p + "norm1"], eps)
        if lc.get("mlp") is not None:
            x = x + rms_norm(dense_ff(x, W, p + "mlp."), W[p + "norm2"], eps)
        if trace is not None:
            trace.append(x.copy())
    return rms_norm(x, W["final.norm"], eps) @ W["embed"].T
