"""CPU oracle for the Novosun design: plain float64 numpy, one function per mechanism.

TEST INFRASTRUCTURE ONLY (see ``oracle/__init__.py``): nothing in ``exo_amd`` imports it, and it
imports nothing from there.  Whole sequences, one token after the other: recurrences are stepped,
every score row is written out, nothing is cached or batched.

Notation: a sequence has T tokens, residual x [T, W]; a recurrent head's state S [keys, values].
"""

from __future__ import annotations

import numpy as np


def rms(x: np.ndarray, eps: float) -> np.ndarray:
    """Root of (mean square over the last axis + eps), kept as an axis."""
    return np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def rms_norm(x, gain, eps):
    return x / rms(x, eps) * gain


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


# ------------------------------------------------------------------ recurrences


def recurrence(q, k, v, decay):
    """S <- diag(decay_t) S + k_t v_t^T, then o_t = S^T q_t, from S = 0.  q, k, decay [T, D], v [T, E]
    of one head; returns (o [T, E], the last S)."""
    S = np.zeros((q.shape[1], v.shape[1]))
    out = np.empty_like(v)
    for t in range(len(q)):
        S = decay[t][:, None] * S + np.outer(k[t], v[t])
        out[t] = q[t] @ S
    return out, S


def channel_decay(h, w, p, tau):
    """Per key channel, through a low-rank product: sigmoid(z) to the power 1 / tau."""
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    return np.exp(-softplus(-z) / tau)


def gated_linear_attention(h, w, p, m, eps):
    T, H, D, E = len(h), m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).reshape(T, H, D) / np.sqrt(D)
    k = (h @ w[p + "k"].T).reshape(T, H, D)
    v = (h @ w[p + "v"].T).reshape(T, H, E)
    a = channel_decay(h, w, p, m["tau"]).reshape(T, H, D)
    o = np.stack([recurrence(q[:, i], k[:, i], v[:, i], a[:, i])[0] for i in range(H)], axis=1)
    o = rms_norm(o, w[p + "norm"], eps).reshape(T, H * E)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def causal_conv(x, w, b):
    """Per channel over the last ``taps`` inputs (zeros before the sequence), the current one's weight
    last; then silu."""
    T, taps = len(x), w.shape[1]
    past = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    out = np.empty_like(x)
    for t in range(T):
        out[t] = (past[t : t + taps] * w.T).sum(0) + b
    return silu(out)


def grouped_norm(y, gain, groups, eps):
    parts = y.reshape(len(y), groups, -1)
    return (parts / rms(parts, eps)).reshape(y.shape) * gain


def state_space(h, w, p, m, eps):
    H, E, N, G, T = m["heads"], m["vdim"], m["state"], m["groups"], len(h)
    inner = H * E
    z, xbc, dt = np.split(h @ w[p + "in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    xbc = causal_conv(xbc, w[p + "conv"], w[p + "conv.b"])
    x = xbc[:, :inner].reshape(T, H, E)
    B = xbc[:, inner : inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N :].reshape(T, G, N)
    dt = softplus(dt + w[p + "dt_bias"])
    y = np.empty((T, H, E))
    for i in range(H):
        g = i // (H // G)
        decay = np.exp(-np.exp(w[p + "A_log"][i]) * dt[:, i])
        o, _ = recurrence(C[:, g], B[:, g], dt[:, i : i + 1] * x[:, i], np.repeat(decay[:, None], N, axis=1))
        y[:, i] = o + w[p + "D"][i] * x[:, i]
    y = y.reshape(T, inner) * silu(z)
    return grouped_norm(y, w[p + "norm"], m["norm_groups"], eps) @ w[p + "o"].T


# ------------------------------------------------------------------ attention


def attend(q, k, v, scale):
    """Causal softmax attention, q [T,H,D], k [T,G,D], v [T,G,E] -> [T,H,E]."""
    T, H, G = len(q), q.shape[1], k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            s = (k[: i + 1, g] @ q[i, h]) * scale
            e = np.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[: i + 1, g]
    return out


def gated_attention(h, w, p, m, eps):
    T, H, G, D, E = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm((h @ w[p + "q"].T).reshape(T, H, D), w[p + "q.norm"], eps)
    k = rms_norm((h @ w[p + "k"].T).reshape(T, G, D), w[p + "k.norm"], eps)
    v = (h @ w[p + "v"].T).reshape(T, G, E)
    o = attend(q, k, v, m["scale"]) * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * E) @ w[p + "o"].T


def parallel(h, w, p, m, eps):
    a = rms_norm(gated_attention(h, w, p + "left.", m["left"], eps), w[p + "left.out"], eps)
    b = rms_norm(state_space(h, w, p + "right.", m["right"], eps), w[p + "right.out"], eps)
    return (a + b) / 2


# ------------------------------------------------------------------ the rest


def clamped_glu(gate, up, limit):
    g, u = np.minimum(gate, limit), np.clip(up, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def feed_forward(h, w, p, m):
    return clamped_glu(h @ w[p + "gate"].T, h @ w[p + "up"].T, m["limit"]) @ w[p + "down"].T


MIXERS = {"gla": gated_linear_attention, "parallel": parallel}


class Float64(dict):
    """Weights already converted to float64 arrays."""


def to_float64(w: dict) -> Float64:
    return w if isinstance(w, Float64) else Float64({k: np.asarray(v, np.float64) for k, v in w.items()})


def forward(cfg: dict, w: dict, tokens, layers_out: list | None = None) -> np.ndarray:
    """Token ids of one sequence -> logits [T, vocab]; ``layers_out`` collects the residual after
    every layer."""
    w, eps, mult = to_float64(w), cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][np.asarray(tokens)]
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        o = MIXERS[L["type"]](rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", L["mixer"], eps)
        x = x + mult * rms_norm(o, w[p + "norm1b"], eps)
        if L.get("mlp"):
            o = feed_forward(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", L["mlp"])
            x = x + mult * rms_norm(o, w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


def greedy(cfg: dict, w: dict, prompt, n: int):
    """n greedy tokens after ``prompt`` by running the whole sequence again for each; returns
    (tokens, the last position's logits before each)."""
    seq, toks, logits = [int(t) for t in prompt], [], []
    w = to_float64(w)
    for _ in range(n):
        lg = forward(cfg, w, seq)[-1]
        logits.append(lg)
        toks.append(int(np.argmax(lg)))
        seq.append(toks[-1])
    return toks, np.stack(logits)
