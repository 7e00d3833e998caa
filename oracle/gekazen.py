"""CPU oracle for the Gekazen design: plain float64 numpy, one function per mechanism.

TEST INFRASTRUCTURE ONLY (see ``oracle/__init__.py``): nothing in ``exo_amd`` imports it, and
it imports nothing from there.  Whole sequences, no cache, no batching: the mask of every
(query, key) pair is written out and each token's experts are looped over one by one.

Notation: a sequence has T tokens at positions 0..T-1, residual x [T, W].
"""

from __future__ import annotations

import numpy as np


def rms_unit(x: np.ndarray, eps: float) -> np.ndarray:
    """x / sqrt(mean over the last axis of x^2, plus eps)."""
    return x / np.sqrt(np.mean(np.square(x), axis=-1, keepdims=True) + eps)


def rms_norm_offset(x: np.ndarray, w: np.ndarray, eps: float) -> np.ndarray:
    """RMS norm whose stored weight is the gain minus one."""
    return rms_unit(x, eps) * (1.0 + w)


def linear(x: np.ndarray, w: np.ndarray, b: np.ndarray | None = None) -> np.ndarray:
    y = x @ w.T
    return y if b is None else y + b


def head_slopes(n_heads: int) -> np.ndarray:
    """Per-head slope of the linear distance penalty: 2^(-8 (h+1) / n_heads)."""
    return np.array([2.0 ** (-8.0 * (h + 1) / n_heads) for h in range(n_heads)])


def visible(T: int, size: int | None, keep_first: int) -> np.ndarray:
    """[query, key] mask: causal, and either fewer than ``size`` positions back or among the
    first ``keep_first`` positions of the sequence (``size`` None: causal only)."""
    i = np.arange(T)[:, None]
    j = np.arange(T)[None, :]
    m = j <= i
    if size is not None:
        m &= ((i - j) < size) | (j < keep_first)
    return m


def softmax(s: np.ndarray) -> np.ndarray:
    e = np.exp(s - s.max(-1, keepdims=True))
    return e / e.sum(-1, keepdims=True)


def attend(q: np.ndarray, k: np.ndarray, v: np.ndarray, scale: float, slopes: np.ndarray,
           mask: np.ndarray) -> np.ndarray:
    """q [T,H,D], k [T,G,D], v [T,G,E] -> [T,H,E]; head h reads key/value head h // (H/G); the
    score of keys d positions back is lowered by slope_h * d."""
    T, H, _ = q.shape
    G = k.shape[1]
    dist = np.arange(T)[:, None] - np.arange(T)[None, :]
    out = np.empty((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale - slopes[h] * dist
        s = np.where(mask, s, -np.inf)
        out[:, h] = softmax(s) @ v[:, g]
    return out


def attention(x, w, p, m, eps, shared_kv=None):
    """One attention mixer -> (output [T,W], (k, v)).  ``m``: the mixer's config entry;
    ``shared_kv``: keys and values of another layer, taken as they are."""
    T = x.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_unit(linear(x, w[p + "q"], w[p + "q.b"]).reshape(T, H, D), eps)
    if shared_kv is None:
        k = rms_unit(linear(x, w[p + "k"], w[p + "k.b"]).reshape(T, G, D), eps)
        v = linear(x, w[p + "v"], w[p + "v.b"]).reshape(T, G, E)
    else:
        k, v = shared_kv
    mask = m.get("mask") or {}
    o = attend(q, k, v, m["scale"], head_slopes(H),
               visible(T, mask.get("size"), mask.get("keep_first", 0)))
    return linear(o.reshape(T, H * E), w[p + "o"], w[p + "o.b"]), (k, v)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def clamped_glu(gate: np.ndarray, up: np.ndarray, limit: float) -> np.ndarray:
    """g sigmoid(1.702 g) (u + 1) with g capped from above and u on both sides at ``limit``."""
    g = np.minimum(gate, limit)
    u = np.clip(up, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def expert(x, w, p, limit):
    return linear(clamped_glu(linear(x, w[p + "gate"]), linear(x, w[p + "up"]), limit), w[p + "down"])


def route(logits: np.ndarray, correction: np.ndarray, top: int, scale: float):
    """One token's (expert ids, weights): chosen by softmax score plus correction, weighted by
    the score alone times ``scale``, not renormalised."""
    s = softmax(logits)
    ids = np.argsort(-(s + correction), kind="stable")[:top]
    return ids, s[ids] * scale


def moe(x, w, p, m):
    """Experts chosen per token, some of which hand the input through, plus the gated shared one."""
    r = m["router"]
    out = np.zeros_like(x)
    for t in range(x.shape[0]):
        ids, wt = route(linear(x[t], w[p + "router"]), w[p + "correction"], r["top"], r["scale"])
        for e, a in zip(ids, wt):
            out[t] += a * (x[t] if e >= r["experts"] else
                           expert(x[t], w, f"{p}e{e}.", m["expert"]["limit"]))
    if m.get("shared"):
        gate = sigmoid(linear(x, w[p + "shared.sg"]))
        out += gate * expert(x, w, p + "shared.", m["shared"]["limit"])
    return out


def forward(cfg: dict, w: dict, tokens, layers_out: list | None = None) -> np.ndarray:
    """Token ids of one sequence -> logits [T, vocab]; ``layers_out`` collects the residual
    after every layer."""
    w = {k: np.asarray(v, np.float64) for k, v in w.items()} if not isinstance(w, Float64) else w
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(tokens)]
    kv = {}
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        src = L["mixer"].get("kv_from")
        o, own = attention(x, w, p + "mix.", L["mixer"], eps, None if src is None else kv[src])
        kv[i] = own
        x = x + rms_norm_offset(o, w[p + "norm1"], eps)
        if L.get("mlp"):
            x = x + rms_norm_offset(moe(x, w, p + "mlp.", L["mlp"]), w[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return linear(rms_norm_offset(x, w["final.norm"], eps), w["head"])


class Float64(dict):
    """Weights already converted to float64 arrays."""


def to_float64(w: dict) -> Float64:
    return Float64({k: np.asarray(v, np.float64) for k, v in w.items()})


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
