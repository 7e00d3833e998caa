"""CPU oracle for the Pimisun design: plain float64 numpy, one function per mechanism.

TEST INFRASTRUCTURE ONLY (see ``oracle/__init__.py``): nothing in ``exo_amd`` imports it, and it
imports nothing from there.  Whole sequences, every score row written out, nothing cached or batched;
latent keys and values are expanded per head.

Notation: a sequence has T tokens, residual x [T, W].
"""

from __future__ import annotations

import numpy as np

from .novosun import rms, rms_norm, silu, to_float64


def layer_norm(x, gain, eps):
    d = x - x.mean(axis=-1, keepdims=True)
    return d / rms(d, eps) * gain


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z**3)))


def relu_squared(z):
    return np.maximum(z, 0.0) ** 2


# ------------------------------------------------------------------ attention


def rotate(x, base, dims):
    """Pairs (2i, 2i + 1) of the first ``dims`` entries of x [T, heads, D] turned by t * base^(-2i / dims)."""
    out = x.copy()
    for t in range(len(x)):
        for i in range(dims // 2):
            a = t * float(base) ** (-2.0 * i / dims)
            u, v = x[t, :, 2 * i], x[t, :, 2 * i + 1]
            out[t, :, 2 * i] = u * np.cos(a) - v * np.sin(a)
            out[t, :, 2 * i + 1] = v * np.cos(a) + u * np.sin(a)
    return out


def attend(q, k, v, scale, window=None, softcap=None):
    """Causal softmax attention, q [T,H,D], k [T,G,D], v [T,G,E] -> [T,H,E]; a query sees fewer than
    ``window`` positions back; scores bent to cap * tanh(score / cap)."""
    T, H, G = len(q), q.shape[1], k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            lo = 0 if window is None else max(0, i - window + 1)
            s = (k[lo : i + 1, g] @ q[i, h]) * scale
            if softcap is not None:
                s = softcap * np.tanh(s / softcap)
            e = np.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[lo : i + 1, g]
    return out


def attention(h, w, p, m, eps, v_first=None):
    """Returns (output, own unmixed values)."""
    T, H, G, D, E = len(h), m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).reshape(T, H, D)
    k = rms_norm(h @ w[p + "k"].T, w[p + "k.norm"], eps).reshape(T, G, D)
    v = own = h @ w[p + "v"].T
    r = m["rot"]
    q, k = rotate(q, r["base"], r["dims"]), rotate(k, r["base"], r["dims"])
    if v_first is not None:
        lam = w[p + "vmix"]
        v = (1.0 - lam) * v + lam * v_first
    o = attend(q, k, v.reshape(T, G, E), m["scale"], m["mask"]["size"], m["softcap"])
    return o.reshape(T, H * E) @ w[p + "o"].T, own


def latent_attention(h, w, p, m, eps):
    T, H, D, R, E, C = len(h), m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).reshape(T, H, D + R)
    z = h @ w[p + "dkv"].T
    c, kr = rms_norm(z[:, :C], w[p + "dkv.norm"], eps), z[:, C:]
    qr = rotate(q[:, :, D:], m["rot"]["base"], R)
    kr = rotate(kr[:, None, :], m["rot"]["base"], R)
    q = np.concatenate([q[:, :, :D], qr], axis=-1)
    k = np.concatenate([(c @ w[p + "uk"].T).reshape(T, H, D), np.repeat(kr, H, axis=1)], axis=-1)
    o = attend(q, k, (c @ w[p + "uv"].T).reshape(T, H, E), m["scale"])
    return o.reshape(T, H * E) @ w[p + "o"].T


# ------------------------------------------------------------------ the rest


def dense(h, w, p):
    return relu_squared(h @ w[p + "up"].T) @ w[p + "down"].T


def glu(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(logits, top):
    """The ``top`` largest (equals: the lower index) and their softmax among themselves."""
    ids = np.argsort(-logits, kind="stable")[:top]
    e = np.exp(logits[ids] - logits[ids].max())
    return ids, e / e.sum()


def experts(h, w, p, f):
    out = np.zeros_like(h)
    logits = h @ w[p + "router"].T + w[p + "router.b"]
    for t in range(len(h)):
        for e, weight in zip(*route(logits[t], f["router"]["top"])):
            out[t] += weight * glu(h[t], w, f"{p}e{e}.")
    return out + glu(h, w, p + "shared.") if f.get("shared") else out


def token_side(x, w, p, e, eps):
    """What a layer adds to the residual from a token's own vector ``e``."""
    y = (gelu_tanh(x @ w[p + "gate"].T) * e) @ w[p + "proj"].T
    return rms_norm(y, w[p + "norm"], eps)


def forward(cfg: dict, w: dict, tokens, layers_out: list | None = None) -> np.ndarray:
    """Token ids of one sequence -> logits [T, vocab]; ``layers_out`` collects the residual after
    every layer."""
    w, eps, alpha = to_float64(w), cfg["norm"]["eps"], cfg["postln_alpha"]
    tokens = np.asarray(tokens)
    x, v_first, S = w["embed"][tokens] * cfg["embedding"]["scale"], None, cfg["token_side"]["dim"]
    for i, L in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", L["mixer"], L.get("mlp")
        if L["type"] == "latent_attention":
            o = latent_attention(x, w, p + "mix.", m, eps)
        else:
            o, own = attention(x, w, p + "mix.", m, eps, v_first if m.get("v_mix") else None)
            if m.get("v_mix") and v_first is None:
                v_first = own
        x = layer_norm(alpha * x + o, w[p + "norm1"], eps)
        if f:
            o = dense(x, w, p + "mlp.") if f["kind"] == "dense" else experts(x, w, p + "mlp.", f)
            x = layer_norm(alpha * x + o, w[p + "norm2"], eps)
        x = x + token_side(x, w, p + "side.", w["side.embed"][tokens, i * S : (i + 1) * S], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return layer_norm(x, w["final.norm"], eps) @ w["embed"].T * cfg["logit_scale"]


def greedy(cfg: dict, w: dict, prompt, n: int):
    """n greedy tokens after ``prompt`` by running the whole sequence again for each."""
    seq, w = [int(t) for t in prompt], to_float64(w)
    for _ in range(n):
        seq.append(int(np.argmax(forward(cfg, w, seq)[-1])))
    return seq[len(prompt) :]


