"""Small random checkpoints of the Novosun design for the tests (sizes are the tests' own)."""

from __future__ import annotations

import numpy as np


def linear(heads=3, dim=40, vdim=24, tau=5.0, ff=56, limit=1.2):
    return dict(type="gla", mixer=dict(heads=heads, dim=dim, vdim=vdim, tau=tau), mlp=mlp(ff, limit))


def parallel(heads=6, kv_heads=3, dim=24, vdim=40, scale=None, ssm_heads=6, ssm_vdim=20, state=12, groups=3, conv=4,
             norm_groups=2, ff=48, limit=0.9):
    return dict(type="parallel", mixer=dict(
        left=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=1.5 / np.sqrt(dim) if scale is None else scale),
        right=dict(heads=ssm_heads, vdim=ssm_vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups)),
        mlp=mlp(ff, limit))


def mlp(ff, limit):
    return None if ff is None else dict(kind="dense", ff=ff, limit=limit)


def config(layers, width=72, vocab=331, eps=1e-4, mult=0.7):
    return dict(architecture="Novosun", layers=layers, norm=dict(eps=eps), residual_mult=mult, vocab=vocab, width=width)


def mixed_config():
    """Every branch, with sizes that meet and sizes that do not: key size above and below the value size
    and past 64, one and several key groups, 1 to 9 taps, norm groups unlike the key groups, layers
    without feed-forward, a tau below 1."""
    return config([
        linear(),
        parallel(),
        parallel(heads=4, kv_heads=4, dim=36, vdim=36, ssm_heads=2, ssm_vdim=70, state=88, groups=1, conv=1, norm_groups=1,
                 ff=None),
        linear(heads=1, dim=72, vdim=136, tau=0.5, ff=None),
        linear(heads=5, dim=16, vdim=16, tau=16.0, ff=130, limit=2.0),
        parallel(heads=5, kv_heads=1, dim=64, vdim=7, ssm_heads=5, ssm_vdim=16, state=16, groups=5, conv=9, norm_groups=5),
    ], width=100)


def weights(cfg: dict, seed: int = 0, rank: int = 10) -> dict[str, np.ndarray]:
    """bf16-representable float32 arrays by tensor name."""
    from oracle.affine import bf16_round

    r = np.random.default_rng(seed)
    W, out = cfg["width"], {}

    def put(name, *shape, std=None, mean=0.0):
        s = 1.0 / np.sqrt(shape[-1]) if std is None else std
        out[name] = bf16_round((mean + r.standard_normal(shape) * s).astype(np.float32))

    def norm(name, n):
        put(name, n, std=0.3, mean=1.0)

    put("embed", cfg["vocab"], W, std=1.0)
    put("head", cfg["vocab"], W)
    norm("final.norm", W)
    for i, L in enumerate(cfg["layers"]):
        m, f, p = L["mixer"], L.get("mlp"), f"l{i}."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            norm(p + n, W)
        if L["type"] == "gla":
            hd, he = m["heads"] * m["dim"], m["heads"] * m["vdim"]
            for n, rows in (("q", hd), ("k", hd), ("v", he), ("g", he), ("a1", rank)):
                put(p + f"mix.{n}", rows, W)
            put(p + "mix.o", W, he)
            norm(p + "mix.norm", m["vdim"])
            put(p + "mix.a2", hd, rank, std=0.6)
            put(p + "mix.a2.b", hd, std=3.0, mean=2.0)  # from a token or two to hundreds
        else:
            a, s, q = m["left"], m["right"], p + "mix.left."
            put(q + "q", a["heads"] * a["dim"], W)
            put(q + "k", a["kv_heads"] * a["dim"], W)
            put(q + "v", a["kv_heads"] * a["vdim"], W)
            norm(q + "q.norm", a["dim"])
            norm(q + "k.norm", a["dim"])
            put(q + "g", a["heads"], W, std=1.5 / np.sqrt(W))
            put(q + "o", W, a["heads"] * a["vdim"])
            q, inner = p + "mix.right.", s["heads"] * s["vdim"]
            ch = inner + 2 * s["groups"] * s["state"]
            put(q + "in", inner + ch + s["heads"], W)
            put(q + "conv", ch, s["conv"], std=0.6)
            put(q + "conv.b", ch, std=0.3)
            put(q + "dt_bias", s["heads"], std=1.0, mean=-2.0)
            put(q + "A_log", s["heads"], std=1.2)
            put(q + "D", s["heads"], std=0.5, mean=0.5)
            norm(q + "norm", inner)
            put(q + "o", W, inner)
            norm(p + "mix.left.out", W)
            norm(p + "mix.right.out", W)
        if f:
            put(p + "mlp.gate", f["ff"], W)
            put(p + "mlp.up", f["ff"], W)
            put(p + "mlp.down", W, f["ff"])
    return out


def ssm_oracle(w: dict, m: dict, y: np.ndarray, dt_raw: np.ndarray, rounding=None) -> np.ndarray:
    """Layer 0's state-space recurrence over given projection columns: ``y`` values | keys, queries ahead of
    the convolution, ``dt_raw``; ``rounding``: of the convolved inputs."""
    from oracle import novosun as O

    T, H, G, N, E = len(y), m["heads"], m["groups"], m["state"], m["vdim"]
    inner = H * E
    p = "l0.mix.right."
    x = O.causal_conv(y.astype(np.float64), w[p + "conv"].astype(np.float64), w[p + "conv.b"].astype(np.float64))
    if rounding is not None:
        x = rounding(x.astype(np.float32)).astype(np.float64)
    dt = O.softplus(dt_raw.astype(np.float64) + w[p + "dt_bias"])
    v, B, C = x[:, :inner].reshape(T, H, E), x[:, inner : inner + G * N].reshape(T, G, N), x[:, inner + G * N :].reshape(T, G, N)
    out = np.empty((T, H, E))
    for h in range(H):
        g = h // (H // G)
        a = np.exp(-np.exp(np.float64(w[p + "A_log"][h])) * dt[:, h])
        o, _ = O.recurrence(C[:, g], B[:, g], dt[:, h : h + 1] * v[:, h], np.repeat(a[:, None], N, 1))
        out[:, h] = o + w[p + "D"][h] * v[:, h]
    return out.reshape(T, inner)
