"""Small random checkpoints of the Gekazen design for the tests (sizes are the tests' own)."""

from __future__ import annotations

import json
from pathlib import Path

import numpy as np


def layer(heads=6, kv_heads=2, dim=32, vdim=32, window=24, keep=3, scale=None, kv_from=None, mlp="default", experts=5,
          identity=2, top=3, ff=40, limit=1.5, rscale=1.7, shared_ff=56, shared_limit=0.9):
    mixer = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=2.0 / np.sqrt(dim) if scale is None else scale,
                 mask=dict(size=window, keep_first=keep))
    if kv_from is not None:
        mixer["kv_from"] = kv_from
    if mlp == "default":
        mlp = dict(kind="moe", expert=dict(ff=ff, limit=limit),
                   router=dict(experts=experts, identity=identity, top=top, scale=rscale))
        if shared_ff:
            mlp["shared"] = dict(ff=shared_ff, limit=shared_limit)
    return dict(type="attention", mixer=mixer, mlp=mlp)


def config(layers, width=72, vocab=331, eps=1e-5):
    return dict(architecture="Gekazen", layers=layers, norm=dict(eps=eps), vocab=vocab, width=width)


def mixed_config():
    """Every branch at once: head groups 3, 2, 1 and 4, key size other than value size, windows of
    several lengths, nothing kept, keys taken from earlier layers under another mask, a layer without
    feed-forward, one without shared expert, one without identity experts, top 1."""
    return config([
        layer(),
        layer(heads=4, kv_heads=2, dim=40, vdim=24, window=70, keep=0, identity=0, top=1, shared_ff=None),
        layer(heads=3, kv_heads=3, dim=64, vdim=20, window=9, keep=17, experts=3, identity=5, top=8, rscale=0.6),
        layer(heads=8, kv_heads=2, dim=40, vdim=24, window=130, keep=5, mlp=None),
        layer(heads=2, kv_heads=2, dim=40, vdim=24, window=33, keep=66, kv_from=1),
        layer(heads=6, kv_heads=3, dim=64, vdim=20, window=1, keep=1, kv_from=2, ff=72, shared_ff=8),
    ], width=100)


def weights(cfg: dict, seed: int = 0) -> dict[str, np.ndarray]:
    """bf16-representable float32 arrays by tensor name."""
    from oracle.affine import bf16_round

    r = np.random.default_rng(seed)
    W, out = cfg["width"], {}

    def put(name, *shape, std=None):
        s = 1.0 / np.sqrt(shape[-1]) if std is None else std
        out[name] = bf16_round((r.standard_normal(shape) * s).astype(np.float32))

    put("embed", cfg["vocab"], W, std=1.0)
    put("head", cfg["vocab"], W)
    put("final.norm", W, std=0.2)
    for i, L in enumerate(cfg["layers"]):
        m, f, p = L["mixer"], L.get("mlp"), f"l{i}."
        put(p + "norm1", W, std=0.3)
        sizes = [("q", m["heads"] * m["dim"])]
        if m.get("kv_from") is None:
            sizes += [("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])]
        for n, rows in sizes:
            put(p + f"mix.{n}", rows, W)
            put(p + f"mix.{n}.b", rows, std=0.3)
        put(p + "mix.o", W, m["heads"] * m["vdim"])
        put(p + "mix.o.b", W, std=0.3)
        if f is None:
            continue
        put(p + "norm2", W, std=0.3)
        rt, ff = f["router"], f["expert"]["ff"]
        n = rt["experts"] + rt["identity"]
        put(p + "mlp.router", n, W)
        put(p + "mlp.correction", n, std=0.3)
        for e in range(rt["experts"]):
            put(p + f"mlp.e{e}.gate", ff, W)
            put(p + f"mlp.e{e}.up", ff, W)
            put(p + f"mlp.e{e}.down", W, ff)
        if f.get("shared"):
            sf = f["shared"]["ff"]
            put(p + "mlp.shared.gate", sf, W)
            put(p + "mlp.shared.up", sf, W)
            put(p + "mlp.shared.down", W, sf)
            put(p + "mlp.shared.sg", 1, W)
    return out


def torch_weights(w: dict[str, np.ndarray], device="cpu"):
    import torch

    return {k: torch.from_numpy(v).to(torch.bfloat16).to(device) for k, v in w.items()}


def write_checkpoint(path, cfg: dict, w: dict[str, np.ndarray]) -> Path:
    from safetensors.torch import save_file

    path = Path(path)
    path.mkdir(parents=True, exist_ok=True)
    save_file(torch_weights(w), str(path / "model.safetensors"))
    (path / "config.json").write_text(json.dumps(cfg))
    return path


def rel_rms(got, want) -> np.ndarray:
    """Per row: RMS of the difference over the RMS of what is expected."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    return np.sqrt(np.mean((got - want) ** 2, -1)) / np.sqrt(np.mean(want**2, -1))


def router_gaps(cfg: dict, w: dict, tokens) -> np.ndarray:
    """Per token: the smallest gap, over the layers, between the last chosen and the first unchosen
    choice score (a bf16 model may choose otherwise where it is tiny)."""
    from oracle import gekazen as O

    gaps, seen = [], []
    orig = O.route

    def spy(logits, corr, top, scale):
        c = np.sort(O.softmax(logits) + corr)[::-1]
        seen.append(c[top - 1] - c[top] if top < len(c) else np.inf)
        return orig(logits, corr, top, scale)

    O.route = spy
    try:
        O.forward(cfg, w, tokens)
    finally:
        O.route = orig
    n = len(tokens)
    for i in range(0, len(seen), n):
        gaps.append(seen[i : i + n])
    return np.min(np.asarray(gaps), axis=0)
