"""Small random checkpoints of the Pimisun design for the tests (sizes are the tests' own)."""

from __future__ import annotations

import numpy as np


def latent(heads=3, dim=24, rot_dim=12, vdim=20, q_rank=36, kv_rank=44, scale=None, base=1e4, mlp="dense", **kw):
    return dict(type="latent_attention", mixer=dict(
        heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, rot=dict(base=base, dims=rot_dim),
        scale=2.0 / np.sqrt(dim + rot_dim) if scale is None else scale), mlp=feed_forward(mlp, **kw))


def attention(heads=6, kv_heads=2, dim=32, vdim=24, window=24, rot=8, base=3e3, scale=None, softcap=12.0, v_mix=True, mlp="moe",
              **kw):
    return dict(type="attention", mixer=dict(
        heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, mask=dict(size=window), rot=dict(base=base, dims=rot),
        scale=2.0 / np.sqrt(dim) if scale is None else scale, softcap=softcap, v_mix=v_mix), mlp=feed_forward(mlp, **kw))


def feed_forward(kind, ff=56, experts=5, top=3, shared=40):
    if kind is None:
        return None
    if kind == "dense":
        return dict(kind="dense", ff=ff)
    f = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))
    return dict(f, shared=dict(ff=shared)) if shared else f


def config(layers, width=72, vocab=331, eps=1e-4, alpha=1.7, embed=0.6, logit=0.4, side=9):
    return dict(architecture="Pimisun", layers=layers, norm=dict(eps=eps), postln_alpha=alpha, embedding=dict(scale=embed),
                logit_scale=logit, token_side=dict(dim=side), vocab=vocab, width=width)


def mixed_config():
    """Every branch, with sizes that meet and sizes that do not: head groups 3, 1, 4 and 5, all dimensions
    rotated and few, latents of full and partial steps of 32 and 64, one head, experts with and without a
    shared one, top 1 and top all, a layer without feed-forward, windows of one token and past a page,
    values that are not mixed between layers that are."""
    return config([
        attention(),
        latent(),
        attention(heads=4, kv_heads=4, dim=40, vdim=12, window=1, rot=40, v_mix=False, softcap=3.0, top=1, shared=None),
        latent(heads=1, dim=40, rot_dim=4, vdim=72, q_rank=20, kv_rank=130, base=50.0, mlp="moe", ff=33, top=5, shared=8),
        attention(heads=8, kv_heads=2, dim=68, vdim=24, window=70, rot=2, mlp=None),
        latent(heads=18, dim=8, rot_dim=8, vdim=8, q_rank=64, kv_rank=32, mlp="dense", ff=130),
        attention(heads=5, kv_heads=1, dim=64, vdim=48, window=131, rot=64, base=7e5, softcap=50.0, mlp="dense", ff=70),
    ], width=100)


def weights(cfg: dict, seed: int = 0, choosy: bool = True) -> dict[str, np.ndarray]:
    """bf16-representable float32 arrays by tensor name.  ``choosy``: every expert is chosen by some token; else the
    routers' logits lie apart from each other and few choices are close enough for bf16 rounding to turn them."""
    from oracle.affine import bf16_round

    r = np.random.default_rng(seed)
    W, S, out = cfg["width"], cfg["token_side"]["dim"], {}

    def put(name, *shape, std=None, mean=0.0):
        s = 1.0 / np.sqrt(shape[-1]) if std is None else std
        out[name] = bf16_round(np.asarray(mean + r.standard_normal(shape) * s, np.float32)).reshape(shape)

    def norm(name, n):
        put(name, n, std=0.3, mean=1.0)

    def glu(p, ff):
        put(p + "gate", ff, W)
        put(p + "up", ff, W)
        put(p + "down", W, ff)

    put("embed", cfg["vocab"], W, std=1.0)
    put("side.embed", cfg["vocab"], len(cfg["layers"]) * S, std=1.0)
    norm("final.norm", W)
    for i, L in enumerate(cfg["layers"]):
        m, f, p = L["mixer"], L.get("mlp"), f"l{i}."
        q = p + "mix."
        norm(p + "norm1", W)
        if L["type"] == "latent_attention":
            put(q + "dq", m["q_rank"], W)
            norm(q + "dq.norm", m["q_rank"])
            put(q + "uq", m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"])
            put(q + "dkv", m["kv_rank"] + m["rot_dim"], W)
            norm(q + "dkv.norm", m["kv_rank"])
            put(q + "uk", m["heads"] * m["dim"], m["kv_rank"])
            put(q + "uv", m["heads"] * m["vdim"], m["kv_rank"])
        else:
            for n, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"])):
                put(q + n, rows, W)
                norm(f"{q}{n}.norm", rows)
            put(q + "v", m["kv_heads"] * m["vdim"], W)
            if m.get("v_mix"):
                put(q + "vmix", std=0.1, mean=0.4)
        put(q + "o", W, m["heads"] * m["vdim"])
        if f:
            norm(p + "norm2", W)
            if f["kind"] == "dense":
                put(p + "mlp.up", f["ff"], W)
                put(p + "mlp.down", W, f["ff"])
            else:
                n = f["router"]["experts"]
                put(p + "mlp.router", n, W, std=(3.0 if choosy else 0.4) / np.sqrt(W))
                put(p + "mlp.router.b", n, std=0.0, mean=r.permutation(n) * (0.3 if choosy else 1.2))
                for e in range(n):
                    glu(f"{p}mlp.e{e}.", f["expert"]["ff"])
                if f.get("shared"):
                    glu(p + "mlp.shared.", f["shared"]["ff"])
        put(p + "side.gate", S, W)
        put(p + "side.proj", W, S)
        norm(p + "side.norm", W)
    return out


def forward_and_gaps(cfg: dict, w, tokens):
    """Oracle logits, and per token the smallest gap over the layers between the last chosen and the first unchosen
    router logit (a bf16 model may choose otherwise where it is tiny)."""
    from oracle import pimisun as O

    seen, orig = [], O.route

    def spy(logits, top):
        z = np.sort(logits)[::-1]
        seen.append(z[top - 1] - z[top] if top < len(z) else np.inf)
        return orig(logits, top)

    O.route = spy
    try:
        lg = O.forward(cfg, w, tokens)
    finally:
        O.route = orig
    return lg, np.min(np.asarray(seen).reshape(-1, len(tokens)), axis=0)
