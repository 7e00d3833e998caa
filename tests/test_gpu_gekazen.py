"""The Gekazen design on the GPU against its plain oracle (``oracle/gekazen.py``): every kernel of
the layer-list decoders alone, whole models under every way to cut and batch sequences, and
generation through the engines.  Float32 mode is the sharp test (1e-4), bf16 the served one."""

import json
import subprocess
import sys
import types
from pathlib import Path

import numpy as np
import pytest
import torch

from exo_amd import dense_ops as D
from exo_amd import native, ops
from exo_amd.engine import SequentialGenerator, ShardBatchGenerator
from exo_amd.generate import generate
from exo_amd.paged_cache import PAGE, PagedKVCache
from exo_amd.prefix_cache import KVPrefixCache
from exo_amd.registry import build_model, config_from_dict
from exo_amd.stack_config import AttentionSpec, GluSpec, MoeSpec, RouterSpec, distance_slopes
from exo_amd.types import TextGenerationTaskParams
from oracle import gekazen as O
from oracle.affine import bf16_round
from tests import gekazen_util as U
from tests import stack_util as S
from tests.stack_util import BF, DTYPES, F32, SCHEDULE, TOL, close, dev, drain, engine, host, mat, play, rand, task
from tests.util import rng

pytestmark = pytest.mark.gpu


def say(*a):
    print("[gekazen]", *a, flush=True)


# ------------------------------------------------------------------ products


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,N,K", [(1, 7, 5), (1, 4100, 200), (3, 331, 72), (16, 50, 1000), (17, 300, 2100),
                                   (33, 20, 64), (65, 130, 448), (200, 1000, 136), (1000, 3000, 320), (300, 17, 4100)])
def test_linear(device, dtype, M, N, K):
    say("linear", dtype, M, N, K)
    x, w, b = rand((M, K), 1), rand((N, K), 2, K**-0.5), rand((N,), 3)
    out = torch.zeros(M, N, dtype=dtype, device="cuda")
    D.linear(mat(x, dtype), mat(w, dtype), out, M, bias=dev(b))
    tag = native.last_variant()
    assert ("dense_gemv" if M <= 16 else "dense_gemm") in tag, tag
    want = x.astype(np.float64) @ w.T + b
    close(host(out), want, 3 * TOL[dtype], f"linear {M}x{N}x{K}")
    out32 = torch.zeros(M, N, dtype=F32, device="cuda")
    D.linear(mat(x, dtype), mat(w, dtype), out32, M)
    close(host(out32), want - b, 2e-5, "float32 output, no bias")
    if M <= 16:
        D.linear(mat(x, dtype), mat(w, dtype), out32, M, force_gemm=True)
        close(host(out32), want - b, 2e-5, "GEMM of few rows")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,N,K", [(5, 40, 72), (70, 33, 200), (700, 130, 96)])
def test_gated_pair(device, dtype, M, N, K):
    say("glu", dtype, M, N, K)
    x, g, u = rand((M, K), 1), rand((N, K), 2, 2 * K**-0.5), rand((N, K), 3, 2 * K**-0.5)
    spec = GluSpec(N, 1.3)
    out = torch.zeros(M, D.pad64(N), dtype=dtype, device="cuda")
    D.glu_gemm(mat(x, dtype), mat(g, dtype), mat(u, dtype), out, M, spec)
    want = O.clamped_glu(x.astype(np.float64) @ g.T, x.astype(np.float64) @ u.T, 1.3)
    close(host(out[:, :N]), want, 3 * TOL[dtype], "gated pair")
    assert not host(out[:, N:]).any()


# ------------------------------------------------------------------ norms, routing, experts


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,H", [(1, 70), (5, 1024), (40, 3000)])
def test_residual_norm(device, dtype, n, H):
    say("post norm", dtype, n, H)
    x, y, w, eps = rand((n, H), 1), rand((n, H), 2, 3e-3), rand((H,), 3), 1e-5  # eps of the order of mean(y^2)
    xt, xb = dev(x), torch.zeros(n, D.pad64(H), dtype=dtype, device="cuda")
    D.post_norm_add(D.Branches(dev(y), dev(1 + w)), eps, xt, xb, n)
    want = x + O.rms_norm_offset(y.astype(np.float64), w, eps)
    close(host(xt), want, 1e-5, "residual")
    close(host(xb[:, :H]), want, TOL[dtype], "its copy")
    rows = torch.tensor([n - 1, 0], dtype=torch.int32, device="cuda")
    out = torch.zeros(2, D.pad64(H), dtype=dtype, device="cuda")
    D.norm_rows(dev(x), dev(1 + w), eps, out, 2, rows=rows)
    close(host(out[:, :H]), O.rms_norm_offset(x[[n - 1, 0]].astype(np.float64), w, eps), TOL[dtype], "norm of rows")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,H,N", [(1, 70, 40), (1, 4096, 5000), (2, 1021, 17), (3, 300, 130), (4, 2048, 331), (4, 1000, 20000)])
def test_residual_norm_inside_a_product(device, dtype, n, H, N):
    say("post gemv", dtype, n, H, N)
    x, y, g, w, b = rand((n, H), 1), rand((n, H), 2, 3e-3), rand((H,), 3), rand((N, H), 4, H**-0.5), rand((N,), 5)
    W, xb = mat(w, dtype), torch.zeros(n, D.pad64(H), dtype=dtype, device="cuda")
    if not native.load().exo_post_linear_fits(n, N, H, xb.shape[1], 0 if dtype == BF else 1):
        assert dtype == F32 or N == 20000  # too many columns for the launch's registers or LDS
        return
    xt, xo, out = dev(x), torch.zeros(n, H, device="cuda"), torch.zeros(n, N, device="cuda")
    D.post_linear(xt, D.Branches(dev(y), dev(1 + g)), 1e-5, xo, xb, W, out, n, bias=dev(b))
    want = x + O.rms_norm_offset(y.astype(np.float64), g, 1e-5)
    close(host(xo), want, 1e-5, "residual")
    close(host(xb[:, :H]), want, TOL[dtype], "its copy")
    assert not host(xb[:, H:]).any() and np.array_equal(host(xt), x)
    close(host(out), host(xb[:, :H]).astype(np.float64) @ w.T + b, 2e-5, "product")


@pytest.mark.parametrize("n,top", [(1, 1), (7, 7), (12, 3), (64, 8), (65, 5), (300, 40), (512, 8)])
def test_router(device, n, top):
    say("router", n, top)
    rows, ld = 33, n + 3
    z, corr = rand((rows, ld), 1, 2.0), rand((n,), 2, 0.05)
    corr[n // 2] += 1.0  # always among the chosen, at its own small weight
    idx = torch.zeros(rows, top, dtype=torch.int32, device="cuda")
    wt = torch.zeros(rows, top, dtype=F32, device="cuda")
    D.moe_route(dev(z), dev(corr), 1.9, idx, wt, rows)
    for t in range(rows):
        ids, want = O.route(z[t, :n].astype(np.float64), corr, top, 1.9)
        assert sorted(idx[t].tolist()) == sorted(ids) and n // 2 in ids
        by = dict(zip(idx[t].tolist(), wt[t].tolist()))
        assert np.allclose([by[int(i)] for i in ids], want, rtol=2e-5)


def moe_case(H, E, I, top, ff, sff, seed=0):
    """A feed-forward of the design by itself: (config entry, oracle weights, spec, layer tensors)."""
    m = dict(expert=dict(ff=ff, limit=1.1), router=dict(experts=E, identity=I, top=top, scale=1.4))
    if sff:
        m["shared"] = dict(ff=sff, limit=0.7)
    cfg = U.config([U.layer(mlp=dict(m, kind="moe"))], width=H)
    w = U.weights(cfg, seed)
    return m, w, config_from_dict(cfg)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,E,I,top,ff,sff", [(72, 5, 2, 3, 40, 56), (200, 3, 6, 4, 17, 0), (128, 9, 0, 9, 64, 100),
                                              (96, 1, 0, 1, 130, 8), (100, 4, 40, 2, 24, 24)])
@pytest.mark.parametrize("n", [1, 2, 16, 17, 150])
def test_feed_forward(device, dtype, H, E, I, top, ff, sff, n):
    say("experts", dtype, (H, E, I, top, ff, sff), "rows", n)
    m, w, cfg = moe_case(H, E, I, top, ff, sff)
    model = build_model(cfg, U.torch_weights(w, "cuda"), dtype=dtype)
    x = rand((n, H), 5)
    bf = model._buffers(1, max(n, 2))
    bf.h[:n].copy_(dev(x))
    bf.xb[:n, :H].copy_(dev(x))
    model._settle(bf, n, model._moe(model.layers[0], bf, n, None), None)
    ww = O.to_float64(w)
    want = O.moe(x.astype(np.float64), ww, "l0.mlp.", m)
    want = x + O.rms_norm_offset(want, ww["l0.norm2"], cfg.eps)
    assert U.rel_rms(host(bf.h[:n]), want).max() < (1e-2 if dtype == BF else 1e-5)


# ------------------------------------------------------------------ attention


def attn_case(spec, T, seed=0, far=()):
    """q|k|v rows of one sequence; ``far``: (query, key) positions whose score is made to stand out
    (the query's heads point along the key's)."""
    H, G, De, E = spec.heads, spec.kv_heads, spec.dim, spec.vdim
    q, k, v = rand((T, H, De), seed), rand((T, G, De), seed + 1), rand((T, G, E), seed + 2)
    for i, j in far:
        q[i] = bf16_round(3 * k[j][np.arange(H) // (H // G)])
    return np.concatenate([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], 1), (q, k, v)


def attn_oracle(spec, qkv, eps, dtype=F32):
    """``dtype`` bf16: normalised queries and keys rounded once, as the kernels hold them."""
    q, k, v = (a.astype(np.float64) for a in qkv)
    sl = np.zeros(spec.heads) if spec.slopes is None else np.asarray(spec.slopes)
    if spec.unit_qk:
        q, k = O.rms_unit(q, eps), O.rms_unit(k, eps)
        if dtype == BF:
            q, k = (bf16_round(a.astype(np.float32)).astype(np.float64) for a in (q, k))
    return O.attend(q, k, v, spec.scale, sl, O.visible(len(q), spec.window, spec.keep_first))


def make_spec(heads, kv_heads, dim, vdim, window, keep, scale=None, slopes=True, unit=True):
    return AttentionSpec(heads, kv_heads, dim, vdim, 4 / np.sqrt(dim) if scale is None else scale, window, keep,
                         unit_qk=unit, slopes=distance_slopes(heads) if slopes else None)


def run_portions(spec, rows_np, cuts, dtype, eps, start_pages=0, fused=True):
    """The sequence through the attention operators in portions; a second sequence's pages lie
    between its own (``start_pages`` of them are taken first)."""
    T = len(rows_np)
    cache = PagedKVCache([(spec.kv_heads, spec.dim, spec.vdim)], 3, 2048, "cuda", dtype)
    sl = None if spec.slopes is None else torch.tensor(spec.slopes, dtype=F32, device="cuda")
    att = D.PagedAttention(spec, sl, 0, cache, eps)
    E = spec.heads * spec.vdim
    ldq = -(-rows_np.shape[1] // 8) * 8
    qkv = torch.zeros(T, ldq, dtype=dtype, device="cuda")
    qkv[:, : rows_np.shape[1]].copy_(dev(rows_np))
    out, got, at = torch.zeros(T, D.pad64(E), dtype=dtype, device="cuda"), [], 0
    i32 = dict(dtype=torch.int32, device="cuda")
    cache.reserve([2], start_pages * PAGE) if start_pages else None
    for n in cuts:
        n = min(n, T - at)
        if n <= 0:
            break
        cache.reserve([1], n)
        cache.reserve([0], 1)
        cache.advance_host(1, [0])
        slot, pos = torch.full((n,), 1, **i32), torch.arange(at, at + n, **i32)
        part, o = qkv[at : at + n].contiguous(), out[:n]
        if n == 1 and fused:
            att.rows(part, o, slot, pos, 1, at + 1, append=True)
        elif dtype == F32 or n == 1:
            att.append(part, slot, pos, n)
            att.rows(part, o, slot, pos, n, at + n, append=False)
        else:
            att.append(part, slot, pos, n)
            bs = att.prompt_block(spec)
            blocks = torch.tensor([(b, 1, at + b, min(bs, n - b)) for b in range(0, n, bs)], **i32)
            att.prompt(part, o, blocks, blocks.shape[0])
        got.append(host(o[:, :E]).reshape(n, spec.heads, spec.vdim).copy())
        cache.advance_host(n, [1])
        at += n
    return np.concatenate(got)


SHAPES = [(5, 5, 64, 64), (6, 2, 48, 80), (8, 2, 128, 128), (5, 1, 96, 32), (40, 2, 32, 32), (2, 2, 256, 192),
          (3, 3, 36, 20), (4, 2, 24, 7), (7, 1, 64, 128)]
WINDOWS = [(None, 0), (1, 0), (33, 0), (64, 5), (65, 64), (100, 70), (40, 500)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", SHAPES)
def test_attention_shapes(device, dtype, shape):
    for i, (window, keep) in enumerate(WINDOWS):
        spec = make_spec(*shape, window, keep, slopes=i % 2 == 0, unit=i % 3 != 2)
        say("attention", dtype, shape, window, keep)
        T, eps = 210, 0.3  # an eps that shows
        rows_np, qkv = attn_case(spec, T, seed=i, far=[(200, 2), (150, 86), (90, 0)])
        want = attn_oracle(spec, qkv, eps, dtype)
        for cuts in ([T], [3, 2, 64, 64, 1, 30, 1, 500], [150] + [1] * 60):
            got = run_portions(spec, rows_np, cuts, dtype, eps, start_pages=2, fused=cuts[0] != 3)
            close(got, want, 1.2e-2 if dtype == BF else 5e-5, f"{shape} {window} {keep} {cuts[:3]}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_attention_edges(device, dtype):
    """One key that carries the whole weight if it is seen, on both sides of every edge: the window,
    the kept first positions, page and tile borders; in a prompt and decoded.  (Scores reach 128, so a
    query element that rounds the other way in bf16 moves a few per cent; a wrong key moves all.)"""
    for window, keep in [(64, 20), (63, 0), (65, 33), (97, 64), (32, 1), (5, 63)]:
        spec = make_spec(4, 2, 64, 32, window, keep, scale=2.0, slopes=False)
        T = 330
        keys = sorted({0, keep - 1, keep, keep + 1, 31, 32, 63, 64, 127, 128} - {-1})
        for key in keys:
            q = [i for d in (-1, 0, 1) for i in (key + window + d, 250 + d, 319 + d) if key < i < T] + [T - 1]
            say("edges", dtype, window, keep, "key", key)
            rows_np, qkv = attn_case(spec, T, seed=key, far=[(i, key) for i in q])
            want = attn_oracle(spec, qkv, 1e-6, dtype)
            seen = [np.abs(want[i] - qkv[2][key][[0, 0, 1, 1]]).max() < 0.3 for i in q]
            vis = O.visible(T, window, keep)
            assert seen == [bool(vis[i, key]) for i in q]  # the planted key decides these rows
            close(run_portions(spec, rows_np, [T], dtype, 1e-6), want, 6e-2 if dtype == BF else 5e-5, "prompt")
            cuts = [min(q) - 1, 2, 2] + [1] * T if min(q) > 1 else [1] * T
            close(run_portions(spec, rows_np, cuts, dtype, 1e-6), want, 6e-2 if dtype == BF else 5e-5, "decoded")


def test_attention_keeps_many_small_weights(device):
    """Five hundred near-equal keys whose values nearly cancel: weights rounded to 8 bits before the
    product with the values would show."""
    spec = make_spec(3, 3, 64, 64, None, 0, scale=0.02)
    T = 512
    rows_np, qkv = attn_case(spec, T, seed=3)
    want = attn_oracle(spec, qkv, 1e-6, BF)
    for cuts in ([T], [T - 6] + [1] * 6):
        got = run_portions(spec, rows_np, cuts, BF, 1e-6)
        assert U.rel_rms(got[-6:].reshape(6, -1), want[-6:].reshape(6, -1)).max() < 4e-3


def test_decode_attention_splits_agree_and_replay(device):
    """A long context over many splits: the same launch three times gives the same bits (arrival
    counters return to zero) and matches the oracle."""
    spec = make_spec(8, 2, 64, 64, None, 0)
    T = 1500
    rows_np, qkv = attn_case(spec, T, seed=9, far=[(T - 1, 3)])
    want = attn_oracle(spec, qkv, 1e-6, BF)[-3:]
    got = run_portions(spec, rows_np, [T - 3, 1, 1, 1], BF, 1e-6)[-3:]
    assert "splits" in native.last_variant() and "splits=1 " not in native.last_variant()
    close(got, want, 1.2e-2, "splits")
    assert np.array_equal(got, run_portions(spec, rows_np, [T - 3, 1, 1, 1], BF, 1e-6)[-3:])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep", [(None, 0), (None, 39), (192, 39), (700, 5)])
def test_decode_attention_over_few_and_many_splits(device, dtype, window, keep):
    """Lengths at which one to eight splits hold tiles, the last one only some of its waves: near
    keys (high slopes) and far ones, in single tokens and portions of seven."""
    spec = make_spec(8, 2, 64, 48, window, keep)
    T = 1100
    rows_np, qkv = attn_case(spec, T, seed=17)
    want = attn_oracle(spec, qkv, 1e-6, dtype)
    for start in (120, 250, 380, 510, 640, 890, 1020):
        say("splits", dtype, window, keep, start)
        for cuts in ([start] + [1] * 50, [start] + [7] * 8):
            got = run_portions(spec, rows_np[: start + 50], cuts, dtype, 1e-6)
            close(got, want[: start + 50], 1.2e-2 if dtype == BF else 5e-5, f"from {start}")


# ------------------------------------------------------------------ whole models


@pytest.fixture(scope="module")
def built():
    """(config, float64 weights, {dtype: model}, tokens, oracle logits) of the mixed configuration."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg = U.mixed_config()
    w = U.weights(cfg, 11)
    models = {t: build_model(config_from_dict(cfg), U.torch_weights(w, "cuda"), dtype=t) for t in DTYPES}
    toks = {name: rng(s).integers(0, cfg["vocab"], n).tolist() for s, (name, n) in
            enumerate({"a": 300, "b": 141, "c": 64, "d": 23, "e": 1}.items())}
    w64 = O.to_float64(w)
    want = {k: O.forward(cfg, w64, t) for k, t in toks.items()}
    gaps = {k: U.router_gaps(cfg, w64, t) for k, t in toks.items()}
    return types.SimpleNamespace(cfg=cfg, w=w64, models=models, toks=toks, want=want, gaps=gaps)


def check_rows(built, dtype, name, places, logits, what):
    """Every row within tolerance; in bf16 a row may be further off once a routing choice was closer
    than bf16 resolves (it and later rows of the sequence may have taken another expert)."""
    err = U.rel_rms(logits, built.want[name][places])
    if dtype == F32:
        assert err.max() < 1e-4, f"{what}: {err.max():.2e} at {places[int(err.argmax())]}"
        return
    assert np.median(err) < 3e-2, f"{what}: median {np.median(err):.2e}"
    tied = np.minimum.accumulate(built.gaps[name])[places] < 4e-3
    assert (err[~tied] < 6e-2).all() and err.max() < 1.0, f"{what}: {err.max():.2e}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("portion", [300, 1, 2, 3, 17, 64, 65, 128])
def test_model_in_portions(built, dtype, portion):
    for name in built.toks if portion in (300, 1) else ("a", "c"):
        say("portions", dtype, portion, name)
        got = play(built.models[dtype], built.toks, [[(name, portion)]] * 300, max_tokens=320)[name]
        check_rows(built, dtype, name, np.arange(len(got)), got, f"portions of {portion}, {name}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_model_layers(built, dtype):
    m, cfg = built.models[dtype], built.cfg
    outs, want = [], []
    O.forward(cfg, built.w, built.toks["c"], want)
    m.layer_hook = lambda i, h: outs.append(host(h).copy())
    try:
        play(m, built.toks, [[("c", 64)]])
    finally:
        m.layer_hook = None
    for i, (g, w) in enumerate(zip(outs, want)):
        err = U.rel_rms(g, w)
        assert np.median(err) < 3e-2 and (dtype == BF or err.max() < 2e-5), f"layer {i}: {err.max():.2e}"


@pytest.mark.parametrize("dtype", DTYPES)
def test_model_mixed_batches_reuse_rows_and_pages(built, dtype):
    """Portions beside single tokens, requests that pause, end and are admitted again in a pool that
    holds them only because pages are used again."""
    say("mixed", dtype)
    got = play(built.models[dtype], built.toks, SCHEDULE, max_tokens=640)
    for name, lg in got.items():
        base = name.split("#")[0]
        check_rows(built, dtype, base, np.arange(len(lg)), lg, f"mixed, {name}")
    for name in ("a", "b"):  # the batch's other members change nothing but rounding
        alone = play(built.models[dtype], built.toks, [[(name, 13)]] * 40)[name]
        err = U.rel_rms(got[name][: len(alone)], alone[: len(got[name])])
        assert np.median(err) < (2e-2 if dtype == BF else 1e-5)


@pytest.mark.parametrize("B", [1, 3, 16, 20])
def test_model_graph_decode_matches_steps(built, B):
    """The captured single-token step over B rows, teacher-forced, against the oracle; several
    replays, eager work between them."""
    m = built.models[F32]
    cache = m.make_cache(B + 1, 320)
    seqs = [built.toks[n][o:] for o in range(8) for n in ("a", "b", "c")][:B]
    n0, n1 = 30, 56
    m.step(cache, [(r, s[: n0 - r % 7], []) for r, s in enumerate(seqs)])
    pos = [n0 - r % 7 for r in range(B)]
    wants = [O.forward(built.cfg, built.w, s[:n1]) for s in seqs]
    for k in range(n1 - n0):
        bf = m._buffers(B, 1)
        bf.tokens.copy_(torch.tensor([s[p] for s, p in zip(seqs, pos)], dtype=torch.int32))
        bf = m.decode_step(cache, B)
        lg = host(bf.logits)
        err = U.rel_rms(lg, np.stack([w[p] for w, p in zip(wants, pos)]))
        assert err.max() < 1e-4, f"step {k}: {err.max():.2e}"
        assert bf.next_token.tolist() == host(m._sampling_logits(bf.logits, bf)).argmax(-1).tolist()
        pos = [p + 1 for p in pos]
        assert cache.pos[:B].tolist() == pos == cache.offsets[:B]
        torch.randn(1000, device="cuda").sum().item()


def test_model_long_decode(built):
    """Four hundred decoded tokens through pages, windows and context regimes."""
    m, toks = built.models[F32], rng(77).integers(0, built.cfg["vocab"], 560).tolist()
    want = O.forward(built.cfg, built.w, toks)
    cache = m.make_cache(1, 600)
    m.step(cache, [(0, toks[:150], [])])
    bf = m._buffers(1, 1)
    for i in range(150, 560):
        bf.tokens[0] = toks[i]
        err = U.rel_rms(host(m.decode_step(cache, 1).logits), want[i : i + 1]).max()
        assert err < 1e-4, f"position {i}: {err:.2e}"


def test_model_pipeline_shards(built):
    cfg = config_from_dict(built.cfg)
    w = U.torch_weights({k: np.asarray(v, np.float32) for k, v in built.w.items()}, "cuda")
    with pytest.raises(ValueError, match="outside the shard"):
        build_model(cfg, w, 3, 6, dtype=F32)
    a, b = build_model(cfg, w, 0, 3, dtype=F32), build_model(cfg, w, 0, 6, dtype=F32)
    ca, cb = a.make_cache(2, 200), b.make_cache(2, 200)
    t = torch.tensor([built.toks["a"][:40], built.toks["b"][:40]])
    h = a(t, ca)
    lo: list = []
    O.forward(built.cfg, built.w, built.toks["b"][:40], lo)
    assert U.rel_rms(host(h)[1], lo[2]).max() < 2e-5
    assert U.rel_rms(host(b(t, cb))[1], built.want["b"][:40]).max() < 1e-4
    # a later shard takes the residual of the one before it
    c = config_from_dict(dict(built.cfg, layers=built.cfg["layers"][:4]))
    x, y = build_model(c, w, 0, 2, dtype=F32), build_model(c, w, 2, 4, dtype=F32)
    cx, cy = x.make_cache(1, 100), y.make_cache(1, 100)
    toks = built.toks["a"]
    for lo_, hi in ((0, 30), (30, 31), (31, 60)):
        got = y(None, cy, input_embeddings=x(torch.tensor([toks[lo_:hi]]), cx), logits="last")
        want = O.forward(dict(built.cfg, layers=built.cfg["layers"][:4]), built.w, toks[:hi])[-1:]
        assert U.rel_rms(host(got)[0], want).max() < 1e-4


def test_step_errors(built):
    m = built.models[BF]
    cache = m.make_cache(2, 128)
    with pytest.raises(ValueError, match="once"):
        m.step(cache, [(0, [1], []), (0, [2], [])])
    with pytest.raises(ValueError, match="places"):
        m.step(cache, [(0, [1, 2], [2])])
    with pytest.raises(ValueError, match="token ids"):
        m.step(cache, [(0, [99999], [])])
    with pytest.raises(ValueError, match="overflow"):
        m.step(cache, [(0, [1] * 129, [])])
    assert cache.offsets == [0, 0] and m.step(cache, [(1, [1, 2], [])]) is None


# ------------------------------------------------------------------ generation


def greedy_agrees(built, prompt, got, dtype):
    S.greedy_agrees(lambda toks: O.forward(built.cfg, built.w, toks), prompt, got, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_engine_mixes_prompts_into_running_batches(built, dtype, monkeypatch):
    """Requests that join while others decode: portions of their prompts share steps with single
    tokens; every sequence is what it is alone, and rows and pages are used again."""
    import exo_amd.engine as E
    monkeypatch.setattr(E, "PREFILL_STEP_SIZE", 37)
    m = built.models[dtype]
    eng = engine(m)
    kinds = []
    step = m.step
    monkeypatch.setattr(m, "step", lambda c, e: (kinds.append(tuple(sorted({len(t) > 1 for _, t, _ in e}))), step(c, e))[1])
    names = ["a", "d", "b", "c", "e", "b"]
    tasks = [task(i, built.toks[n], 20 + 3 * i) for i, n in enumerate(names)]
    got = drain(eng, tasks, join_at=[0, 2, 9, 12, 30, 41])
    assert (False, True) in kinds  # single tokens and portions together
    for t, n in zip(tasks, names):
        assert len(got[t.task_id]) == t.task_params.max_output_tokens
        greedy_agrees(built, built.toks[n], got[t.task_id], dtype)
    c = eng._gen.cache
    assert len(c._free) == c.n_pages and not eng._gen.filling
    eng.close()


def test_engine_waits_for_pages(built):
    """A pool too small for all requests at once: admission waits, nothing fails."""
    eng = engine(built.models[F32], pool_tokens=8 * PAGE)
    names = ["a", "b", "b", "c", "a"]
    tasks = [task(i, built.toks[n], 30) for i, n in enumerate(names)]
    got = drain(eng, tasks)
    for t, n in zip(tasks, names):
        greedy_agrees(built, built.toks[n], got[t.task_id], F32)
    eng.close()


def test_engine_cancels_while_a_prompt_is_filling(built, monkeypatch):
    import exo_amd.engine as E
    monkeypatch.setattr(E, "PREFILL_STEP_SIZE", 16)
    asked: list = []
    eng = engine(built.models[F32], cancel_receiver=types.SimpleNamespace(collect=lambda: [asked.pop()] if asked else []))
    for i, n in enumerate(("d", "a", "b")):
        eng.submit(task(i, built.toks[n], 25))
    seen, k = {}, 0
    while sum(type(e).__name__ in ("FinishedResponse", "CancelledResponse") for v in seen.values() for e in v) < 3:
        if k == 4:
            asked.append("t1")
        for tid, ev in eng.step():
            seen.setdefault(tid, []).append(ev)
        k += 1
        assert k < 500
    assert [type(e).__name__ for e in seen["t1"]] == ["CancelledResponse"]
    for tid, n in (("t0", "d"), ("t2", "b")):
        toks = [e.token_id for e in seen[tid] if hasattr(e, "token_id")]
        assert len(toks) == 25
        greedy_agrees(built, built.toks[n], toks, F32)
    assert len(eng._gen.cache._free) == eng._gen.cache.n_pages
    eng.close()


def test_engine_prefix_cache_and_sequential(built):
    m = built.models[F32]
    kv = KVPrefixCache(None, "cuda:0")
    eng = engine(m, kv_prefix_cache=kv)
    p = built.toks["a"]
    first = drain(eng, [task(0, p, 12, use_prefix_cache=True)])["t0"]
    assert len(kv.caches) == 1
    again = drain(eng, [task(1, p, 12, use_prefix_cache=True)])["t1"]
    longer = drain(eng, [task(2, p + built.toks["d"], 12, use_prefix_cache=True)])["t2"]
    assert first == again
    greedy_agrees(built, p, first, F32)
    greedy_agrees(built, p + built.toks["d"], longer, F32)
    eng.close()
    seq = SequentialGenerator(model=m, tokenizer=None, model_id="gekazen", max_seq=512)
    got = drain(seq, [task(3, p, 12)])["t3"]
    greedy_agrees(built, p, got, F32)
    seq.close()


def test_paged_rows_travel_over_the_wire(built):
    """Keys and values of a paged row through the prefill wire format into another pool, whole and
    behind a prefix; head sizes or an element type that the format cannot say are refused."""
    import io

    from exo_amd import disaggregated as W

    cfg = U.config([U.layer(), U.layer(kv_from=0), U.layer(heads=4, kv_heads=4, window=50)])
    w = U.weights(cfg, 4)
    m = build_model(config_from_dict(cfg), U.torch_weights(w, "cuda"))
    toks = [t % cfg["vocab"] for t in built.toks["b"]]
    src, dst, ref = m.make_cache(2, 256), m.make_cache(2, 256), m.make_cache(1, 256)
    m.step(src, [(1, toks[:130], [])])
    m.step(dst, [(1, toks[:70], [])])
    for start in (0, 70):
        buf = io.BytesIO()
        assert W.write_cache_to_wire(buf, src, row=1, request_id="r", model_id="m", start_pos=start) == 130 - start
        buf.seek(0)
        row = 1 if start else 0
        assert W.ingest_into_cache(W.read_result(buf), dst, row=row, start_pos=start) == 130
        for i in range(len(src)):
            for a, b in zip(src.read_nhd(i, 1, 0, 130), dst.read_nhd(i, row, 0, 130)):
                assert torch.equal(a, b)
    m.step(ref, [(0, toks[:130], [])])
    want = host(m.step(ref, [(0, toks[130:133], [0, 1, 2])])).copy()
    got = host(m.step(dst, [(0, toks[130:133], [0, 1, 2])]))
    assert np.array_equal(got, want)
    for bad in (built.models[BF], build_model(config_from_dict(cfg), U.torch_weights(w, "cuda"), dtype=F32)):
        c = bad.make_cache(1, 64)
        bad.step(c, [(0, [1, 2, 3], [])])
        with pytest.raises(ValueError, match="the wire carries"):
            W.write_cache_to_wire(io.BytesIO(), c, row=0)


def test_engine_samples_on_device_and_on_host(built):
    """Sampled requests and one whose settings only the host takes share mixed steps."""
    g = ShardBatchGenerator(built.models[BF], None, 4, 512)
    par = dict(model="gekazen", max_output_tokens=15, bench=True, seed=5)
    g.submit(TextGenerationTaskParams(input=[], temperature=0.8, **par), built.toks["d"])
    g.submit(TextGenerationTaskParams(input=[], temperature=0.0, repetition_penalty=1.1, repetition_context_size=400,
                                      logprobs=True, **par), built.toks["c"])
    g.submit(TextGenerationTaskParams(input=[], temperature=0.8, top_k=5, **par), built.toks["b"])
    out: dict = {}
    while g.has_work:
        for uid, r in g.step():
            out.setdefault(uid, []).append(r)
    assert sorted(len(v) for v in out.values()) == [15, 15, 15]
    assert all(0 <= r.token < built.cfg["vocab"] for v in out.values() for r in v)
    assert out[1][0].logprob is not None
    g.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_generate_greedy(built, dtype):
    p = built.toks["c"]
    toks = [r.token for r in generate(built.models[dtype], None, TextGenerationTaskParams(
        model="gekazen", max_output_tokens=60, temperature=0.0), p)]
    assert len(toks) == 60
    greedy_agrees(built, p, toks, dtype)


def test_builder_serves_a_checkpoint(built, tmp_path):
    from exo_amd.engine import Mi355xBuilder
    from exo_amd.types import BoundInstance, ShardMetadata

    U.write_checkpoint(tmp_path, built.cfg, {k: np.asarray(v, np.float32) for k, v in built.w.items()})
    b = Mi355xBuilder(model_id="gekazen", max_seq=512)
    n = len(built.cfg["layers"])
    bound = BoundInstance(bound_shard=ShardMetadata(model_id="gekazen", start_layer=0, end_layer=n, n_layers=n),
                          model_path=str(tmp_path))
    b.connect(bound)
    assert [r.layers_loaded for r in b.load(bound)] == list(range(1, n + 1))
    eng = b.build()
    eng.warmup()
    got = drain(eng, [task(0, built.toks["d"], 10)])["t0"]
    greedy_agrees(built, built.toks["d"], got, BF)
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_program(built, tmp_path, dtype):
    root = Path(__file__).resolve().parent.parent
    U.write_checkpoint(tmp_path / "m", built.cfg, {k: np.asarray(v, np.float32) for k, v in built.w.items()})
    (tmp_path / "o").mkdir()
    t = built.toks
    steps = [dict(entries=[dict(id="x", tokens=t["b"][:100], want=[99, 3]), dict(id="y", tokens=t["d"][:2], want=[1])], end=[]),
             dict(entries=[dict(id="x", tokens=t["b"][100:101], want=[])], end=[]),
             dict(entries=[dict(id="y", tokens=t["d"][2:], want=[20]), dict(id="x", tokens=t["b"][101:103], want=[1, 0])],
                  end=["x", "y"]),
             dict(entries=[dict(id="z", tokens=t["d"], want=[22])], end=["z"])]
    text = "".join(json.dumps(dict(s, step=i)) + "\n" for i, s in enumerate(steps))
    r = subprocess.run([sys.executable, str(root / "bin" / "trace_run"), "--model", str(tmp_path / "m"), "--dtype",
                        str(dtype).split(".")[1], "--out", str(tmp_path / "o"), "--max-tokens", "192"],
                       input=text, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr
    assert [ln for ln in r.stdout.splitlines() if ln.startswith("done")] == ["done 0", "done 1", "done 2", "done 3"]
    assert not (tmp_path / "o" / "1.f32").exists()

    def rows(i):
        return np.fromfile(tmp_path / "o" / f"{i}.f32", "<f4").reshape(-1, built.cfg["vocab"])

    got = np.concatenate([rows(0), rows(2), rows(3)])
    want = np.stack([built.want["b"][99], built.want["b"][3], built.want["d"][1], built.want["d"][22],
                     built.want["b"][102], built.want["b"][101], built.want["d"][22]])
    assert U.rel_rms(got, want).max() < (1e-4 if dtype == F32 else 0.5)
