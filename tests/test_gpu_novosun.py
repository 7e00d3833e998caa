"""The Novosun design on the GPU against its plain oracle (``oracle/novosun.py``): its kernels alone, whole
models under every way to cut and batch sequences, and generation through the engines.  Float32 mode
is the sharp test, bf16 the served one."""

import json
import subprocess
import sys
import types
from pathlib import Path

import numpy as np
import pytest
import torch

from exo_amd import dense_ops as D
from exo_amd import disaggregated as W
from exo_amd import native
from exo_amd.engine import Mi355xBuilder, SequentialGenerator
from exo_amd.generate import generate
from exo_amd.paged_cache import PAGE, PagedKVCache
from exo_amd.prefix_cache import KVPrefixCache
from exo_amd.registry import build_model, config_from_dict
from exo_amd.stack_config import AttentionSpec, GluSpec
from exo_amd.types import BoundInstance, ShardMetadata, TextGenerationTaskParams
from oracle import novosun as O
from oracle.affine import bf16_round
from tests import novosun_util as U
from tests import stack_util as S
from tests.gekazen_util import rel_rms, torch_weights, write_checkpoint
from tests.stack_util import BF, DTYPES, F32, SCHEDULE, TOL, close, dev, drain, engine, host, mat, play, rand, task
from tests.util import rng

pytestmark = pytest.mark.gpu


def say(*a):
    print("[novosun]", *a, flush=True)


def f64(*arrays):
    return [np.asarray(a, np.float64) for a in arrays]


# ------------------------------------------------------------------ products and norms


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,N,nt,K", [(1, 50, 6, 72), (2, 4100, 33, 200), (16, 39, 1, 1000), (17, 300, 20, 2100), (40, 96, 5, 3000),
                                      (1000, 2900, 44, 320)])
def test_columns_that_leave_in_float32(device, dtype, M, N, nt, K):
    say("tail columns", dtype, M, N, nt, K)
    x, w, b = rand((M, K), 1), rand((N + nt, K), 2, K**-0.5), rand((N + nt,), 3)
    out, tail = torch.zeros(M, N + 3, dtype=dtype, device="cuda"), torch.zeros(M, nt + 2, dtype=F32, device="cuda")
    D.linear(mat(x, dtype), mat(w, dtype), out, M, bias=dev(b), tail=(tail, nt))
    want = x.astype(np.float64) @ w.T + b
    close(host(out[:, :N]), want[:, :N], 3 * TOL[dtype], "element type")
    close(host(tail[:, :nt]), want[:, N:], 2e-5, "float32")
    assert not host(out[:, N:]).any() and not host(tail[:, nt:]).any()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,N0,K0,N1,K1", [(1, 100, 72, 100, 200), (5, 17, 1000, 300, 64), (16, 4096, 128, 70, 320), (30, 90, 100, 50, 7)])
def test_two_products_in_a_launch(device, dtype, M, N0, K0, N1, K1):
    a, v, b, w = rand((M, K0), 1), rand((N0, K0), 2, K0**-0.5), rand((M, K1), 3), rand((N1, K1), 4, K1**-0.5)
    o0, o1 = torch.zeros(M, N0, device="cuda"), torch.zeros(M, N1, device="cuda")
    D.linear_pair(mat(a, dtype), mat(v, dtype), o0, mat(b, dtype), mat(w, dtype), o1, M)
    if M <= 16:
        assert "dual" in native.last_variant()
    close(host(o0), a.astype(np.float64) @ v.T, 2e-5, "first")
    close(host(o1), b.astype(np.float64) @ w.T, 2e-5, "second")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,N,K", [(1, 40, 72), (7, 4100, 100), (16, 330, 1000), (20, 130, 448)])
def test_gated_pair(device, dtype, M, N, K):
    x, g, u = rand((M, K), 1), rand((N, K), 2, 2 * K**-0.5), rand((N, K), 3, 2 * K**-0.5)
    out = torch.zeros(M, D.pad64(N), dtype=dtype, device="cuda")
    D.glu(mat(x, dtype), mat(g, dtype), mat(u, dtype), out, M, GluSpec(N, 1.3))
    x, g, u = f64(x, g, u)
    want = O.clamped_glu(x @ g.T, x @ u.T, 1.3)
    assert (x @ g.T > 1.3).any() and (np.abs(x @ u.T) > 1.3).any()
    close(host(out[:, :N]), want, 2 * TOL[dtype], "gated unit")


def branches(n, H, two):
    """(arrays of the test, D.Branches, what they add to the residual)"""
    y, y2, g, ga, gb, mult = rand((n, H), 2, 3e-3), rand((n, H), 6, 0.2), rand((H,), 3), rand((H,), 7), rand((H,), 8), 0.35
    eps = 1e-5  # of the order of mean(y^2)
    v = O.rms_norm(y.astype(np.float64), ga, eps) / 2 + O.rms_norm(y2.astype(np.float64), gb, eps) / 2 if two else y.astype(np.float64)
    br = D.Branches(dev(y), dev(g), mult, *((dev(y2), dev(ga), dev(gb)) if two else ()))
    return br, mult * O.rms_norm(v, g, eps), eps


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("two", [False, True])
@pytest.mark.parametrize("pre", [False, True])
@pytest.mark.parametrize("n,H", [(1, 70), (5, 1024), (40, 3001), (3, 9000)])
def test_residual_norms(device, dtype, n, H, two, pre):
    say("post norm", dtype, n, H, two, pre)
    x, gp = rand((n, H), 1), rand((H,), 9)
    br, add, eps = branches(n, H, two)
    xt, xb = dev(x), torch.zeros(n, D.pad64(H), dtype=dtype, device="cuda")
    D.post_norm_add(br, eps, xt, xb, n, dev(gp) if pre else None)
    close(host(xt), x + add, 1e-5, "residual")
    close(host(xb[:, :H]), O.rms_norm(x + add, gp, eps) if pre else x + add, TOL[dtype], "operand")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("two,pre,pair", [(True, True, True), (True, False, False), (False, True, True), (False, True, False)])
@pytest.mark.parametrize("n,H,N", [(1, 70, 40), (1, 4096, 5000), (2, 1021, 17), (3, 300, 130), (4, 2048, 331), (4, 1000, 18000)])
def test_residual_norms_inside_a_product(device, dtype, n, H, N, two, pre, pair):
    say("post product", dtype, n, H, N, two, pre, pair)
    x, gp = rand((n, H), 1), rand((H,), 9)
    w, u = rand((N, H), 4, H**-0.5), rand((N, H), 5, H**-0.5)
    br, add, eps = branches(n, H, two)
    A, B, xb = mat(w, dtype), mat(u, dtype), torch.zeros(n, D.pad64(H), dtype=dtype, device="cuda")
    if not native.load().exo_post_linear_fits(n, N, H, xb.shape[1], 0 if dtype == BF else 1):
        assert dtype == F32 or N == 18000  # too many columns for the launch's registers or LDS
        return
    xt, xo, tail = dev(x), torch.zeros(n, H, device="cuda"), torch.zeros(n, 3, device="cuda")
    out = torch.zeros(n, N, dtype=dtype if pair else F32, device="cuda")
    D.post_linear(xt, br, eps, xo, xb, A, out, n, tail=None if pair else (tail, 3), pre=dev(gp) if pre else None,
                  up=B if pair else None, spec=GluSpec(N, 0.9) if pair else None)
    close(host(xo), x + add, 1e-5, "residual")
    op = O.rms_norm(x + add, gp, eps) if pre else x + add
    close(host(xb[:, :H]), op, TOL[dtype], "operand")
    assert not host(xb[:, H:]).any() and np.array_equal(host(xt), x)
    op = host(xb[:, :H]).astype(np.float64)
    if pair:
        close(host(out), O.clamped_glu(op @ w.T, op @ u.T, 0.9), 2 * TOL[dtype], "gated pair")
    else:
        close(host(out[:, : N - 3]), (op @ w.T)[:, : N - 3], 2e-5, "product")
        close(host(tail), (op @ w.T)[:, N - 3 :], 2e-5, "its last columns")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,groups,period", [(72, 3, 24), (130, 1, 130), (4096, 4, 4096), (2048, 16, 128), (700, 7, 100)])
@pytest.mark.parametrize("first", [True, False])
def test_gated_norm(device, dtype, width, groups, period, first):
    n, eps = 5, 1e-3
    y, z, g = rand((n, width), 1, 0.05), rand((n, width + 8), 2, 2.0), rand((period,), 3)
    out = torch.zeros(n, D.pad64(width), dtype=dtype, device="cuda")
    D.gated_norm(dev(y), dev(z, dtype), dev(g), out, n, width, groups, eps, first)
    y, z, g = f64(y, z[:, :width], np.tile(g, width // period))
    want = O.grouped_norm(y * O.silu(z), g, groups, eps) if first else O.grouped_norm(y, g, groups, eps) * O.silu(z)
    close(host(out[:, :width]), want, 2 * TOL[dtype], "gated norm")


# ------------------------------------------------------------------ attention


ATT_SHAPES = [(6, 3, 24, 40), (5, 5, 64, 32), (8, 2, 128, 96), (5, 1, 36, 7), (4, 2, 40, 256), (16, 1, 64, 64)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", ATT_SHAPES)
def test_gated_attention(device, dtype, shape):
    """Normed queries and keys with gains, a gate per head, no positions: portions and single tokens.
    Planted queries each see one far key that carries most of the weight, at page and tile borders and
    at the sequence's first position."""
    H, G, De, E = shape
    T, eps, far = 200, 0.2, {60: 0, 90: 63, 91: 64, 130: 31, 131: 32, 150: 127, 170: 128, 199: 1}
    spec = AttentionSpec(H, G, De, E, 3.0 / np.sqrt(De), unit_qk=True, qk_gain=True, head_gate=True)
    say("attention", dtype, shape)
    q, k, v, gate = rand((T, H, De), 1), rand((T, G, De), 2), rand((T, G, E), 3), rand((T, H + 3), 4, 2.0)
    qg, kg = bf16_round(1 + rand((De,), 5, 0.3)), bf16_round(1 + rand((De,), 6, 0.3))
    for i, j in far.items():
        q[i] = bf16_round(4 * k[j][np.arange(H) // (H // G)])
    qn, kn = (O.rms_norm(a.astype(np.float64), g, eps) for a, g in ((q, qg), (k, kg)))
    if dtype == BF:  # as the kernels hold them
        qn, kn = (bf16_round(a.astype(np.float32)).astype(np.float64) for a in (qn, kn))
    want = O.attend(qn, kn, v.astype(np.float64), spec.scale) * O.sigmoid(gate[:, :H].astype(np.float64))[:, :, None]
    rows = np.concatenate([a.reshape(T, -1) for a in (q, k, v)], 1)
    i32 = dict(dtype=torch.int32, device="cuda")
    for cuts in ([T], [3, 2, 64, 1, 60, 2, 2, 500], [58] + [1] * T):
        cache = PagedKVCache([(G, De, E)], 2, 512, "cuda", dtype)
        att, at, got = D.PagedAttention(spec, None, 0, cache, eps, dev(qg), dev(kg)), 0, []
        cache.reserve([0], 70)
        for n in cuts:
            n = min(n, T - at)
            if n <= 0:
                break
            cache.reserve([1], n)
            slot, pos = torch.full((n,), 1, **i32), torch.arange(at, at + n, **i32)
            qkv = torch.zeros(n, 8 + -(-rows.shape[1] // 8) * 8, dtype=dtype, device="cuda")  # (not from column 0)
            qkv[:, 8 : 8 + rows.shape[1]].copy_(dev(rows[at : at + n]))
            qkv, gt, o = qkv[:, 8:], dev(gate[at : at + n]), torch.zeros(n, D.pad64(H * E), dtype=dtype, device="cuda")
            if n == 1:
                att.rows(qkv, o, slot, pos, 1, at + 1, append=True, gate=gt)
            else:
                att.append(qkv, slot, pos, n)
                if dtype == F32:
                    att.rows(qkv, o, slot, pos, n, at + n, append=False, gate=gt)
                else:
                    bs = att.prompt_block(spec)
                    blocks = torch.tensor([(b, 1, at + b, min(bs, n - b)) for b in range(0, n, bs)], **i32)
                    att.prompt(qkv, o, blocks, blocks.shape[0], gate=gt)
            got.append(host(o[:, : H * E]).reshape(n, H, E))
            cache.advance_host(n, [1])
            at += n
        close(np.concatenate(got), want, 2e-2 if dtype == BF else 5e-5, f"{shape} {cuts[:3]}")


# ------------------------------------------------------------------ recurrences


def one_layer(layer, w_edit=None, dtype=F32, width=72, seed=3, rank=10):
    """(model of one layer, its oracle weights); ``w_edit`` changes the weights in place."""
    cfg = U.config([layer], width=width)
    w = U.weights(cfg, seed, rank)
    if w_edit is not None:
        w_edit(w)
    return build_model(config_from_dict(cfg), torch_weights(w, "cuda"), dtype=dtype), w


def run_part(model, part, y, y2, schedule, rows=3):
    """The recurrence of ``model``'s layer over given projection columns, sequence by sequence:
    ``schedule``: steps of [(sequence, tokens)]; ``y``, ``y2``: per sequence its columns.  Returns what it
    leaves ahead of its gated norm, per sequence."""
    cache = model.make_cache(rows, 1024)
    op, p, at, got = model._mixers(cache)[0][part], model.layers[0].parts[part], {}, {}
    for step in schedule:
        counts, ys, y2s = [], [], []
        for s, n in step:
            a = at.get(s, 0)
            n = min(n, len(y[s]) - a)
            if n > 0:
                counts.append((s, n))
                ys.append(y[s][a : a + n])
                y2s.append(y2[s][a : a + n])
        if not counts:
            continue
        cache.reserve_each(counts)
        n = sum(c for _, c in counts)
        b, bf = model._batch(cache, counts, []), model._buffers(1, max(n, 2))
        p.run(op, bf, b, dev(np.concatenate(ys), model.dtype), dev(np.concatenate(y2s)), model.cfg.eps)
        o, k = host(bf.f32("recur", p.width)[:n]), 0
        for s, c in counts:
            got.setdefault(s, []).append(o[k : k + c].copy())
            at[s] = at.get(s, 0) + c
            k += c
            cache.advance_host(c, [s])
        cache.sync_pos()
    return {s: np.concatenate(v) for s, v in got.items()}


CUTS = [[500], [2] * 250, [1] * 500, [64, 1, 63, 65, 64, 500], [3, 61, 2, 1, 1, 62, 128, 500], [15, 17, 16, 48, 33, 500]]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,vdim,tau,rank", [(3, 40, 24, 5.0, 10), (1, 72, 136, 0.5, 4), (2, 128, 64, 16.0, 16), (4, 16, 20, 1.0, 33),
                                                     (2, 7, 5, 2.0, 1)])
def test_decay_per_channel(device, dtype, heads, dim, vdim, tau, rank):
    """Channels that forget within a token beside channels that keep everything; keys planted a chunk and
    several chunks back that decide their queries' outputs."""
    m, w = one_layer(U.linear(heads, dim, vdim, tau), dtype=dtype, rank=rank)
    T = 210
    hd, he = heads * dim, heads * vdim
    y = rand((T, 2 * hd + 2 * he), 1)
    low = rand((T, rank), 2, 1.0)
    b = w["l0.mix.a2.b"].reshape(heads, dim)
    keep = np.argmax(b, axis=1)  # per head, the channel that forgets least
    far = {64: 63, 70: 0, 128: 64, 130: 62, 200: 5, 209: 127}
    for h in range(heads):
        w["l0.mix.a2"].reshape(heads, dim, rank)[h, keep[h]] = 0
        b[h, keep[h]] = 20.0
        q, k = y[:, h * dim : (h + 1) * dim], y[:, hd + h * dim : hd + (h + 1) * dim]
        k[:, keep[h]] = 0
        for n, (i, j) in enumerate(far.items()):
            q[i], k[j, keep[h]] = 0, 30.0 + n
            q[i, keep[h]] = 8.0
    p = m.layers[0].parts[0]
    p.decay_w.copy_(dev(w["l0.mix.a2"].T))
    p.decay_b.copy_(dev(w["l0.mix.a2.b"]))
    y, low = y.astype(np.float32), low.astype(np.float32)
    z = low.astype(np.float64) @ w["l0.mix.a2"].T.astype(np.float64) + w["l0.mix.a2.b"]
    a = np.exp(-O.softplus(-z) / tau).reshape(T, heads, dim)
    yy = y.astype(np.float64)
    q, k = (yy[:, i * hd : (i + 1) * hd].reshape(T, heads, dim) for i in (0, 1))
    v = yy[:, 2 * hd : 2 * hd + he].reshape(T, heads, vdim)
    want = np.stack([O.recurrence(q[:, h] / np.sqrt(dim), k[:, h], v[:, h], a[:, h])[0] for h in range(heads)], 1).reshape(T, he)
    for cuts in CUTS:
        say("channel decay", dtype, heads, dim, vdim, tau, cuts[:4])
        got = run_part(m, 0, {1: y}, {1: low}, [[(1, n)] for n in cuts])[1]
        err = np.abs(got - want).max(-1) / np.sqrt(np.mean(want**2, -1) + 1e-3)
        assert err.max() < (3e-3 if dtype == BF else 6e-5), f"{cuts[:4]}: {err.max():.1e} at {int(err.argmax())}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,vdim,state,groups,conv", [(6, 20, 12, 3, 4), (2, 70, 88, 1, 1), (4, 64, 128, 2, 2), (5, 16, 16, 5, 9), (3, 5, 7, 1, 3)])
def test_decay_per_head(device, dtype, heads, vdim, state, groups, conv):
    """Convolution, step sizes, grouped keys and queries, skip: heads that forget at once and heads that keep
    everything; two sequences in one batch."""
    layer = U.parallel(ssm_heads=heads, ssm_vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=heads)

    def edit(w):
        w["l0.mix.right.A_log"][:] = np.linspace(-7, 2, heads)
        w["l0.mix.right.dt_bias"][:] = np.linspace(-1, 1.5, heads)
    m, w = one_layer(layer, edit, dtype)
    spec, p = layer["mixer"]["right"], m.layers[0].parts[1]
    inner, ch = heads * vdim, heads * vdim + 2 * groups * state
    w = {k: bf16_round(v) for k, v in w.items()}
    seqs = {s: (rand((T, ch), 10 + s), rand((T, heads), 20 + s)) for s, T in ((0, 90), (2, 210))}
    for x, dt in seqs.values():  # a planted input far from where it is asked for
        x[5, inner:], x[-1, inner:], dt[5] = 3.0, 3.0, 4.0
    want = {s: U.ssm_oracle(w, spec, x, dt, bf16_round if dtype == BF else None) for s, (x, dt) in seqs.items()}
    off = p.col + -(-inner // 8) * 8
    y, y2 = {}, {}
    for s, (x, dt) in seqs.items():
        y[s] = np.zeros((len(x), -(-m.layers[0].n_main // 8) * 8), np.float32)
        y[s][:, off : off + ch] = x
        y2[s] = np.zeros((len(x), m.layers[0].n_tail), np.float32)
        y2[s][:, p.tcol : p.tcol + heads] = dt
    for cuts in CUTS:
        say("head decay", dtype, heads, vdim, state, groups, conv, cuts[:4])
        other = [40, 1, 1, 2, 70] + [3] * 500
        got = run_part(m, 1, y, y2, [[(2, n), (0, k)] for n, k in zip(cuts, other)] + [[(0, 9), (2, 100)]] * 30)
        for s in got:
            err = np.abs(got[s] - want[s]).max(-1) / np.sqrt(np.mean(want[s] ** 2, -1) + 1e-2)
            assert err.max() < (2e-2 if dtype == BF else 6e-5), f"{cuts[:4]}, {s}: {err.max():.1e} at {int(err.argmax())}"


# ------------------------------------------------------------------ whole models


@pytest.fixture(scope="module")
def built():
    """(config, float64 weights, {dtype: model}, tokens, oracle logits) of the mixed configuration."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg = U.mixed_config()
    w = U.weights(cfg, 11)
    models = {t: build_model(config_from_dict(cfg), torch_weights(w, "cuda"), dtype=t) for t in DTYPES}
    toks = {name: rng(s).integers(0, cfg["vocab"], n).tolist() for s, (name, n) in
            enumerate({"a": 300, "b": 141, "c": 64, "d": 23, "e": 1}.items())}
    w64 = O.to_float64(w)
    want = {k: O.forward(cfg, w64, t) for k, t in toks.items()}
    return types.SimpleNamespace(cfg=cfg, w=w64, models=models, toks=toks, want=want)


LIMIT = {BF: 8e-2, F32: 1e-4}  # of the worst position; a typical one in bf16: 1e-2


def check_rows(built, dtype, name, places, logits, what):
    err = rel_rms(logits, built.want[name][places])
    say(what, f"worst {err.max():.1e}")
    assert err.max() < LIMIT[dtype], f"{what}: {err.max():.2e} at {places[int(err.argmax())]}"
    assert np.median(err) < LIMIT[dtype] / 4, f"{what}: median {np.median(err):.2e}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("portion", [300, 1, 2, 3, 17, 64, 65, 128])
def test_model_in_portions(built, dtype, portion):
    for name in built.toks if portion in (300, 1) else ("a", "c"):
        got = play(built.models[dtype], built.toks, [[(name, portion)]] * 300, max_tokens=320)[name]
        check_rows(built, dtype, name, np.arange(len(got)), got, f"portions of {portion}, {name}")


@pytest.mark.parametrize("dtype", DTYPES)
def test_model_layers(built, dtype):
    m, outs, want = built.models[dtype], [], []
    O.forward(built.cfg, built.w, built.toks["c"], want)
    m.layer_hook = lambda i, h: outs.append(host(h).copy())
    try:
        play(m, built.toks, [[("c", 64)]])
    finally:
        m.layer_hook = None
    for i, (g, w) in enumerate(zip(outs, want)):
        err = rel_rms(g, w)
        assert err.max() < (3e-2 if dtype == BF else 3e-5), f"layer {i}: {err.max():.2e}"


@pytest.mark.parametrize("dtype", DTYPES)
def test_model_mixed_batches_reuse_rows_pages_and_slots(built, dtype):
    got = play(built.models[dtype], built.toks, SCHEDULE, max_tokens=640)
    for name, lg in got.items():
        check_rows(built, dtype, name.split("#")[0], np.arange(len(lg)), lg, f"mixed, {name}")


def test_slots_hold_nothing_over(built):
    """A row that served another sequence, was cut off in the middle or moved: the next sequence starts from
    nothing, and a moved one goes on."""
    m, t = built.models[F32], built.toks
    c = m.make_cache(3, 320)
    m.step(c, [(0, t["a"][:77], []), (1, t["b"][:50], [])])
    c.release(0)
    err = rel_rms(host(m.step(c, [(0, t["c"], [63])])), built.want["c"][63:])
    assert err.max() < 1e-4
    c.copy_row(1, 2)  # slots and pages change hands
    assert rel_rms(host(m.step(c, [(2, t["b"][50:60], [9])])), built.want["b"][59:60]).max() < 1e-4
    c.swap_rows(0, 2)
    lg = host(m.step(c, [(1, t["d"][:1], [0]), (0, t["b"][60:61], [0])]))
    assert rel_rms(lg, np.stack([built.want["d"][0], built.want["b"][60]])).max() < 1e-4
    with pytest.raises(ValueError, match="cut back"):
        c.trim(1, rows=[0])
    c.trim(61, rows=[0])  # to nothing is the same as a reset
    assert rel_rms(host(m.step(c, [(0, t["d"], [22])])), built.want["d"][22:]).max() < 1e-4


@pytest.mark.parametrize("B", [1, 3, 4, 16, 20])
def test_model_graph_decode_matches_steps(built, B):
    """The captured single-token step over B rows (capturing must not advance a state), several replays with
    eager work between them."""
    m = built.models[F32]
    cache = m.make_cache(B + 1, 320)
    seqs = [built.toks[n][o:] for o in range(8) for n in ("a", "b", "c")][:B]
    n0, n1 = 30, 46
    m.step(cache, [(r, s[: n0 - r % 7], []) for r, s in enumerate(seqs)])
    pos = [n0 - r % 7 for r in range(B)]
    wants = [O.forward(built.cfg, built.w, s[:n1]) for s in seqs]
    for k in range(n1 - n0):
        bf = m._buffers(B, 1)
        bf.tokens.copy_(torch.tensor([s[p] for s, p in zip(seqs, pos)], dtype=torch.int32))
        bf = m.decode_step(cache, B)
        err = rel_rms(host(bf.logits), np.stack([w[p] for w, p in zip(wants, pos)]))
        assert err.max() < 1e-4, f"step {k}: {err.max():.2e}"
        pos = [p + 1 for p in pos]
        torch.randn(1000, device="cuda").sum().item()


def test_model_long_decode(built):
    m, toks = built.models[F32], rng(77).integers(0, built.cfg["vocab"], 560).tolist()
    want = O.forward(built.cfg, built.w, toks)
    cache = m.make_cache(1, 600)
    m.step(cache, [(0, toks[:150], [])])
    bf = m._buffers(1, 1)
    for i in range(150, 560):
        bf.tokens[0] = toks[i]
        err = rel_rms(host(m.decode_step(cache, 1).logits), want[i : i + 1]).max()
        assert err < 1e-4, f"position {i}: {err:.2e}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layers", [
    [U.linear(), U.linear(heads=2, dim=24, vdim=72, ff=None)],  # nothing is kept per token
    [U.parallel(ff=None), U.parallel(kv_heads=6, groups=6, norm_groups=6, conv=2)],
    [U.parallel(heads=2, kv_heads=1, dim=200, vdim=130, ssm_heads=1, ssm_vdim=200, state=130, groups=1, norm_groups=4, ff=300)]])
def test_other_orders_and_sizes(device, dtype, layers):
    cfg = U.config(layers, width=130, vocab=97, eps=3e-3, mult=1.0)
    w = U.weights(cfg, 5, rank=19)
    m = build_model(config_from_dict(cfg), torch_weights(w, "cuda"), dtype=dtype)
    toks = {"a": rng(1).integers(0, 97, 140).tolist(), "b": rng(2).integers(0, 97, 9).tolist()}
    want = {k: O.forward(cfg, w, t) for k, t in toks.items()}
    for sched in ([[("a", 140)]], [[("a", 70), ("b", 1)], [("b", 2), ("a", 3)]] + [[("a", 1), ("b", 1)]] * 90):
        for k, lg in play(m, toks, sched, max_tokens=256).items():
            assert rel_rms(lg, want[k]).max() < LIMIT[dtype]


@pytest.mark.parametrize("dtype", DTYPES)
def test_recurrences_with_many_heads(device, dtype):
    """Enough heads that a portion's states are carried in wide tiles."""
    for layer in (U.linear(heads=64, dim=64, vdim=256), U.parallel(ssm_heads=128, ssm_vdim=64, state=128, groups=2, norm_groups=4)):
        cfg = U.config([dict(layer, mlp=None)], width=64)
        w = U.weights(cfg, 7)
        m = build_model(config_from_dict(cfg), torch_weights(w, "cuda"), dtype=dtype)
        toks = {"a": rng(1).integers(0, cfg["vocab"], 200).tolist()}
        want = O.forward(cfg, w, toks["a"])
        for sched in ([[("a", 200)]], [[("a", 70)], [("a", 129)], [("a", 1)]]):
            assert rel_rms(play(m, toks, sched)["a"], want).max() < (3e-2 if dtype == BF else 1e-4)


def test_model_pipeline_shards(built):
    w = torch_weights({k: np.asarray(v, np.float32) for k, v in built.w.items()}, "cuda")
    c = config_from_dict(built.cfg)
    n = c.num_hidden_layers
    x, y = build_model(c, w, 0, 3, dtype=F32), build_model(c, w, 3, n, dtype=F32)
    cx, cy = x.make_cache(1, 100), y.make_cache(1, 100)
    toks = built.toks["a"]
    for lo, hi in ((0, 30), (30, 31), (31, 60)):
        got = y(None, cy, input_embeddings=x(torch.tensor([toks[lo:hi]]), cx), logits="last")
        assert rel_rms(host(got)[0], built.want["a"][hi - 1 : hi]).max() < 1e-4


# ------------------------------------------------------------------ generation


def greedy_agrees(built, prompt, got, dtype):
    S.greedy_agrees(lambda toks: O.forward(built.cfg, built.w, toks), prompt, got, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_engine_mixes_prompts_into_running_batches(built, dtype, monkeypatch):
    import exo_amd.engine as E
    monkeypatch.setattr(E, "PREFILL_STEP_SIZE", 37)
    m, kinds = built.models[dtype], []
    eng, step = engine(m), m.step
    monkeypatch.setattr(m, "step", lambda c, e: (kinds.append(tuple(sorted({len(t) > 1 for _, t, _ in e}))), step(c, e))[1])
    names = ["a", "d", "b", "c", "e", "b"]
    tasks = [task(i, built.toks[n], 20 + 3 * i) for i, n in enumerate(names)]
    got = drain(eng, tasks, join_at=[0, 2, 9, 12, 30, 41])
    assert (False, True) in kinds  # single tokens and portions together
    for t, n in zip(tasks, names):
        assert len(got[t.task_id]) == t.task_params.max_output_tokens
        greedy_agrees(built, built.toks[n], got[t.task_id], dtype)
    c = eng._gen.cache
    assert len(c._free) == c.n_pages and sorted(c.states.slot) == list(range(c.batch))
    eng.close()


def test_engine_waits_for_pages_and_warms_up(built):
    eng = engine(built.models[F32], pool_tokens=8 * PAGE)
    eng.warmup()
    names = ["a", "b", "b", "c", "a"]
    tasks = [task(i, built.toks[n], 30) for i, n in enumerate(names)]
    got = drain(eng, tasks)
    for t, n in zip(tasks, names):
        greedy_agrees(built, built.toks[n], got[t.task_id], F32)
    eng.close()


@pytest.mark.parametrize("kind", ["batch", "sequential"])
def test_prefix_cache_goes_on_only_from_where_a_state_stands(built, kind):
    m, p, d = built.models[F32], built.toks["a"], built.toks["d"]
    kv = KVPrefixCache(None, "cuda:0")
    eng = engine(m, kv_prefix_cache=kv) if kind == "batch" else SequentialGenerator(
        model=m, tokenizer=None, model_id="m", max_seq=512, kv_prefix_cache=kv)
    hits = []
    find = kv.get_kv_cache
    kv.get_kv_cache = lambda *a, **k: (lambda r: (hits.append(r[2] is not None), r)[1])(find(*a, **k))
    prompts = [p, p, p + d, p[:100] + d]  # new, the same, one that goes on, one that leaves it in the middle
    for i, q in enumerate(prompts):
        got = drain(eng, [task(i, q, 12, use_prefix_cache=True)])[f"t{i}"]
        greedy_agrees(built, q, got, F32)
    assert hits == [False, True, True, False]
    eng.close()


def test_states_do_not_travel(built):
    import io
    m = built.models[BF]
    c = m.make_cache(1, 64)
    m.step(c, [(0, [1, 2, 3], [])])
    with pytest.raises(ValueError, match="no recurrent states"):
        W.write_cache_to_wire(io.BytesIO(), c, row=0)
    eng = engine(m)
    with pytest.raises(ValueError, match="recurrent states"):
        eng.serve_prefill(W.PrefillRequest("r", "m", [1, 2, 3, 4], 0), io.BytesIO())
    # a task that names a prefill server is prefilled here
    got = drain(eng, [task(0, (built.toks["a"] * 4)[:450], 5, prefill_endpoint="127.0.0.1:1")])["t0"]
    assert len(got) == 5
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_generate_greedy(built, dtype):
    p = built.toks["c"]
    toks = [r.token for r in generate(built.models[dtype], None, TextGenerationTaskParams(
        model="m", max_output_tokens=60, temperature=0.0), p)]
    assert len(toks) == 60
    greedy_agrees(built, p, toks, dtype)


def test_builder_serves_a_checkpoint(built, tmp_path):
    write_checkpoint(tmp_path, built.cfg, {k: np.asarray(v, np.float32) for k, v in built.w.items()})
    n = len(built.cfg["layers"])
    b = Mi355xBuilder(model_id="m", max_seq=512)
    bound = BoundInstance(bound_shard=ShardMetadata(model_id="m", start_layer=0, end_layer=n, n_layers=n), model_path=str(tmp_path))
    b.connect(bound)
    assert [r.layers_loaded for r in b.load(bound)] == list(range(1, n + 1))
    eng = b.build()
    eng.warmup()
    greedy_agrees(built, built.toks["d"], drain(eng, [task(0, built.toks["d"], 10)])["t0"], BF)
    eng.close()


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_program(built, tmp_path, dtype):
    root = Path(__file__).resolve().parent.parent
    write_checkpoint(tmp_path / "m", built.cfg, {k: np.asarray(v, np.float32) for k, v in built.w.items()})
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
    got = np.concatenate([np.fromfile(tmp_path / "o" / f"{i}.f32", "<f4").reshape(-1, built.cfg["vocab"]) for i in (0, 2, 3)])
    want = np.stack([built.want["b"][99], built.want["b"][3], built.want["d"][1], built.want["d"][22],
                     built.want["b"][102], built.want["b"][101], built.want["d"][22]])
    assert rel_rms(got, want).max() < LIMIT[dtype]
