"""The Pimisun design on the GPU against its plain oracle (``oracle/pimisun.py``): its kernels alone, whole
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
from exo_amd.stack_config import AttentionSpec, NormSpec, RotarySpec
from exo_amd.types import BoundInstance, ShardMetadata, TextGenerationTaskParams
from oracle import pimisun as O
from oracle.affine import bf16_round
from tests import pimisun_util as U
from tests import stack_util as S
from tests.gekazen_util import rel_rms, torch_weights, write_checkpoint
from tests.stack_util import BF, DTYPES, F32, SCHEDULE, TOL, close, dev, drain, engine, host, mat, play, rand, task
from tests.util import rng

pytestmark = pytest.mark.gpu
I32 = dict(dtype=torch.int32, device="cuda")


def say(*a):
    print("[pimisun]", *a, flush=True)


def f64(*arrays):
    return [np.asarray(a, np.float64) for a in arrays]


# ------------------------------------------------------------------ products and norms


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("act", ["relu2", "gelu_tanh", None])
@pytest.mark.parametrize("M,N,K", [(1, 50, 72), (4, 3, 1100), (16, 4100, 200), (17, 300, 2100), (40, 96, 3000), (700, 1500, 320)])
def test_products_with_an_activation_and_a_table(device, dtype, act, M, N, K):
    say("after", dtype, act, M, N, K)
    x, w = rand((M, K), 1), rand((N, K), 2, K**-0.5)
    table, rows = rand((9, N + 11), 3), rng(4).integers(0, 9, M).astype(np.int32)
    out = torch.zeros(M, D.pad64(N), dtype=dtype, device="cuda")
    tab = dev(table, dtype)[:, 5 : 5 + N]
    D.linear(mat(x, dtype), mat(w, dtype), out, M, after=D.After(act, tab, dev(rows, torch.int32)))
    z = np.asarray(x, np.float64) @ w.T
    f = {"relu2": O.relu_squared, "gelu_tanh": O.gelu_tanh, None: lambda v: v}[act]
    close(host(out[:, :N]), f(z) * table[rows, 5 : 5 + N], 2 * TOL[dtype], "with a table")
    assert not host(out[:, N:]).any()
    D.linear(mat(x, dtype), mat(w, dtype), out, M, after=D.After(act, dev(table[np.arange(M) % 9][:, :N], dtype)))
    close(host(out[:, :N]), f(z) * table[np.arange(M) % 9][:, :N], 2 * TOL[dtype], "a row each")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,H", [(1, 72), (3, 130), (4, 1024), (2, 2048), (5, 4100), (300, 700)])
@pytest.mark.parametrize("center", [True, False])
def test_norm_of_the_sum(device, dtype, n, H, center):
    """By itself, ahead of a product, and with the experts' sum; a mean far from zero."""
    x, y, g, eps = rand((n, H), 1, 2.0) + 3, rand((n, H), 2) - 9, rand((H,), 3), 0.3
    norm = NormSpec(eps, of_sum=True, keep=0.7, center=center)
    f = O.layer_norm if center else O.rms_norm
    say("norm of the sum", dtype, n, H, center)
    want = f(0.7 * x.astype(np.float64) + y, g, eps)
    xt, xb = dev(x), torch.zeros(n, D.pad64(H), dtype=dtype, device="cuda")
    D.post_norm_add(D.Branches(dev(y), dev(g), norm=norm), eps, xt, xb, n)
    close(host(xt), want, 2e-5, "residual")
    close(host(xb[:, :H]), want, TOL[dtype], "operand")
    xt, w, N = dev(x), rand((40, H), 5, H**-0.5), 40
    if native.load().exo_post_linear_fits(n, N, H, xb.shape[1], 0 if dtype == BF else 1):
        xo, out = torch.zeros_like(xt), torch.zeros(n, 64, device="cuda")
        D.post_linear(xt, D.Branches(dev(y), dev(g), norm=norm), eps, xo, xb.zero_(), mat(w, dtype), out, n)
        close(host(xo), want, 2e-5, "residual ahead of a product")
        close(host(out[:, :N]), host(xb[:, :H]).astype(np.float64) @ w.T, 2e-5, "product")
    z = rand((n, 3, H), 6)
    idx, wt = np.tile(np.array([2, 0, 1], np.int32), (n, 1)), rand((n, 3), 7)
    sh = rand((n, H), 8)
    yt = torch.zeros(n, 3, H, dtype=dtype, device="cuda").copy_(dev(z))
    xt = dev(x)
    D.moe_sum_post_norm(yt, dev(idx, torch.int32), dev(wt), dev(sh, dtype), dev(rand((n, 3), 9)), 3, -1, dev(g), eps, xt, xb, n, norm=norm)
    want = f(0.7 * x.astype(np.float64) + (z.astype(np.float64) * wt[:, :, None]).sum(1) + sh, g, eps)
    close(host(xt), want, 5e-5, "with the experts' sum")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,R,N", [(1, 36, 50), (4, 1536, 300), (3, 20, 700), (7, 200, 33), (40, 130, 90)])
def test_product_of_a_normed_part(device, dtype, n, R, N):
    x, g, w, eps = rand((n, R + 21), 1, 3.0), rand((R,), 2), rand((N, R), 3, R**-0.5), 0.02
    say("normed part", dtype, n, R, N)
    xt = torch.zeros(n, -(-(R + 21) // 8) * 8, device="cuda")
    xt[:, : R + 21] = dev(x)
    op, out = (torch.zeros(n, D.pad64(k), dtype=dtype, device="cuda") for k in (R, N))
    D.norm_linear(xt, dev(g), eps, op, mat(w, dtype), out, n)
    want = O.rms_norm(x[:, :R].astype(np.float64), g, eps) @ w.T
    close(host(out[:, :N]), want, 2 * TOL[dtype], "product")
    xc = dev(x[:, :R]) + 5
    D.norm_rows(xc, dev(g), eps, op, n, center=True)
    close(host(op[:, :R]), O.layer_norm(x[:, :R].astype(np.float64) + 5, g, eps), max(TOL[dtype], 5e-5), "centered rows")


@pytest.mark.parametrize("rows,E,top", [(1, 5, 3), (9, 64, 1), (33, 130, 8), (4, 300, 64), (2, 7, 7)])
def test_routing_among_the_chosen(device, rows, E, top):
    z = rand((rows, E + 2), 1, 3.0)
    z[0, 1] = z[0, 3] = 20.0  # equals: the lower index first
    idx, wt = torch.zeros(rows, top, **I32), torch.zeros(rows, top, device="cuda")
    D.moe_route(dev(z), torch.zeros(E, device="cuda"), 1.0, idx, wt, rows, renorm=True)
    for t in range(rows):
        ids, w = O.route(z[t, :E].astype(np.float64), top)
        assert idx[t].tolist() == list(ids)
        close(host(wt[t]), w, 1e-5, "weights")


# ------------------------------------------------------------------ attention


def unrotated(x, i, base, dims):
    """What rotation at position i turns into x [heads, D]."""
    flip = np.where(np.arange(x.shape[-1]) < dims, np.where(np.arange(x.shape[-1]) % 2, -1.0, 1.0), 1.0)
    a = np.zeros((i + 1, *x.shape))
    a[i] = x * flip
    return O.rotate(a, base, dims)[i] * flip


ATT_SHAPES = [(6, 2, 32, 24, 24, 8, 12.0), (4, 4, 40, 12, 1, 40, 3.0), (8, 2, 68, 24, 70, 2, None), (5, 1, 64, 48, 131, 64, 50.0),
              (2, 1, 256, 136, 64, 200, 20.0), (16, 1, 128, 128, None, 128, 30.0), (3, 3, 25, 7, 65, 24, 9.0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", ATT_SHAPES)
def test_attention(device, dtype, shape):
    """Norms over the whole projections, rotation, bent scores, a window, mixed values: portions and single
    tokens.  Planted queries each see one key that carries most of the weight, or would if it were seen: the
    last inside and the first outside the window, at page borders and the sequence's first position."""
    H, G, De, E, win, rot, cap = shape
    T, eps, base, lam = 200, 0.2, 400.0, 0.3
    spec = AttentionSpec(H, G, De, E, 3.0 / np.sqrt(De), window=win, whole_norm=True, rot=RotarySpec(base, rot), softcap=cap, v_mix_from=0)
    say("attention", dtype, shape)
    q, k, v, first = rand((T, H, De), 1), rand((T, G, De), 2), rand((T, G * E), 3), rand((T, G * E), 4)
    qg, kg = bf16_round(1 + rand((H * De,), 5, 0.3)), bf16_round(1 + rand((G * De,), 6, 0.3))
    kn = O.rotate(O.rms_norm(k.reshape(T, -1).astype(np.float64), kg, eps).reshape(T, G, De), base, rot)
    w = win or 10 ** 6
    far = {i: j for i, j in {60: 0, 90: 63, 91: 64, 130: 31, 150: 127, 170: 128, 199: 1}.items() if i - j < w}
    for i in (65, 100, 128, 140, 195):
        for d in (w - 1, w):
            if 0 <= i - d:
                far[i + (d == w)] = i + (d == w) - d
    for i, j in far.items():
        x = unrotated(kn[j][np.arange(H) // (H // G)], i, base, rot)
        q[i] = bf16_round((x / qg.reshape(H, De)).astype(np.float32))
    qn = O.rotate(O.rms_norm(q.reshape(T, -1).astype(np.float64), qg, eps).reshape(T, H, De), base, rot)
    vm = (1 - lam) * v.astype(np.float64) + lam * first
    if dtype == BF:  # as the kernels hold them
        qn, kn, vm = (bf16_round(a.astype(np.float32)).astype(np.float64) for a in (qn, kn, vm))
    want = O.attend(qn, kn, vm.reshape(T, G, E), spec.scale, win, cap)
    rows = np.concatenate([a.reshape(T, -1) for a in (q, k, v)], 1)
    freq = torch.tensor(spec.rot.turns(), dtype=torch.float64, device="cuda")
    for cuts in ([T], [3, 2, 64, 1, 60, 2, 2, 500], [58] + [1] * T):
        cache = PagedKVCache([(G, De, E)], 2, 512, "cuda", dtype)
        att, at, got = D.PagedAttention(spec, None, 0, cache, eps, dev(qg), dev(kg), freq), 0, []
        cache.reserve([0], 70)
        for n in cuts:
            n = min(n, T - at)
            if n <= 0:
                break
            cache.reserve([1], n)
            slot, pos = torch.full((n,), 1, **I32), torch.arange(at, at + n, **I32)
            qkv = torch.zeros(n, -(-rows.shape[1] // 8) * 8, dtype=dtype, device="cuda")
            qkv[:, : rows.shape[1]].copy_(dev(rows[at : at + n]))
            mixed = torch.zeros(n, 3 + G * E, dtype=dtype, device="cuda")  # (not from column 0)
            mixed[:, 3:].copy_(dev(first[at : at + n]))
            att.mix_values(mixed[:, 3:], lam)
            o = torch.zeros(n, D.pad64(H * E), dtype=dtype, device="cuda")
            if n == 1:
                att.rows(qkv, o, slot, pos, 1, at + 1, append=True)
            else:
                att.append(qkv, slot, pos, n)
                if dtype == F32:
                    att.rows(qkv, o, slot, pos, n, at + n, append=False)
                else:
                    bs = att.prompt_block(spec)
                    blocks = torch.tensor([(b, 1, at + b, min(bs, n - b)) for b in range(0, n, bs)], **I32)
                    att.prompt(qkv, o, blocks, blocks.shape[0])
            got.append(host(o[:, : H * E]).reshape(n, H, E))
            cache.advance_host(n, [1])
            at += n
        close(np.concatenate(got), want, 2.5e-2 if dtype == BF else 1e-4, f"{shape} {cuts[:3]}")


def test_rotation_far_from_the_start(device):
    """Angles keep their accuracy at positions past 10^5 (keys are written at such a position and read back)."""
    G, De, base = 1, 64, 7e5
    spec = AttentionSpec(G, G, De, 8, 1.0, whole_norm=True, rot=RotarySpec(base, De))
    cache = PagedKVCache([(G, De, 8)], 1, 200000, "cuda", F32)
    gain, freq = torch.ones(De, device="cuda"), torch.tensor(spec.rot.turns(), dtype=torch.float64, device="cuda")
    att = D.PagedAttention(spec, None, 0, cache, 0.0, gain, gain, freq)
    x, p0, n = rand((5, 2 * De + 8), 1), 131071, 5
    cache.reserve([0], p0 + n)
    att.append(dev(x), torch.zeros(n, **I32), torch.arange(p0, p0 + n, **I32), n)
    k = O.rms_norm(x[:, De : 2 * De].astype(np.float64), 1.0, 0.0)
    z = (k[:, 0::2] + 1j * k[:, 1::2]) * np.exp(1j * np.arange(p0, p0 + n)[:, None] * base ** (-np.arange(De // 2) / (De // 2)))
    want = np.stack([z.real, z.imag], -1).reshape(n, De)
    assert np.abs(host(cache.read_nhd(0, 0, p0, n)[0])[:, 0] - want).max() < 1e-5


LATENT_SHAPES = [dict(), dict(heads=1, dim=40, rot_dim=4, vdim=72, kv_rank=130), dict(heads=18, dim=8, rot_dim=8, vdim=8, kv_rank=32),
                 dict(heads=5, dim=128, rot_dim=64, vdim=100, kv_rank=256), dict(heads=16, dim=96, rot_dim=32, vdim=140, kv_rank=512),
                 dict(heads=17, dim=64, rot_dim=128, vdim=20, kv_rank=480), dict(heads=2, dim=30, rot_dim=6, vdim=9, kv_rank=90)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", LATENT_SHAPES)
def test_latent_attention(device, dtype, shape):
    """Absorbed rows (with and without the append inside), expanded portions; a sequence beside another in the
    same launch.  Planted queries see one far key each, at page and tile borders and the first position."""
    cfg = U.config([U.latent(**shape)])
    w, m = U.weights(cfg, 3), cfg["layers"][0]["mixer"]
    model = build_model(config_from_dict(cfg), torch_weights(w, "cuda"), dtype=dtype)
    part = model.layers[0].parts[0]
    H, De, R, E, C, T, eps = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], 200, cfg["norm"]["eps"]
    say("latent", dtype, shape)
    w64 = {k: v.astype(np.float64) for k, v in w.items()}
    uk, uv = w64["l0.mix.uk"].reshape(H, De, C), w64["l0.mix.uv"].reshape(H, E, C)
    seqs, want = {}, {}
    for s, n in ((0, T), (2, 90)):
        kv, q = rand((n, C + R), 10 + s), rand((n, H, De + R), 20 + s)
        c = O.rms_norm(kv[:, :C].astype(np.float64), w64["l0.mix.dkv.norm"], eps)
        kr = O.rotate(kv[:, None, C:].astype(np.float64), m["rot"]["base"], R)
        kn = np.einsum("tc,hdc->thd", c, uk)
        far = {i: j for i, j in {60: 0, 64: 63, 89: 31, 90: 63, 91: 64, 130: 32, 150: 127, 170: 128, 199: 1}.items() if i < n}
        for i, j in far.items():
            q[i, :, :De] = bf16_round((2.5 * kn[j]).astype(np.float32))
        key = np.concatenate([kn, np.repeat(kr, H, 1)], -1)
        qt = np.concatenate([q[..., :De].astype(np.float64), O.rotate(q[..., De:].astype(np.float64), m["rot"]["base"], R)], -1)
        want[s] = O.attend(qt, key, np.einsum("tc,hec->the", c, uv), m["scale"])
        seqs[s] = (q, kv)
    schedules = ([[(0, T)], [(2, 90)]], [[(0, 3), (2, 33)], [(0, 2), (2, 1)], [(0, 64)], [(0, 1), (2, 40)], [(0, 60), (2, 2)], [(0, 2)], [(2, 500), (0, 500)]],
                 [[(0, 58)], [(2, 20)]] + [[(0, 1), (2, 1)]] * T)
    for sched in schedules:
        cache = model.make_cache(3, 512)
        op, at, got = model._mixers(cache)[0][0], {}, {}
        cache.reserve([1], 70)
        for step in sched:
            counts, qs, kvs = [], [], []
            for s, n in step:
                a = at.get(s, 0)
                n = min(n, len(seqs[s][1]) - a)
                if n > 0:
                    counts.append((s, n))
                    q = np.zeros((n, part.q_cols), np.float32)
                    q[:, : part.rot_col].reshape(n, H, -1)[..., :De] = seqs[s][0][a : a + n, :, :De]
                    q[:, part.rot_col :].reshape(n, H, -1)[..., :R] = seqs[s][0][a : a + n, :, De:]
                    qs.append(q)
                    kvs.append(seqs[s][1][a : a + n])
            if not counts:
                continue
            cache.reserve_each(counts)
            n = sum(c for _, c in counts)
            b, bf = model._batch(cache, counts, []), model._buffers(1, max(n, 2))
            q = torch.zeros(n, D.pad64(part.q_cols), dtype=dtype, device="cuda")
            q[:, : part.q_cols].copy_(dev(np.concatenate(qs)))
            kv = torch.zeros(n, C + R + 3, device="cuda")  # (not from column 0)
            kv[:, 3:] = dev(np.concatenate(kvs))
            out = torch.zeros(n, D.pad64(H * E), dtype=dtype, device="cuda")
            ql, ol = (torch.zeros(n, H * D.pad64(C), dtype=dtype, device="cuda") for _ in range(2))
            if b.decode:
                op.rows(q, kv[:, 3:], ql, ol, out, b.slot, b.pos, n, b.keys, append=True)
            else:
                op.prepare(q, kv[:, 3:], b.slot, b.pos, n)
                if b.latent.n_blocks:
                    op.prompt(q, kv[:, 3:], out, b.slot, b.pos, *b.latent.lists)
                if b.latent.n_rows:
                    op.rows(q, kv[:, 3:], ql, ol, out, b.slot, b.pos, b.latent.n_rows, b.keys, append=False, lst=b.latent.rows)
            o, k = host(out[:, : H * E]).reshape(n, H, E), 0
            for s, c in counts:
                got.setdefault(s, []).append(o[k : k + c])
                at[s] = at.get(s, 0) + c
                k += c
                cache.advance_host(c, [s])
            cache.sync_pos()
        for s in got:
            err = rel_rms(np.concatenate(got[s]).reshape(len(want[s]), -1), want[s].reshape(len(want[s]), -1))
            assert err.max() < (3e-2 if dtype == BF else 5e-5), f"{sched[0]} sequence {s}: {err.max():.1e} at {int(err.argmax())}"


@pytest.mark.parametrize("dtype", DTYPES)
def test_product_per_head_over_listed_rows(device, dtype):
    n, R, H, N, K = 37, 50, 3, 70, 24
    x, w = rand((R, H, K), 1), rand((H, N, K), 2)
    rows = rng(3).permutation(R)[:n].astype(np.int32)
    xt = torch.zeros(R, H, 64, dtype=dtype, device="cuda")
    xt[..., :K].copy_(dev(x))
    out = torch.zeros(R, H * 72, dtype=dtype, device="cuda")
    D.head_linear(xt.view(R, -1), 64, mat(w, dtype), out, 72, n, K, dev(rows, torch.int32))
    want = np.zeros((R, H, 72))
    want[rows, :, :N] = np.einsum("rhk,hnk->rhn", x.astype(np.float64), w)[rows]
    close(host(out).reshape(R, H, 72), want, TOL[dtype], "rows")


# ------------------------------------------------------------------ whole models


@pytest.fixture(scope="module")
def built():
    """The mixed configuration: config, tokens; by dtype float64 weights, model, oracle logits."""
    if not torch.cuda.is_available():
        pytest.skip("no GPU")
    cfg = U.mixed_config()
    w = {t: U.weights(cfg, 11, choosy=t == F32) for t in DTYPES}
    models = {t: build_model(config_from_dict(cfg), torch_weights(w[t], "cuda"), dtype=t) for t in DTYPES}
    toks = {name: rng(s).integers(0, cfg["vocab"], n).tolist() for s, (name, n) in
            enumerate({"a": 300, "b": 141, "c": 64, "d": 23, "e": 1}.items())}
    w64 = {t: O.to_float64(x) for t, x in w.items()}
    both = {t: {k: U.forward_and_gaps(cfg, w64[t], x) for k, x in toks.items()} for t in DTYPES}
    want, gaps = ({t: {k: v[i] for k, v in x.items()} for t, x in both.items()} for i in (0, 1))
    return types.SimpleNamespace(cfg=cfg, w=w64, models=models, toks=toks, want=want, gaps=gaps)


LIMIT = {BF: 1e-1, F32: 1e-4}  # of nearly all positions (bf16: a router's close choice may turn); a typical one: 2e-2


def check_rows(built, dtype, name, places, logits, what):
    err = rel_rms(logits, built.want[dtype][name][places])
    say(what, f"worst {err.max():.1e}, median {np.median(err):.1e}")
    assert np.quantile(err, 0.95) < LIMIT[dtype], f"{what}: {np.quantile(err, 0.95):.2e}"
    err = np.where(built.gaps[dtype][name][places] < (0.05 if dtype == BF else 0), 0, err)
    assert err.max() < LIMIT[dtype] * (5 if dtype == BF else 1), f"{what}: {err.max():.2e} at {places[int(err.argmax())]}"
    assert np.median(err) < LIMIT[dtype] / 2, f"{what}: median {np.median(err):.2e}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("portion", [300, 1, 2, 3, 17, 31, 32, 64, 65, 128])
def test_model_in_portions(built, dtype, portion):
    for name in built.toks if portion in (300, 1) else ("a", "c"):
        got = play(built.models[dtype], built.toks, [[(name, portion)]] * 300, max_tokens=320)[name]
        check_rows(built, dtype, name, np.arange(len(got)), got, f"portions of {portion}, {name}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("portion", [64, 1])
def test_model_layers(built, dtype, portion):
    m, outs, want = built.models[dtype], [], []
    O.forward(built.cfg, built.w[dtype], built.toks["c"], want)
    m.layer_hook = lambda i, h: outs.append(host(h).copy())
    try:
        play(m, built.toks, [[("c", portion)]] * 64)
    finally:
        m.layer_hook = None
    n = len(want)
    for i, w in enumerate(want):
        err = rel_rms(np.concatenate(outs[i::n]), w)
        assert np.median(err) < (3e-2 if dtype == BF else 3e-5), f"layer {i}: {np.median(err):.2e}"
        err = np.where(built.gaps[dtype]["c"] < (0.05 if dtype == BF else 0), 0, err)
        assert err.max() < (3e-1 if dtype == BF else 3e-5), f"layer {i}: {err.max():.2e}"


@pytest.mark.parametrize("dtype", DTYPES)
def test_model_mixed_batches_reuse_rows_and_pages(built, dtype):
    got = play(built.models[dtype], built.toks, SCHEDULE, max_tokens=640)
    for name, lg in got.items():
        check_rows(built, dtype, name.split("#")[0], np.arange(len(lg)), lg, f"mixed, {name}")


def test_rows_move_and_are_cut_back(built):
    m, t = built.models[F32], built.toks
    c = m.make_cache(3, 320)
    m.step(c, [(0, t["a"][:77], []), (1, t["b"][:50], [])])
    c.release(0)
    assert rel_rms(host(m.step(c, [(0, t["c"], [63])])), built.want[F32]["c"][63:]).max() < 1e-4
    c.copy_row(1, 2)
    assert rel_rms(host(m.step(c, [(2, t["b"][50:60], [9])])), built.want[F32]["b"][59:60]).max() < 1e-4
    c.swap_rows(0, 2)
    lg = host(m.step(c, [(1, t["d"][:1], [0]), (0, t["b"][60:61], [0])]))
    assert rel_rms(lg, np.stack([built.want[F32]["d"][0], built.want[F32]["b"][60]])).max() < 1e-4
    c.trim(30, rows=[0])
    assert rel_rms(host(m.step(c, [(0, t["b"][31:90], [58])])), built.want[F32]["b"][89:90]).max() < 1e-4


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("B", [1, 3, 4, 16, 20])
def test_model_graph_decode_matches_steps(built, dtype, B):
    """The captured single-token step over B rows, several replays with eager work between them."""
    m = built.models[dtype]
    cache = m.make_cache(B + 1, 320)
    seqs = [built.toks[n][o:] for o in range(8) for n in ("a", "b", "c")][:B]
    n0, n1 = 30, 46
    m.step(cache, [(r, s[: n0 - r % 7], []) for r, s in enumerate(seqs)])
    pos = [n0 - r % 7 for r in range(B)]
    wants, errs = [O.forward(built.cfg, built.w[dtype], s[:n1]) for s in seqs], []
    for k in range(n1 - n0):
        bf = m._buffers(B, 1)
        bf.tokens.copy_(torch.tensor([s[p] for s, p in zip(seqs, pos)], dtype=torch.int32))
        bf = m.decode_step(cache, B)
        errs.append(rel_rms(host(bf.logits), np.stack([w[p] for w, p in zip(wants, pos)])))
        pos = [p + 1 for p in pos]
        torch.randn(1000, device="cuda").sum().item()
    assert np.quantile(errs, 0.9 if dtype == BF else 1) < LIMIT[dtype] and np.median(errs) < LIMIT[dtype] / 2


def test_model_long_decode(built):
    m, toks = built.models[F32], rng(77).integers(0, built.cfg["vocab"], 560).tolist()
    want = O.forward(built.cfg, built.w[F32], toks)
    cache = m.make_cache(1, 600)
    m.step(cache, [(0, toks[:150], [])])
    bf = m._buffers(1, 1)
    for i in range(150, 560):
        bf.tokens[0] = toks[i]
        err = rel_rms(host(m.decode_step(cache, 1).logits), want[i : i + 1]).max()
        assert err < 1e-4, f"position {i}: {err:.2e}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layers", [
    [U.latent(), U.latent(heads=2, dim=140, rot_dim=120, vdim=20, mlp=None)],
    [U.attention(v_mix=False, mlp="dense"), U.attention(v_mix=True, window=500), U.attention(mlp=None, dim=48, rot=4)],
    [U.latent(heads=20, dim=16, rot_dim=16, vdim=32, q_rank=64, kv_rank=256, mlp="moe", experts=40, top=8, shared=None),
     U.attention(heads=2, kv_heads=1, dim=256, vdim=256, rot=256, window=100, mlp="dense", ff=300)]])
def test_other_orders_and_sizes(device, dtype, layers):
    """... among them key sizes that are too large to expand."""
    cfg = U.config(layers, width=130, vocab=97, eps=3e-3, alpha=1.0, embed=1.0, logit=1.0, side=1)
    w = U.weights(cfg, 5, choosy=dtype == F32)
    m = build_model(config_from_dict(cfg), torch_weights(w, "cuda"), dtype=dtype)
    toks = {"a": rng(1).integers(0, 97, 140).tolist(), "b": rng(2).integers(0, 97, 9).tolist()}
    want = {k: O.forward(cfg, w, t) for k, t in toks.items()}
    for sched in ([[("a", 140)]], [[("a", 70), ("b", 1)], [("b", 2), ("a", 3)]] + [[("a", 1), ("b", 1)]] * 90):
        for k, lg in play(m, toks, sched, max_tokens=256).items():
            err = rel_rms(lg, want[k])
            assert np.quantile(err, 0.95 if dtype == BF else 1) < LIMIT[dtype] and np.median(err) < LIMIT[dtype] / 2


def test_shards(built):
    """Every layer reads the tokens: a shard starts at layer 0, and layers that mix values hold the first."""
    w = torch_weights({k: np.asarray(v, np.float32) for k, v in built.w[F32].items()}, "cuda")
    c = config_from_dict(built.cfg)
    x = build_model(c, w, 0, 3, dtype=F32)
    want = []
    O.forward(built.cfg, built.w[F32], built.toks["c"], want)
    got = x(torch.tensor([built.toks["c"]]), x.make_cache(1, 100))
    assert rel_rms(host(got)[0], want[2]).max() < 1e-4
    with pytest.raises(ValueError, match="start at layer 0"):
        build_model(c, w, 3, 7, dtype=F32)


# ------------------------------------------------------------------ generation


def greedy_agrees(built, prompt, got, dtype):
    S.greedy_agrees(lambda toks: O.forward(built.cfg, built.w[dtype], toks), prompt, got, dtype)


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
    assert len(c._free) == c.n_pages
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
def test_prefix_cache(built, kind):
    m, p, d = built.models[F32], built.toks["a"], built.toks["d"]
    kv = KVPrefixCache(None, "cuda:0")
    eng = engine(m, kv_prefix_cache=kv) if kind == "batch" else SequentialGenerator(
        model=m, tokenizer=None, model_id="m", max_seq=512, kv_prefix_cache=kv)
    for q in (p, p, p + d, p[:100] + d):
        got = drain(eng, [task(0, q, 12, use_prefix_cache=True)])["t0"]
        greedy_agrees(built, q, got, F32)
    eng.close()


def test_latents_do_not_travel(built):
    import io
    m = built.models[BF]
    c = m.make_cache(1, 64)
    m.step(c, [(0, [1, 2, 3], [])])
    with pytest.raises(ValueError):
        W.write_cache_to_wire(io.BytesIO(), c, row=0)


@pytest.mark.parametrize("dtype", DTYPES)
def test_generate_greedy(built, dtype):
    p = built.toks["c"]
    toks = [r.token for r in generate(built.models[dtype], None, TextGenerationTaskParams(
        model="m", max_output_tokens=60, temperature=0.0), p)]
    assert len(toks) == 60
    greedy_agrees(built, p, toks, dtype)


def test_builder_serves_a_checkpoint(built, tmp_path):
    write_checkpoint(tmp_path, built.cfg, {k: np.asarray(v, np.float32) for k, v in built.w[BF].items()})
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
    write_checkpoint(tmp_path / "m", built.cfg, {k: np.asarray(v, np.float32) for k, v in built.w[dtype].items()})
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
    want = np.stack([built.want[dtype]["b"][99], built.want[dtype]["b"][3], built.want[dtype]["d"][1], built.want[dtype]["d"][22],
                     built.want[dtype]["b"][102], built.want[dtype]["b"][101], built.want[dtype]["d"][22]])
    assert rel_rms(got, want).max() < LIMIT[dtype] * (5 if dtype == BF else 1)
