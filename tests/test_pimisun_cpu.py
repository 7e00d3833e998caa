"""The Pimisun design without a GPU: its oracle against independent restatements, configuration and
registry, which tensors a shard loads, a pool layer without values, and argument checks."""

import copy
import math

import numpy as np
import pytest
import torch

from exo_amd import native
from exo_amd.loader import load_shard_weights
from exo_amd.paged_cache import PAGE, PagedKVCache
from exo_amd.registry import config_from_dict, load_config
from exo_amd.stack_config import (
    AttentionSpec, DenseSpec, GluSpec, LatentSpec, MoeSpec, RotarySpec, RouterSpec, StackConfig, pimisun_dict,
)
from oracle import pimisun as O
from tests import pimisun_util as U
from tests.gekazen_util import write_checkpoint
from tests.util import rng

# ------------------------------------------------------------------ oracle


def test_oracle_rotation_is_a_complex_product():
    x = rng(0).standard_normal((9, 3, 10))
    z = x[..., 0:6:2] + 1j * x[..., 1:6:2]
    a = np.arange(9)[:, None, None] * 100.0 ** (-np.arange(3) / 3.0)
    want = z * np.exp(1j * a)
    got = O.rotate(x, 100.0, 6)
    assert np.allclose(got[..., 0:6:2], want.real) and np.allclose(got[..., 1:6:2], want.imag)
    assert np.array_equal(got[..., 6:], x[..., 6:])


def test_oracle_attention_matches_torch():
    r, T, H, G, D, E = rng(2), 17, 6, 2, 8, 5
    q, k, v = (r.standard_normal((T, n, d)) for n, d in ((H, D), (G, D), (G, E)))
    t = lambda a: torch.from_numpy(a).permute(1, 0, 2)  # noqa: E731
    i = np.arange(T)
    mask = (i[:, None] >= i) & (i[:, None] - i < 4)
    want = torch.nn.functional.scaled_dot_product_attention(
        t(q), t(k).repeat_interleave(3, 0), t(v).repeat_interleave(3, 0), attn_mask=torch.from_numpy(mask), scale=0.4)
    assert np.allclose(O.attend(q, k, v, 0.4, 4), want.permute(1, 0, 2).numpy())
    assert np.allclose(O.attend(q, k, v, 0.4, 4, 1e6), want.permute(1, 0, 2).numpy(), atol=1e-6)


def test_oracle_latent_attention_absorbed():
    """Scores against the latents themselves, with the queries through the key matrices."""
    cfg = U.config([U.latent()])
    m, w = cfg["layers"][0]["mixer"], {k: v.astype(np.float64) for k, v in U.weights(cfg, 3).items()}
    p, T, H, D, C, E = "l0.mix.", 19, 3, 24, 44, 20
    h = rng(1).standard_normal((T, 72))
    want = O.latent_attention(h, w, p, m, 1e-4)
    q = (O.rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], 1e-4) @ w[p + "uq"].T).reshape(T, H, 36)
    z = h @ w[p + "dkv"].T
    c = O.rms_norm(z[:, :C], w[p + "dkv.norm"], 1e-4)
    ql = np.einsum("thd,hdc->thc", q[..., :D], w[p + "uk"].reshape(H, D, C))
    key = np.concatenate([c[:, None], O.rotate(z[:, None, C:], 1e4, 12)], -1)
    o = O.attend(np.concatenate([ql, O.rotate(q[..., D:], 1e4, 12)], -1), key, c[:, None], m["scale"])
    o = np.einsum("thc,hec->the", o, w[p + "uv"].reshape(H, E, C)).reshape(T, -1) @ w[p + "o"].T
    assert np.allclose(o, want)


def test_oracle_small_pieces_by_hand():
    assert np.allclose(O.layer_norm(np.array([[1.0, 3.0]]), np.array([2.0, 5.0]), 3.0), [[-1.0, 2.5]])
    assert np.allclose(O.relu_squared(np.array([-2.0, 3.0])), [0, 9])
    z = torch.linspace(-4, 4, 17, dtype=torch.float64)
    assert np.allclose(O.gelu_tanh(z.numpy()), torch.nn.functional.gelu(z, approximate="tanh").numpy())
    ids, wt = O.route(np.log([0.1, 0.5, 0.3, 0.1]), 2)
    assert list(ids) == [1, 2] and np.allclose(wt, [0.625, 0.375])
    q = np.full((1, 1, 1), 2.0)
    assert np.allclose(O.attend(q, q, q, 1.0, None, 3.0), q)  # one key: whatever its score


def test_oracle_is_causal_and_every_tensor_matters():
    cfg = U.mixed_config()
    w = U.weights(cfg, 1)
    toks = rng(1).integers(0, cfg["vocab"], 40).tolist()
    full = O.forward(cfg, w, toks)
    assert np.allclose(O.forward(cfg, w, toks[:23]), full[:23], atol=1e-9)
    skip = {"embed", "l0.mix.vmix", "l2.mix.q", "l2.mix.k", "l2.mix.q.norm", "l2.mix.k.norm"}  # (first values; a window of one)
    for name in w:
        if name in skip:
            continue
        other = dict(w, **{name: w[name] + (0.5 * rng(2).standard_normal(w[name].shape)).astype(np.float32)})
        assert np.abs(O.forward(cfg, other, toks) - full).max() > 1e-5, name
    other = dict(w, **{"l0.mix.vmix": w["l0.mix.vmix"] + 1})
    assert np.array_equal(O.forward(cfg, other, toks), full)


# ------------------------------------------------------------------ configuration


def test_config_reads_every_size_and_constant():
    d = U.mixed_config()
    c = config_from_dict(d)
    assert isinstance(c, StackConfig) and c.to_dict() == d
    assert (c.vocab_size, c.hidden_size, c.num_hidden_layers, c.side_dim, c.tied) == (331, 100, 7, 9, True)
    assert (c.embed_scale, c.logit_scale) == (0.6, 0.4)
    n = c.norm
    assert (n.eps, n.of_sum, n.keep, n.center, n.pre, n.offset) == (1e-4, True, 1.7, True, False, 0.0)
    assert c.layers[1].mixer == LatentSpec(3, 24, 12, 20, 36, 44, 2 / 6.0, RotarySpec(1e4, 12))
    assert c.layers[4].mixer == AttentionSpec(8, 2, 68, 24, 2 / np.sqrt(68), window=70, whole_norm=True, rot=RotarySpec(3e3, 2),
                                              softcap=12.0, v_mix_from=0)
    assert [getattr(L.mixer, "v_mix_from", None) for L in c.layers] == [None, None, None, None, 0, None, 0]
    assert c.layers[4].mlp is None and c.layers[5].mlp == DenseSpec(130, "relu2")
    e = lambda ff: GluSpec(ff, math.inf, 1.0, 0.0)  # noqa: E731
    assert c.layers[3].mlp == MoeSpec(RouterSpec(5, 0, 5, 1.0, bias=True, correction=False, renorm=True), e(33), e(8), shared_gate=False)
    assert c.layers[2].mlp.shared is None
    assert c.layers[1].mixer.pooled == (1, 64 + 12, 0) and c.layers[3].mixer.pooled == (1, 160 + 4, 0)
    assert np.allclose(RotarySpec(100.0, 4).turns(), [1 / (2 * np.pi), 0.1 / (2 * np.pi)])


@pytest.mark.parametrize("change, text", [
    (lambda d: d["layers"][0]["mixer"].update(heads=5), "query heads"),
    (lambda d: d["layers"][0]["mixer"]["mask"].update(size=0), "window"),
    (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=34), "rotated"),
    (lambda d: d["layers"][0]["mixer"].update(softcap=-1), "softcap"),
    (lambda d: d["layers"][4]["mixer"].update(vdim=20), "do not fit"),
    (lambda d: d["layers"][1]["mixer"].update(rot_dim=5), "latent"),
    (lambda d: d["layers"][0]["mlp"]["router"].update(top=6), "top 6"),
    (lambda d: d["layers"][0].update(type="gla"), "mixer type"),
    (lambda d: d["layers"][0]["mlp"].update(kind="sparse"), "feed-forward kind"),
])
def test_config_errors(change, text):
    d = copy.deepcopy(U.mixed_config())
    change(d)
    with pytest.raises(ValueError, match=text):
        config_from_dict(d)


def test_benchmark_config():
    d = pimisun_dict(64, 100, "lal", heads=4, kv_heads=2, dim=16, rot=8, window=32, lat_heads=4, lat_dim=16, lat_rot=8, lat_vdim=16,
                     q_rank=32, kv_rank=32, ff=96, experts=8, top=2, expert_ff=24, shared_ff=24, side=8)
    c = config_from_dict(d)
    assert [type(L.mixer) for L in c.layers] == [LatentSpec, AttentionSpec, LatentSpec]
    assert isinstance(c.layers[0].mlp, DenseSpec) and isinstance(c.layers[1].mlp, MoeSpec)


def test_loader_takes_the_shard_of_a_layer_range(tmp_path):
    cfg = U.mixed_config()
    w = U.weights(cfg, 2)
    write_checkpoint(tmp_path, cfg, w)
    c = load_config(tmp_path)

    def names(lo, hi):
        it = load_shard_weights(tmp_path, c, lo, hi, "cpu")
        while True:
            try:
                next(it)
            except StopIteration as stop:
                return set(stop.value)

    own = lambda lo, hi: {k for k in w if k[0] == "l" and lo <= int(k[1 : k.index(".")]) < hi}  # noqa: E731
    assert names(0, 7) == set(w)
    assert names(0, 3) == own(0, 3) | {"embed", "side.embed"}
    assert names(3, 7) == own(3, 7) | {"embed", "side.embed", "final.norm"}  # (the head is the embedding table)


def test_pool_layers_without_values():
    c = PagedKVCache([(2, 24, 20), (1, 76, 0)], 2, 200, "cpu", torch.float32, pool_tokens=4 * PAGE)
    assert c.k[1].shape == (4, 1, PAGE, 96) and c.v[1].numel() == 0
    c.reserve([0], 70)
    k = torch.randn(70, 1, 76)
    c.write_nhd(1, 0, 0, k, torch.empty(70, 1, 0))
    c.advance_host(70, [0])
    saved = c.snapshot(0)
    assert torch.equal(saved[1][0], k) and saved[1][1].shape == (70, 1, 0)
    c.reset()
    c.reserve([1], 65)
    c.restore(0, saved, 66)
    assert torch.equal(c.read_nhd(1, 0, 3, 63)[0], k[3:66])


def test_new_entry_points_check_their_arguments():
    lib = native.load()
    ok = dict(q=16, q_latent=16, kv=16, gain=16, freq=16, pool=16, table=16, slot=16, pos=16, out=16, n=1, heads=2, rank=40, rot=8,
              rot_col=128, ldq=144, ldql=128, ldkv=48, ldk=96, ldo=128, max_pages=1, nsplit=1)
    for change in (dict(rank=600), dict(rot=7), dict(rot=200), dict(ldk=64), dict(ldkv=47), dict(ldq=140), dict(dtype=3), dict(pool=None),
                   dict(nsplit=65), dict(nsplit=2), dict(ldql=64), dict(ldo=64)):
        assert lib.exo_latent_rows(native.LatentAttn(**{**ok, **change}), 0, None) == -1, change
    assert lib.exo_latent_rows(native.LatentAttn(**ok, prepared=1), 1, None) == -1
    assert lib.exo_latent_prepare(native.LatentAttn(**ok, prepared=1), None) == -1
    head = dict(x=16, w=16, y=16, n=1, heads=2, N=40, K=24, ldx=128, x_head=64, ldw=64, ldy=80, y_head=40, nsplit=1)
    for change in (dict(ldx=64), dict(ldw=48), dict(ldy=79), dict(y_head=39), dict(x_head=20), dict(w=None), dict(parts=16)):
        assert lib.exo_head_linear(native.HeadLinear(**{**head, **change}), None) == -1, change
    pr = dict(q=16, k=16, k_rot=16, v=16, list=16, out=16, n=1, heads=2, vdim=20, d8=24, r8=16, ldq=160, q_head=64, rot_col=128, ldk=48,
              ldv=64, ldo=64)
    for change in (dict(d8=20), dict(d8=250), dict(r8=0), dict(vdim=300), dict(ldk=40), dict(ldv=63), dict(rot_col=100), dict(ldo=39)):
        assert lib.exo_latent_prompt(native.LatentPrompt(**{**pr, **change}), None) == -1, change
    att = dict(qkv=16, k_pool=16, v_pool=16, table=16, slot=16, pos=16, out=16, n=1, heads=2, kv_heads=2, dim=64, vdim=64, ldk=64,
               ldv=64, ldq=999, ldo=1000, max_pages=1, list=16)
    for change in (dict(rot=8), dict(rot=66, freq=16), dict(rot=8, freq=16, unit_qk=1), dict(whole_norm=1), dict(softcap=-1.0),
                   dict(v_mix=16, ldmix=100)):
        assert lib.exo_paged_prepare(native.PagedAttn(**{**att, **change}), None) == -1, change
    assert lib.exo_paged_append(native.PagedAttn(**att, rot=8, freq=16), None) == -1 and b"exo_paged_prepare" in lib.exo_last_error()
    assert lib.exo_paged_attn_prompt(native.PagedAttn(**att, rot=8, freq=16), None) == -1 and b"prepared" in lib.exo_last_error()
    lin = dict(x=16, w=16, y=16, M=1, N=8, n1=8, ldx=64, ldw=64, ldy=8)
    for change in (dict(act=3), dict(act=1, w_up=16), dict(mul=16, ldmul=7), dict(act=1, n1=4, y2=16, ldy2=4)):
        assert lib.exo_linear_rows(native.Linear(**{**lin, **change}), None, None) == -1, change
    q = dict(x=16, x_out=16, branch=16, gain=16, operand=16, H=64, ldb=64)
    assert lib.exo_post_norm_add(native.PostNorm(**q, center=1), 1, 64, 0, None) == -1
    assert lib.exo_post_norm_add(native.PostNorm(**q, sum=1, branch2=16, gain_a=16, gain_b=16), 1, 64, 0, None) == -1
