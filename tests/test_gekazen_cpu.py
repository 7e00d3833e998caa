"""The Gekazen design without a GPU: its oracle against independent restatements, configuration and
registry, which tensors a shard loads, and the paged pool's bookkeeping."""

import copy
import json

import numpy as np
import pytest
import torch

from exo_amd import native
from exo_amd.cache import cache_length
from exo_amd.config import ModelConfig
from exo_amd.engine import ShardBatchGenerator
from exo_amd.loader import load_shard_weights, wanted
from exo_amd.paged_cache import PAGE, PagedKVCache, PoolExhausted
from exo_amd.registry import config_from_dict, load_config
from exo_amd.stack_config import StackConfig, distance_slopes, gekazen_dict
from oracle import gekazen as O
from tests import gekazen_util as U
from tests.util import rng, tiny_config

# ------------------------------------------------------------------ oracle


def test_oracle_attention_matches_torch_sdpa():
    r, T, H, G, D = rng(0), 37, 6, 2, 16
    q, k, v = (r.standard_normal((T, n, D)) for n in (H, G, G))
    slopes = O.head_slopes(H)
    mask = O.visible(T, 11, 4)
    bias = -slopes[:, None, None] * (np.arange(T)[:, None] - np.arange(T)[None, :])
    t = lambda a: torch.from_numpy(a).permute(1, 0, 2)  # noqa: E731
    want = torch.nn.functional.scaled_dot_product_attention(
        t(q), t(k).repeat_interleave(H // G, 0), t(v).repeat_interleave(H // G, 0),
        attn_mask=torch.from_numpy(np.where(mask, bias, -np.inf)), scale=0.7)
    got = O.attend(q, k, v, 0.7, slopes, mask)
    assert np.allclose(got, want.permute(1, 0, 2).numpy(), atol=1e-12)


def test_oracle_mask_rows_by_hand():
    m = O.visible(8, 3, 2)
    assert [list(np.flatnonzero(row)) for row in m] == [
        [0], [0, 1], [0, 1, 2], [0, 1, 2, 3], [0, 1, 2, 3, 4], [0, 1, 3, 4, 5], [0, 1, 4, 5, 6], [0, 1, 5, 6, 7]]
    assert O.visible(5, 1, 0).sum() == 5 and O.visible(5, None, 0).sum() == 15


def test_oracle_norm_unit_and_router_by_hand():
    x = np.array([[3.0, -4.0]])
    assert np.allclose(O.rms_unit(x, 0.0), x / np.sqrt(12.5))
    assert np.allclose(O.rms_norm_offset(x, np.array([0.0, 1.0]), 0.5), x / np.sqrt(13.0) * [1.0, 2.0])
    g, u = np.array([9.0, -1.0]), np.array([-9.0, 0.5])
    want = [2 / (1 + np.exp(-1.702 * 2)) * (1 - 2), -1 / (1 + np.exp(1.702)) * 1.5]
    assert np.allclose(O.clamped_glu(g, u, 2.0), want)
    ids, wt = O.route(np.log([0.5, 0.3, 0.2]), np.array([0.0, -0.25, 0.2]), 2, 3.0)
    assert list(ids) == [0, 2] and np.allclose(wt, [1.5, 0.6])  # chosen with, weighted without the correction


def test_oracle_shared_keys_and_causality():
    cfg = U.mixed_config()
    w = O.to_float64(U.weights(cfg, 1))
    toks = rng(1).integers(0, cfg["vocab"], 120).tolist()
    full = O.forward(cfg, w, toks)
    assert np.allclose(O.forward(cfg, w, toks[:50]), full[:50], atol=1e-9)
    other = copy.deepcopy(cfg)  # the layer that takes layer 1's keys has a mask of its own: one
    other["layers"][4]["mixer"]["mask"]["size"] += 1  # more key shows where key 66 left the window, not before
    d = np.abs(O.forward(other, w, toks) - full).max(-1)
    assert d[:99].max() < 1e-12 and d[99] > 1e-6


# ------------------------------------------------------------------ configuration


def test_config_reads_every_size_and_constant():
    d = U.mixed_config()
    c = config_from_dict(d)
    assert isinstance(c, StackConfig) and c.to_dict() == d
    assert (c.vocab_size, c.hidden_size, c.num_hidden_layers, c.eps) == (331, 100, 6, 1e-5)
    m = c.layers[4].mixer
    assert (m.kv_from, m.window, m.keep_first, m.dim, m.vdim) == (1, 33, 66, 40, 24)
    assert c.layers[3].mlp is None and c.layers[1].mlp.shared is None
    f = c.layers[2].mlp
    assert (f.router.experts, f.router.identity, f.router.top, f.router.scale) == (3, 5, 8, 0.6)
    assert (f.expert.limit, f.shared.limit, f.expert.ff, f.shared.ff) == (1.5, 0.9, 40, 56)
    assert distance_slopes(3) == pytest.approx(list(O.head_slopes(3)))


def test_config_of_a_full_causal_layer():
    d = U.config([U.layer()])
    del d["layers"][0]["mixer"]["mask"]
    m = config_from_dict(d).layers[0].mixer
    assert m.window is None and m.keep_first == 0


@pytest.mark.parametrize("change, text", [
    (lambda d: d["layers"][0]["mixer"].update(heads=5), "query heads"),
    (lambda d: d["layers"][4]["mixer"].update(kv_from=5), "kv_from"),
    (lambda d: d["layers"][5]["mixer"].update(kv_from=4), "kv_from"),
    (lambda d: d["layers"][4]["mixer"].update(dim=48), "head sizes"),
    (lambda d: d["layers"][1]["mlp"]["router"].update(top=6), "top"),
    (lambda d: d["layers"][1].update(type="recurrent"), "mixer type"),
    (lambda d: d["layers"][1]["mlp"].update(kind="dense"), "feed-forward kind"),
    (lambda d: d.update(architecture="Other"), "not supported"),
    (lambda d: d["layers"][0]["mixer"]["mask"].update(size=0), "window"),
])
def test_config_errors(change, text):
    d = U.mixed_config()
    change(d)
    with pytest.raises(ValueError, match=text):
        config_from_dict(d)


def test_registry_chooses_by_config(tmp_path):
    U.write_checkpoint(tmp_path / "a", U.mixed_config(), {"embed": np.zeros((1, 1), np.float32)})
    assert isinstance(load_config(tmp_path / "a"), StackConfig)
    (tmp_path / "b").mkdir()
    (tmp_path / "b" / "config.json").write_text(json.dumps(tiny_config("llama").to_dict()))
    assert isinstance(load_config(tmp_path / "b"), ModelConfig)
    assert config_from_dict(gekazen_dict(64, 100, 3, heads=4, kv_heads=2, dim=16, vdim=16, experts=4, identity=1,
                                         top=2, ff=32, shared_ff=32, kv_from={2: 1})).layers[2].mixer.kv_from == 1


def test_loader_takes_the_shard_of_a_layer_range(tmp_path):
    cfg_d = U.mixed_config()
    w = U.weights(cfg_d, 2)
    U.write_checkpoint(tmp_path, cfg_d, w)
    cfg = load_config(tmp_path)
    assert wanted("embed", cfg, 0, 2) and not wanted("embed", cfg, 1, 6) and wanted("head", cfg, 3, 6)
    assert wanted("l3.mix.q.b", cfg, 3, 4) and not wanted("l3.mix.q", cfg, 0, 3) and not wanted("final.norm", cfg, 0, 5)
    it = load_shard_weights(tmp_path, cfg, 1, 3, "cpu")
    seen = []
    try:
        while True:
            seen.append(next(it))
    except StopIteration as s:
        got = s.value
    assert seen == [(1, 2), (2, 2)]
    assert set(got) == {k for k in w if k.startswith(("l1.", "l2."))}
    assert np.array_equal(got["l1.mix.q"].float().numpy(), w["l1.mix.q"])


# ------------------------------------------------------------------ paged pool


def pool(rows=3, max_seq=400, tokens=None):
    return PagedKVCache([(2, 40, 24), (1, 64, 64)], rows, max_seq, "cpu", torch.float32, tokens)


def fill(c, row, n, seed):
    c.reserve([row], n)
    at = c.offsets[row]
    g = torch.Generator().manual_seed(seed)
    kv = []
    for i, (G, d, e) in enumerate(c.shapes):
        kv.append((torch.randn(n, G, d, generator=g), torch.randn(n, G, e, generator=g)))
        c.write_nhd(i, row, at, *kv[-1])
    c.advance_host(n, [row])
    c.sync_pos()
    return kv


def same(c, row, kv, start, n):
    return all(torch.equal(c.read_nhd(i, row, start, n)[j], kv[i][j][start : start + n]) for i in range(len(kv))
               for j in (0, 1))


def test_pool_counts_pages_not_rows():
    c = pool(tokens=5 * PAGE)
    fill(c, 0, 65, 0)
    fill(c, 1, 130, 1)
    assert c.free_tokens == 0 and len(c.pages[0]) == 2 and len(c.pages[1]) == 3
    with pytest.raises(PoolExhausted):
        c.reserve([2], 1)
    c.reserve([0], 63)  # fits the row's last page
    assert c.offsets == [65, 130, 0] and cache_length(c) == 130
    c.trim(65, rows=[1])  # 65 left: two pages
    assert c.free_tokens == PAGE
    c.release(0)
    assert c.free_tokens == 3 * PAGE and c.pos.tolist() == [0, 65, 0]
    with pytest.raises(ValueError, match="overflow"):
        c.reserve([1], 400)


def test_pool_reserve_is_all_or_nothing():
    c = pool(tokens=2 * PAGE)
    with pytest.raises(PoolExhausted):
        c.reserve_each([(0, PAGE), (1, PAGE + 1)])
    assert c.free_tokens == 2 * PAGE and not c.pages[0] and not c.pages[1]


def test_pool_pages_are_used_again_and_rows_move():
    c = pool(tokens=6 * PAGE)
    a, b = fill(c, 0, 100, 0), fill(c, 1, 190, 1)
    assert same(c, 0, a, 0, 100) and same(c, 1, b, 60, 130) and same(c, 1, b, 64, 64)
    first = list(c.pages[0])
    c.release(0)
    d = fill(c, 2, 70, 2)
    assert set(c.pages[2]) <= set(first) | set(range(6)) and same(c, 1, b, 0, 190)
    c.copy_row(2, 0)
    assert same(c, 0, d, 0, 70) and c.offsets == [70, 190, 0] and not c.pages[2]
    c.swap_rows(0, 1)
    assert same(c, 1, d, 0, 70) and same(c, 0, b, 0, 190) and c.pos.tolist() == [190, 70, 0]
    assert c.table[0, :3].tolist() == c.pages[0] and c.table[1, :2].tolist() == c.pages[1]


def test_pool_snapshot_and_restore():
    c = pool()
    a = fill(c, 1, 150, 3)
    snap = c.snapshot(1)
    c.release(1)
    fill(c, 0, 30, 4)
    c.restore(2, snap, 133)
    assert c.offsets == [30, 0, 133] and same(c, 2, a, 0, 133)


# ------------------------------------------------------------------ scheduler


class FakePaged:
    """A model with a mixed step whose 'logits' say which token comes next: last token + 1."""

    mixed_steps = True

    def __init__(self, vocab=50):
        self.cfg = type("C", (), {"vocab_size": vocab})()
        self.device, self.is_first, self.is_last = torch.device("cpu"), True, True
        self.steps: list = []

    def make_cache(self, rows, max_seq, pool_tokens=None):
        return PagedKVCache([(1, 32, 32)], rows, max_seq, "cpu", torch.float32, pool_tokens)


def test_can_admit_counts_requests_to_their_end(monkeypatch):
    import exo_amd.engine as E
    monkeypatch.setattr(E, "DeviceSampler", lambda *a: None)
    monkeypatch.setattr(torch, "zeros", lambda *a, pin_memory=None, _z=torch.zeros, **k: _z(*a, **k))
    g = ShardBatchGenerator(FakePaged(), None, 4, 1000, pool_tokens=10 * PAGE)
    assert g.max_seq == 10 * PAGE
    assert g.can_admit(500, 100) and g.can_admit(5000, None)  # clipped to the pool
    params = type("P", (), {"max_output_tokens": 100})()
    g.rows.append(type("Q", (), {"prompt_tokens": [0] * 200, "params": params})())
    assert g.can_admit(200, 100) and not g.can_admit(300, 100)


def test_new_entry_points_check_their_arguments():
    lib = native.load()
    lin = dict(x=16, w=16, y=16, M=1, N=8, n1=8, ldx=64, ldw=64, ldy=8)
    assert lib.exo_linear_rows(native.Linear(**dict(lin, w=None)), None, None) == -1
    assert lib.exo_linear_rows(native.Linear(**dict(lin, M=17)), None, None) == -1
    assert lib.exo_linear_rows(native.Linear(**dict(lin, n1=4)), None, None) == -1  # no second output
    assert lib.exo_linear_rows(native.Linear(**dict(lin, ldx=72, ldw=72)), None, None) == -1
    assert b"multiples of 64" in lib.exo_last_error()
    assert lib.exo_moe_route(16, 16, 16, 16, 1, 600, 600, 2, 1.0, 0, None) == -1
    a = native.PagedAttn(qkv=16, k_pool=16, v_pool=16, table=16, slot=16, pos=16, out=16, n=1, heads=3, kv_heads=2,
                         dim=64, vdim=64, ldk=64, ldv=64, ldq=999, ldo=999, max_pages=1)
    assert lib.exo_paged_attn_rows(a, 1, 0, None, 0, None) == -1
    a.heads, a.dim, a.ldk = 2, 300, 320
    assert lib.exo_paged_attn_rows(a, 1, 0, None, 0, None) == -1 and b"head sizes" in lib.exo_last_error()
    assert [lib.exo_paged_prompt_block(h, 2) for h in (2, 4, 6, 8)] == [128, 64, 32, 32]
