"""The Novosun design without a GPU: its oracle against independent restatements, configuration and
registry, which tensors a shard loads, the state pool beside the paged pool, and argument checks."""

import copy

import numpy as np
import pytest
import torch

from exo_amd import native
from exo_amd.loader import load_shard_weights
from exo_amd.paged_cache import PAGE, PagedKVCache
from exo_amd.prefix_cache import KVPrefixCache, restore_row, snapshot_row
from exo_amd.registry import config_from_dict, load_config
from exo_amd.stack_config import AttentionSpec, LinearAttentionSpec, ParallelSpec, StackConfig, novosun_dict
from oracle import novosun as O
from tests import novosun_util as U
from tests.gekazen_util import write_checkpoint
from tests.util import rng

# ------------------------------------------------------------------ oracle


def test_oracle_recurrence_is_decayed_attention():
    """o_t = sum over j <= t of (q_t . prod of the decays behind j . k_j) v_j, pair by pair."""
    r, T, D, E = rng(0), 21, 5, 3
    q, k, v, a = r.standard_normal((T, D)), r.standard_normal((T, D)), r.standard_normal((T, E)), r.uniform(0.2, 1, (T, D))
    want = np.zeros((T, E))
    for t in range(T):
        for j in range(t + 1):
            want[t] += (q[t] * a[j + 1 : t + 1].prod(0) * k[j]).sum() * v[j]
    got, S = O.recurrence(q, k, v, a)
    assert np.allclose(got, want)
    assert np.allclose(S, sum(np.outer(a[j + 1 :].prod(0) * k[j], v[j]) for j in range(T)))


def test_oracle_convolution_matches_torch():
    r = rng(1)
    x, w, b = r.standard_normal((13, 6)), r.standard_normal((6, 4)), r.standard_normal(6)
    t = torch.nn.functional.conv1d(torch.from_numpy(x.T)[None], torch.from_numpy(w)[:, None], torch.from_numpy(b), padding=3, groups=6)
    assert np.allclose(O.causal_conv(x, w, b), torch.nn.functional.silu(t)[0, :, :13].numpy().T)


def test_oracle_attention_matches_torch():
    r, T, H, G, D, E = rng(2), 17, 6, 2, 8, 5
    q, k, v = (r.standard_normal((T, n, d)) for n, d in ((H, D), (G, D), (G, E)))
    t = lambda a: torch.from_numpy(a).permute(1, 0, 2)  # noqa: E731
    want = torch.nn.functional.scaled_dot_product_attention(
        t(q), t(k).repeat_interleave(3, 0), t(v).repeat_interleave(3, 0), is_causal=True, scale=0.4)
    assert np.allclose(O.attend(q, k, v, 0.4), want.permute(1, 0, 2).numpy())


def test_oracle_small_pieces_by_hand():
    assert np.allclose(O.grouped_norm(np.array([[3.0, 4, 0, 2]]), np.array([1.0, 2, 3, 4]), 2, 0.0),
                       [[3 / np.sqrt(12.5), 8 / np.sqrt(12.5), 0, 8 / np.sqrt(2)]])
    w = {"a1": np.array([[2.0]]), "a2": np.array([[1.0], [-3.0]]), "a2.b": np.array([0.5, 0.0])}
    z = np.array([[2 * 1.5 + 0.5, -9.0]])
    assert np.allclose(O.channel_decay(np.array([[1.5]]), w, "", 4.0), (1 / (1 + np.exp(-z))) ** 0.25)
    assert np.allclose(O.softplus(np.array([-800.0, 0, 800])), [0, np.log(2), 800])
    assert np.allclose(O.clamped_glu(np.array([9.0, -1]), np.array([-9.0, 0.5]), 2.0),
                       [2 / (1 + np.exp(-3.404)) * -1, -1 / (1 + np.exp(1.702)) * 1.5])


def test_oracle_is_causal_and_every_tensor_matters():
    cfg = U.mixed_config()
    w = U.weights(cfg, 1)
    toks = rng(1).integers(0, cfg["vocab"], 40).tolist()
    full = O.forward(cfg, w, toks)
    assert np.allclose(O.forward(cfg, w, toks[:23]), full[:23], atol=1e-9)
    for name in w:
        if name in ("embed", "head"):
            continue
        other = dict(w, **{name: w[name] + rng(2).standard_normal(w[name].shape).astype(np.float32) * 0.5})
        assert np.abs(O.forward(cfg, other, toks) - full).max() > 1e-4, name


def test_planted_input_reaches_a_far_query():
    m = U.parallel(ssm_heads=3, ssm_vdim=5, state=7, groups=1, conv=3, norm_groups=3)
    w = U.weights(U.config([m]), 3)
    w["l0.mix.right.A_log"][:] = -7
    x, dt = rng(12).standard_normal((210, 29)), rng(13).standard_normal((210, 3))
    a = U.ssm_oracle(w, m["mixer"]["right"], x, dt)
    x[5, 15:], dt[5] = 3.0, 4.0
    b = U.ssm_oracle(w, m["mixer"]["right"], x, dt)
    assert np.abs(a[-1] - b[-1]).max() > 0.05 * np.abs(a[-1]).max() and np.abs(a[:5] - b[:5]).max() == 0


# ------------------------------------------------------------------ configuration


def test_config_reads_every_size_and_constant():
    d = U.mixed_config()
    c = config_from_dict(d)
    assert isinstance(c, StackConfig) and c.to_dict() == d
    assert (c.vocab_size, c.hidden_size, c.num_hidden_layers) == (331, 100, 6)
    assert (c.norm.eps, c.norm.pre, c.norm.offset, c.norm.mult) == (1e-4, True, 0.0, 0.7)
    assert c.norm.names(2) == ("norm2", "norm2b")
    assert c.layers[3].mixer == LinearAttentionSpec(1, 72, 136, 0.5) and c.layers[3].mlp is None
    m = c.layers[5].mixer
    assert isinstance(m, ParallelSpec)
    assert m.left == AttentionSpec(5, 1, 64, 7, 1.5 / 8, unit_qk=True, qk_gain=True, head_gate=True)
    assert (m.right.core, m.right.conv, m.right.norm_groups, m.right.channels) == ((5, 5, 16, 16), 9, 5, 240)
    assert (c.layers[4].mlp.ff, c.layers[4].mlp.limit, c.layers[4].mlp.alpha, c.layers[4].mlp.shift) == (130, 2.0, 1.702, 1.0)


@pytest.mark.parametrize("change, text", [
    (lambda d: d["layers"][1]["mixer"]["left"].update(heads=5), "query heads"),
    (lambda d: d["layers"][1]["mixer"]["right"].update(groups=4), "recurrent heads"),
    (lambda d: d["layers"][1]["mixer"]["right"].update(conv=0), "taps"),
    (lambda d: d["layers"][1]["mixer"]["right"].update(norm_groups=7), "norm groups"),
    (lambda d: d["layers"][0]["mixer"].update(tau=0), "tau"),
    (lambda d: d["layers"][0].update(type="attention"), "mixer type"),
    (lambda d: d["layers"][0]["mlp"].update(kind="moe"), "feed-forward kind"),
])
def test_config_errors(change, text):
    d = copy.deepcopy(U.mixed_config())
    change(d)
    with pytest.raises(ValueError, match=text):
        config_from_dict(d)


def test_benchmark_config():
    d = novosun_dict(64, 100, "gpg", heads=4, kv_heads=2, dim=16, vdim=32, ff=96, lin_heads=2, lin_dim=16, lin_vdim=32,
                     ssm_heads=8, ssm_vdim=16, ssm_state=24)
    c = config_from_dict(d)
    assert [type(L.mixer) for L in c.layers] == [LinearAttentionSpec, ParallelSpec, LinearAttentionSpec]
    c.layers[0].mixer.core  # (usable as it stands)


def test_loader_takes_the_shard_of_a_layer_range(tmp_path):
    cfg_d = U.mixed_config()
    w = U.weights(cfg_d, 2)
    write_checkpoint(tmp_path, cfg_d, w)
    it = load_shard_weights(tmp_path, load_config(tmp_path), 1, 3, "cpu")
    try:
        while True:
            next(it)
    except StopIteration as s:
        got = s.value
    assert set(got) == {k for k in w if k.startswith(("l1.", "l2."))}
    assert np.array_equal(got["l1.mix.right.A_log"].float().numpy(), w["l1.mix.right.A_log"])


def test_every_layer_of_the_design_loads():
    """Shapes the configuration does not expect fail by name."""
    from exo_amd.stack_layers import Layer
    c = config_from_dict(U.mixed_config())
    w = {k: torch.from_numpy(v).to(torch.bfloat16) for k, v in U.weights(U.mixed_config(), 0).items()}
    for i, spec in enumerate(c.layers):
        L = Layer(spec, w, i, c.hidden_size, c.norm, torch.float32, torch.device("cpu"))
        assert L.proj.shape[0] == L.n_main + L.n_tail and all(p.col % 8 == 0 for p in L.parts)
        assert (L.ff is None) == (spec.mlp is None) and L.pre1 is not None
        assert torch.equal(L.norm1, w[f"l{i}.norm1b"].float())
    bad = dict(w, **{"l1.mix.right.conv": torch.zeros(3, 4)})
    with pytest.raises(ValueError, match="l1.mix.right.conv"):
        Layer(c.layers[1], bad, 1, c.hidden_size, c.norm, torch.float32, torch.device("cpu"))


# ------------------------------------------------------------------ state pool


def pool(rows=3, max_seq=400, tokens=None, kv=((2, 8, 8),)):
    return PagedKVCache(list(kv), rows, max_seq, "cpu", torch.float32, tokens, states=[(2, 5, 20, 0, 0), (3, 4, 7, 4, 10)])


def fill(c, row, n, seed):
    """Tokens and states of the sequence in ``row``."""
    g = torch.Generator().manual_seed(seed)
    c.reserve([row], n)
    for i, (G, d, e) in enumerate(c.shapes):
        c.write_nhd(i, row, 0, torch.randn(n, G, d, generator=g), torch.randn(n, G, e, generator=g))
    c.advance_host(n, [row])
    c.sync_pos()
    s = [torch.randn(1, *t.shape[1:], generator=g) for t in c.states.tensors()]
    c.load_states([row], s)
    return s


def same(c, row, want):
    return all(torch.equal(a, b) for a, b in zip(c.save_states([row]), want))


def test_states_follow_their_rows():
    c = pool()
    a, b = fill(c, 0, 70, 0), fill(c, 1, 30, 1)
    assert len(c) == 3 and not c.trimmable and not c[0].is_trimmable()
    where = [t.data_ptr() for t in c.states.tensors()]
    before = [t.clone() for t in c.states.tensors()]
    c.swap_rows(0, 1)
    assert same(c, 1, a) and same(c, 0, b) and c.offsets == [30, 70, 0]
    c.copy_row(1, 2)
    assert same(c, 2, a) and same(c, 0, b) and sorted(c.states.slot) == [0, 1, 2]
    assert c.states.map.tolist() == c.states.slot
    assert where == [t.data_ptr() for t in c.states.tensors()]  # nothing was moved to get there
    assert all(torch.equal(x, y) for x, y in zip(before, c.states.tensors()))


def test_a_row_with_a_state_goes_back_to_nothing_only():
    c = pool()
    fill(c, 0, 70, 0)
    with pytest.raises(ValueError, match="cut back"):
        c.trim(2, rows=[0])
    assert c.offsets[0] == 70
    assert c.trim(70, rows=[0]) == 70 and c.offsets[0] == 0 and c.free_tokens == 3 * 7 * PAGE
    assert c.trim(5, rows=[1]) == 0


def test_snapshot_restores_states_at_their_position_only():
    c = pool()
    a = fill(c, 1, 70, 3)
    snap = snapshot_row(c, 1)
    fill(c, 0, 10, 4)
    c.release(1)
    restore_row(snap, c, 2, 70)
    assert same(c, 2, a) and c.offsets == [10, 0, 70]
    with pytest.raises(ValueError, match="recurrent state"):
        restore_row(snap, c, 1, 69)


@pytest.mark.parametrize("kv", [((2, 8, 8),), ()])
def test_prefix_cache_takes_only_prompts_that_go_on(kv):
    c = pool(kv=kv)
    p = list(range(100, 171))
    store = KVPrefixCache(None, "cpu")
    store.get_memory_used_percentage = lambda: 0.0
    a = fill(c, 0, 70, 3)
    store.add_kv_cache(p, c, 0)
    for prompt, hit in ((p, 70), (p + [1, 2], 70), (p[:70] + [5, 6, 7], 70), (p[:60] + [5] * 30, 0), (p[:70], 0), ([1, 2, 3], 0)):
        c.reset([1])
        _, rest, index, _ = store.get_kv_cache(c, prompt, row=1)
        assert len(prompt) - len(rest) == hit == c.offsets[1] and (index is not None) == (hit > 0), len(prompt)
        assert not hit or same(c, 1, a)


def test_new_entry_points_check_their_arguments():
    lib = native.load()
    ok = dict(heads=2, groups=2, dim=8, vdim=8, lds=16, state=16, map=16, y=16, ldy=16, per_channel=1, low=16, decay_w=16,
              decay_b=16, rank=4, ldlow=4)
    for change in (dict(heads=3), dict(dim=0), dict(lds=4), dict(dtype=3), dict(rank=0), dict(state=None), dict(taps=4), {}):
        assert lib.exo_recur_step(native.Recurrence(**{**ok, **change}), None) == -1
    assert b"rows" in lib.exo_last_error()  # (the last one lacks only its rows)
    head = dict(heads=4, groups=2, dim=8, vdim=8, lds=16, state=16, map=16, y=16, ldy=32, dt_raw=16, dt_bias=16, decay_rate=16,
                lddt=4, taps=4, channels=64, ldraw=64, raw=16, ring=16, conv_w=16, conv_b=16, k_channel=32, q_channel=48)
    for change in (dict(taps=17), dict(channels=60), dict(q_channel=50), dict(lddt=3)):
        assert lib.exo_recur_chunks(native.Recurrence(**{**head, **change}), None, 0, None) == -1
        assert b"exo_recur_chunks" in lib.exo_last_error()
    assert lib.exo_gated_norm_rows(native.GatedNorm(y=16, gate=16, gain=16, out=16, width=10, groups=3, period=10, ldy=10, ldg=10,
                                                    ldo=10), None, 1, None) == -1
    q = native.PostNorm(x=16, x_out=16, branch=16, gain=16, operand=16, H=64, ldb=64, branch2=16)
    assert lib.exo_post_norm_add(q, 1, 64, 0, None) == -1 and b"gain each" in lib.exo_last_error()
    lin = native.Linear(x=16, w=16, w_up=16, y=16, M=1, N=8, n1=8, ldx=64, ldw=64, ldy=8)
    assert lib.exo_linear_rows(lin, lin, None) == -1 and b"gated pair" in lib.exo_last_error()
    assert lib.exo_post_linear(q, lin, None) == -1
