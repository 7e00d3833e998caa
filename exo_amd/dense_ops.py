"""Operators of the layer-list decoders on torch device tensors (C ABI of include/exo_mi355x.h):
products with unquantised matrices, residual norms, routing, experts and attention over a paged
pool.  Element type bf16 or float32 throughout (the tensors' dtype decides); like ``ops``, every
function launches on torch's current stream and never synchronises.

Matrix operands have row strides of multiples of 64 elements with zeros past the logical size
(``padded``): no kernel has a tail in K.
"""

from __future__ import annotations

import ctypes as C

import torch

from . import native
from .native import check
from .ops import _ptr, _stream

GEMV_MAX_ROWS = 16


def pad64(n: int) -> int:
    return -(-n // 64) * 64


def padded(w: torch.Tensor, dtype, device) -> torch.Tensor:
    """[..., N, K] -> contiguous [..., N, pad64(K)] of ``dtype`` with zeros behind K."""
    out = torch.zeros(*w.shape[:-1], pad64(w.shape[-1]), dtype=dtype, device=device)
    out[..., : w.shape[-1]].copy_(w)
    return out


def _code(t: torch.Tensor) -> int:
    if t.dtype == torch.bfloat16:
        return 0
    if t.dtype == torch.float32:
        return 1
    raise ValueError(f"element type {t.dtype} not supported (bfloat16, float32)")


def embed_rows(ids, table, x, xb, H: int) -> None:
    n = ids.numel()
    check(native.load().exo_embed_rows(_ptr(ids), _ptr(table), _ptr(x), _ptr(xb), n, table.shape[0], H,
                                       table.shape[1], xb.shape[1], _code(xb), _stream()), "embed_rows")


def norm_rows(x, gain, eps: float, out, n: int, rows=None) -> None:
    check(native.load().exo_norm_rows(_ptr(x), _ptr(rows), _ptr(gain), _ptr(out), n, gain.numel(), out.shape[1], eps,
                                      _code(out), _stream()), "norm_rows")


def post_norm_add(branch, gain, eps: float, x, xb, n: int) -> None:
    """x += norm(branch); xb = x in the element type.  branch and x float32."""
    check(native.load().exo_post_norm_add(_ptr(branch), branch.shape[1], _ptr(gain), _ptr(x), _ptr(xb), n,
                                          gain.numel(), xb.shape[1], eps, _code(xb), _stream()), "post_norm_add")


def moe_sum_post_norm(y, idx, wt, shared, logits, experts: int, gate_col: int, gain, eps: float, x, xb, n: int) -> None:
    """x += norm(weighted sum of the chosen experts' outputs y [n, top, ld] + gated shared)."""
    check(native.load().exo_moe_sum_post_norm(
        _ptr(y), _ptr(idx), _ptr(wt), _ptr(shared), _ptr(logits), idx.shape[1], experts, y.shape[-1],
        0 if shared is None else shared.shape[1], logits.shape[1], gate_col, _ptr(gain), _ptr(x), _ptr(xb), n,
        gain.numel(), xb.shape[1], eps, _code(xb), _stream()), "moe_sum_post_norm")


def moe_route(logits, correction, scale: float, idx, wt, n: int) -> None:
    check(native.load().exo_moe_route(_ptr(logits), _ptr(correction), _ptr(idx), _ptr(wt), n, correction.numel(),
                                      logits.shape[1], idx.shape[1], scale, _stream()), "moe_route")


_GEMM_WS: dict[int, torch.Tensor] = {}
GEMM_WS_FLOATS = 1 << 24


def gemm_workspace(device) -> torch.Tensor:
    """Float32 partial tiles of GEMMs that split K; one per device (work is in stream order)."""
    key = torch.device(device).index or 0
    if key not in _GEMM_WS:
        _GEMM_WS[key] = torch.empty(GEMM_WS_FLOATS, dtype=torch.float32, device=device)
    return _GEMM_WS[key]


def linear(x, w, out, n: int, bias=None, force_gemm: bool = False) -> None:
    """out[:n] = x[:n] @ w^T (+ bias float32); out in x's element type or float32."""
    lib, N = native.load(), w.shape[0]
    f32 = int(out.dtype == torch.float32)
    if n <= GEMV_MAX_ROWS and not force_gemm:
        check(lib.exo_dense_gemv(_ptr(x), _ptr(w), _ptr(bias), _ptr(out), f32, n, N, x.shape[1], w.shape[1],
                                 out.shape[1], _code(x), _stream()), "linear")
        return
    ws = gemm_workspace(x.device)
    check(lib.exo_dense_gemm(_ptr(x), _ptr(w), _ptr(bias), _ptr(out), f32, _ptr(ws), ws.numel(), n, N, x.shape[1],
                             w.shape[1], out.shape[1], _code(x), _stream()), "linear(gemm)")


POST_MAX_ROWS = 4  # beyond, every workgroup repeating the norm costs more than a launch


def post_linear_fits(n: int, w, xb, H: int) -> bool:
    return n <= POST_MAX_ROWS and bool(native.load().exo_post_gemv_fits(n, w.shape[0], H, xb.shape[1], _code(xb)))


def post_linear(x, branch, gain, eps: float, x_out, xb, w, out, n: int, bias=None) -> None:
    """``post_norm_add`` and ``linear`` in one launch: x_out = x + norm(branch) (another buffer than
    x), xb (may be None) its copy, out = x_out @ w^T (+ bias)."""
    check(native.load().exo_post_gemv(
        _ptr(x), _ptr(branch), _ptr(gain), eps, _ptr(x_out), _ptr(xb), _ptr(w), _ptr(bias), _ptr(out),
        int(out.dtype == torch.float32), n, w.shape[0], gain.numel(), w.shape[1], w.shape[1], out.shape[1], _code(w),
        _stream()), "post_linear")


def glu_gemm(x, gate, up, out, n: int, spec) -> None:
    """out[:n] = clamped gated unit of x[:n] (any n)."""
    check(native.load().exo_dense_glu_gemm(
        _ptr(x), _ptr(gate), _ptr(up), _ptr(out), spec.limit, spec.alpha, spec.shift, n, gate.shape[0], x.shape[1],
        gate.shape[1], out.shape[1], _code(x), _stream()), "glu_gemm")


def grouped_gemm(x, w, group_ws, out, T: int, topk: int, up=None, spec=None, x_per_pair: bool = False) -> None:
    """Experts w [E, N, K] over (token, slot) pairs sorted by ``ops.moe_group``: out row = pair.
    ``up`` and ``spec``: the gated pair."""
    lim, al, sh = (spec.limit, spec.alpha, spec.shift) if up is not None else (0.0, 0.0, 0.0)
    check(native.load().exo_dense_grouped_gemm(
        _ptr(x), _ptr(w), _ptr(up), _ptr(group_ws), _ptr(out), lim, al, sh, T, topk, int(x_per_pair), w.shape[0],
        w.shape[1], x.shape[-1], w.shape[2], out.shape[-1], _code(x), _stream()), "grouped_gemm")


class ExpertRows:
    """The experts of a decode step (up to 16 rows): argument block built once per layer and
    residual buffer, launched as gated products (which also route) and as weighted down-projections."""

    def __init__(self, moe, w, bf, H: int, h):
        """``moe``: MoeSpec; ``w``: the layer's tensors; ``bf``: the activation buffers; ``h``: the
        residual that enters the feed-forward."""
        r, e, s = moe.router, moe.expert, moe.shared
        p = lambda t: None if t is None else t.data_ptr()  # noqa: E731
        self.args = native.MoeRows(
            x=p(bf.xb), gate=p(w.gate), up=p(w.up), down=p(w.down),
            shared_gate=p(w.s_gate), shared_up=p(w.s_up), shared_down=p(w.s_down),
            act=p(bf.act(r.top, e.ff)), shared_act=p(bf.shared_act(s.ff)) if s else None, out=p(bf.branch),
            x_res=p(h), idx=p(bf.idx(r.top)), wt=p(bf.wt(r.top)), logits=p(bf.router_logits(w.router.shape[0])),
            correction=p(w.correction),
            top=r.top, experts=r.experts, ff=e.ff, shared_ff=s.ff if s else 0, H=H, ldx=bf.xb.shape[1],
            lda=pad64(e.ff), ldsa=pad64(s.ff) if s else 0, ldl=w.router.shape[0], gate_col=r.outputs, outputs=r.outputs, router_scale=r.scale,
            dtype=_code(bf.xb), limit=e.limit, alpha=e.alpha, shift=e.shift,
            shared_limit=s.limit if s else 0.0, shared_alpha=s.alpha if s else 0.0, shared_shift=s.shift if s else 0.0)

    def glu(self, n: int) -> None:
        self.args.rows = n
        check(native.load().exo_moe_glu_rows(C.byref(self.args), _stream()), "moe_glu_rows")

    def down(self, n: int) -> None:
        self.args.rows = n
        check(native.load().exo_moe_down_rows(C.byref(self.args), _stream()), "moe_down_rows")


_ATTN_WS: dict[int, list[torch.Tensor]] = {}


def attn_workspace(n: int, heads: int, vdim: int, nsplit: int, device) -> torch.Tensor:
    """Partials and arrival counters of split decode attention, one per device, grown on demand (a
    replaced buffer stays alive: a captured graph may point at it)."""
    need = native.load().exo_paged_attn_workspace(n, heads, vdim, nsplit)
    key = torch.device(device).index or 0
    have = _ATTN_WS.setdefault(key, [])
    if not have or have[-1].numel() < need:
        have.append(torch.zeros(need, dtype=torch.uint8, device=device))  # counters start at zero
    return have[-1]


class PagedAttention:
    """Attention of one layer over a paged pool.  ``spec``: AttentionSpec; ``li``: index of the
    pool's layer that holds its keys and values."""

    def __init__(self, spec, slopes, li: int, cache, eps: float):
        self.spec, self.slopes, self.cache = spec, slopes, cache
        k, v = cache.k[li], cache.v[li]
        self.args = native.PagedAttn(
            k_pool=k.data_ptr(), v_pool=v.data_ptr(), table=cache.table.data_ptr(),
            slopes=None if slopes is None else slopes.data_ptr(), scale=spec.scale, eps=eps,
            heads=spec.heads, kv_heads=spec.kv_heads, dim=spec.dim, vdim=spec.vdim, ldk=k.shape[3], ldv=v.shape[2],
            max_pages=cache.table.shape[1], window=spec.window or 0, keep_first=spec.keep_first,
            unit_qk=int(spec.unit_qk), dtype=_code(k))

    def _bind(self, qkv, out, slot, pos, lst, n: int):
        a = self.args
        assert qkv.dtype == self.cache.k[0].dtype
        a.qkv, a.ldq, a.n = qkv.data_ptr(), qkv.shape[1], n
        a.out, a.ldo = (None, 0) if out is None else (out.data_ptr(), out.shape[1])
        a.slot = None if slot is None else slot.data_ptr()
        a.pos = None if pos is None else pos.data_ptr()
        a.list = None if lst is None else lst.data_ptr()
        return C.byref(a)

    def append(self, qkv, slot, pos, n: int) -> None:
        check(native.load().exo_paged_append(self._bind(qkv, None, slot, pos, None, n), _stream()), "paged_append")

    def visible(self, keys: int) -> int:
        """Most keys one query sees when its sequence holds ``keys``."""
        s = self.spec
        return keys if s.window is None else min(keys, s.window + s.keep_first)

    def rows(self, qkv, out, slot, pos, n: int, keys: int, append: bool, lst=None) -> None:
        """One query position per row (``lst``: which rows, else the first n).  ``keys``: most keys
        any of the sequences holds, as the host knows it (lays out the launch)."""
        s = self.spec
        tiles = -(-self.visible(keys) // 32) + 2
        wgs = n * s.kv_heads * (-(-(s.heads // s.kv_heads) // 16))
        nsplit = max(1, min(-(-tiles // 4), 256 // wgs, 16))
        if nsplit > 8:
            nsplit -= nsplit % 8  # (the head groups of one split then share an XCD's L2)
        if n * s.heads > 16384:
            nsplit = 1
        ws = attn_workspace(n, s.heads, s.vdim, nsplit, qkv.device) if nsplit > 1 else None
        check(native.load().exo_paged_attn_rows(self._bind(qkv, out, slot, pos, lst, n), nsplit, int(append), _ptr(ws),
                                                0 if ws is None else ws.numel(), _stream()), "paged_attn_rows")

    @staticmethod
    def prompt_block(spec) -> int:
        return native.load().exo_paged_prompt_block(spec.heads, spec.kv_heads)

    def prompt(self, qkv, out, blocks, n: int) -> None:
        """Portions of prompts: blocks int32 [n, 4] = first row, slot, first position, tokens."""
        check(native.load().exo_paged_attn_prompt(self._bind(qkv, out, None, None, blocks, n), _stream()),
              "paged_attn_prompt")
