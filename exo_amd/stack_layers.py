"""The layers of a layer-list decoder (``stack_config``): their tensors on the device and the launches
of each kind of mixer and feed-forward.

A layer's mixer is one or several parts over the same input.  The parts' projections are rows of one
matrix, so a layer starts with one product: columns in the element type (queries, keys, values, gates
of outputs, inputs of a convolution) and behind them float32 columns (what 32-bit arithmetic starts
from: step sizes, the low-rank decay, gates per head).  Each part turns its columns into the operand
of its own output projection.
"""

from __future__ import annotations

import torch

from . import dense_ops as D
from .dense_ops import pad64, padded
from .stack_config import (
    AttentionSpec, GluSpec, LayerSpec, LinearAttentionSpec, MoeSpec, NormSpec, ParallelSpec, StateSpaceSpec,
)


def pad8(n: int) -> int:
    return -(-n // 8) * 8


class Tensors:
    """The checkpoint's tensors under a name prefix, with shape checks."""

    def __init__(self, w: dict, prefix: str, dtype, device):
        self.w, self.prefix, self.dtype, self.device = w, prefix, dtype, device

    def at(self, name: str) -> "Tensors":
        return Tensors(self.w, self.prefix + name, self.dtype, self.device)

    def shape(self, name: str) -> tuple[int, ...]:
        return tuple(self.w[self.prefix + name].shape)

    def get(self, name: str, *shape: int) -> torch.Tensor:
        t = self.w[self.prefix + name]
        if tuple(t.shape) != shape:
            raise ValueError(f"{self.prefix}{name}: shape {tuple(t.shape)}, config says {shape}")
        return t.to(self.device)

    def f32(self, name: str, *shape: int) -> torch.Tensor:
        return self.get(name, *shape).float().contiguous()

    def mat(self, *parts) -> torch.Tensor:
        return padded(torch.cat([self.get(*x) for x in parts]), self.dtype, self.device)

    def gain(self, name: str | None, n: int, norm: NormSpec) -> torch.Tensor | None:
        return None if name is None else (norm.offset + self.get(name, n).float()).contiguous()


class _Part:
    """A mixer, or one of the parts of one.  ``main`` / ``tail``: its rows of the layer's projection, in
    element-type and float32 columns; ``biases`` of ``main`` (or None); ``col`` / ``tcol``: where its
    columns start; ``width``: columns of the operand that its output projection ``o`` takes."""

    main: list[torch.Tensor]
    tail: list[torch.Tensor]
    biases: list[torch.Tensor] | None = None
    o_b: torch.Tensor | None = None
    col = tcol = 0


class AttentionPart(_Part):
    def __init__(self, spec: AttentionSpec, t: Tensors, H: int, norm: NormSpec):
        self.spec = m = spec
        outs = [("q", m.heads * m.dim)]
        if m.kv_from is None:
            outs += [("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim)]
        self.main = [t.get(n, rows, H) for n, rows in outs]
        self.tail = [t.get("g", m.heads, H)] if m.head_gate else []
        self.width = m.heads * m.vdim
        self.o = t.mat(("o", H, self.width))
        if m.bias:
            self.biases = [t.get(f"{n}.b", rows) for n, rows in outs]
            self.o_b = t.f32("o.b", H)
        self.slopes = None if m.slopes is None else torch.tensor(m.slopes, dtype=torch.float32, device=t.device)
        self.q_gain = t.f32("q.norm", m.dim) if m.qk_gain else None
        self.k_gain = t.f32("k.norm", m.dim) if m.qk_gain and m.kv_from is None else None

    def bind(self, cache, kv_index: int, dtype, eps: float) -> D.PagedAttention:
        return D.PagedAttention(self.spec, self.slopes, kv_index, cache, eps, self.q_gain, self.k_gain)

    def run(self, att: D.PagedAttention, bf, b, y, y2, eps: float) -> torch.Tensor:
        m, n, own = self.spec, b.rows, self.spec.kv_from is None
        qkv, out = y[:, self.col :], bf.mixed("attn", self.width)
        gate = y2[:, self.tcol :] if m.head_gate else None
        if b.decode:
            att.rows(qkv, out, b.slot, b.pos, n, b.keys, append=own, gate=gate)
            return out
        if own:
            att.append(qkv, b.slot, b.pos, n)
        if b.blocks:
            att.prompt(qkv, out, *b.blocks[att.prompt_block(m)], gate=gate)
        if b.n_single:
            att.rows(qkv, out, b.slot, b.pos, b.n_single, b.keys, append=False, lst=b.single, gate=gate)
        return out


class _RecurrentPart(_Part):
    """What the recurrent mixers share: single tokens of a step and portions of prompts."""

    def bind(self, cache, state_index: int, dtype, eps: float) -> D.Recurrence:
        return D.Recurrence(self.spec.core, state_index, cache, dtype, self.consts)

    def _recur(self, rec: D.Recurrence, bf, b, cum: int, dt: bool) -> None:
        if b.decode:
            rec.step(b.slot, b.pos, b.rows)
            return
        if b.n_chunks:
            c, d = bf.f32("cum", cum), bf.f32("dt", cum) if dt else None
            if dt:  # a head's tokens in a run
                c, d = c.view(cum, -1), d.view(cum, -1)
            rec.chunks(b.chunks, b.n_chunks, b.seqs, b.n_seqs, c, d)
        if b.n_alone:
            rec.step(b.slot, b.pos, b.n_alone, lst=b.alone)


class LinearAttentionPart(_RecurrentPart):
    def __init__(self, spec: LinearAttentionSpec, t: Tensors, H: int, norm: NormSpec):
        self.spec = m = spec
        hd, he, self.rank = m.heads * m.dim, m.heads * m.vdim, t.shape("a1")[0]
        self.main = [t.get("q", hd, H), t.get("k", hd, H), t.get("v", he, H), t.get("g", he, H)]
        self.tail = [t.get("a1", self.rank, H)]
        self.width = he
        self.o = t.mat(("o", H, he))
        self.norm = t.f32("norm", m.vdim)
        self.decay_w = t.get("a2", hd, self.rank).float().t().contiguous()  # [rank, heads * dim]
        self.decay_b = t.f32("a2.b", hd)
        self.consts = dict(per_channel=1, rank=self.rank, decay_w=self.decay_w, decay_b=self.decay_b,
                           inv_tau=1.0 / m.tau, q_scale=m.dim ** -0.5)

    def run(self, rec: D.Recurrence, bf, b, y, y2, eps: float) -> torch.Tensor:
        m = self.spec
        hd, he = m.heads * m.dim, self.width
        o, out = bf.f32("recur", he), bf.mixed("recur_out", he)
        cols = y[:, self.col :]
        rec.bind(o, q=(cols, "ldq"), k=(cols[:, hd:], "ldk"), v=(cols[:, 2 * hd :], "ldv"), low=(y2[:, self.tcol :], "ldlow"))
        self._recur(rec, bf, b, hd, dt=False)
        D.gated_norm(o, cols[:, 2 * hd + he :], self.norm, out, b.rows, he, m.heads, eps, gate_first=False)
        return out


class StateSpacePart(_RecurrentPart):
    def __init__(self, spec: StateSpaceSpec, t: Tensors, H: int, norm: NormSpec):
        self.spec = m = spec
        inner, ch = m.inner, m.channels
        w = t.get("in", inner + ch + m.heads, H)  # z | values, keys, queries | step sizes
        self.main, self.tail = [w[:inner], w[inner : inner + ch]], [w[inner + ch :]]
        self.width = inner
        self.o = t.mat(("o", H, inner))
        self.norm = t.f32("norm", inner)
        self.conv_w = t.get("conv", ch, m.conv).float().t().contiguous()  # [taps, channels]
        self.conv_b = t.f32("conv.b", ch)
        self.dt_bias, self.skip = t.f32("dt_bias", m.heads), t.f32("D", m.heads)
        self.decay_rate = torch.exp(t.f32("A_log", m.heads))
        self.consts = dict(per_channel=0, conv_w=self.conv_w, conv_b=self.conv_b, dt_bias=self.dt_bias,
                           decay_rate=self.decay_rate, skip=self.skip, q_scale=1.0, v_channel=0, k_channel=inner,
                           q_channel=inner + m.groups * m.state)

    def run(self, rec: D.Recurrence, bf, b, y, y2, eps: float) -> torch.Tensor:
        m, inner = self.spec, self.width
        gn = m.groups * m.state
        o, out, act = bf.f32("recur", inner), bf.mixed("recur_out", inner), bf.cols("conv", pad8(m.channels))
        cols = y[:, self.col :]
        rec.bind(o, raw=(cols[:, pad8(inner) :], "ldraw"), act=(act, "ldact"), v=(act, "ldv"), k=(act[:, inner:], "ldk"),
                 q=(act[:, inner + gn :], "ldq"), dt_raw=(y2[:, self.tcol :], "lddt"))
        self._recur(rec, bf, b, m.heads, dt=True)
        D.gated_norm(o, cols, self.norm, out, b.rows, inner, m.norm_groups, eps, gate_first=True)
        return out


class DenseFF:
    def __init__(self, spec: GluSpec, t: Tensors, H: int):
        self.spec = spec
        self.gate, self.up = t.mat(("gate", spec.ff, H)), t.mat(("up", spec.ff, H))
        self.down = t.mat(("down", H, spec.ff))


class MoeFF:
    """Experts stacked; the shared expert's gate is one more output of the router product."""

    def __init__(self, spec: MoeSpec, t: Tensors, H: int):
        self.spec = f = spec
        r, ff = f.router, f.expert.ff

        def stack(name: str, n: int, k: int) -> torch.Tensor:
            out = torch.zeros(r.experts, n, pad64(k), dtype=t.dtype, device=t.device)
            for e in range(r.experts):
                out[e, :, :k].copy_(t.get(f"e{e}.{name}", n, k))
            return out

        self.gate, self.up, self.down = stack("gate", ff, H), stack("up", ff, H), stack("down", H, ff)
        self.correction = t.f32("correction", r.outputs)
        rows = [("router", r.outputs, H)]
        self.s_gate = self.s_up = self.s_down = None
        if f.shared is not None:
            rows.append(("shared.sg", 1, H))
            self.s_gate, self.s_up = t.mat(("shared.gate", f.shared.ff, H)), t.mat(("shared.up", f.shared.ff, H))
            self.s_down = t.mat(("shared.down", H, f.shared.ff))
        self.router = t.mat(*rows)


class Layer:
    """One layer's tensors: the parts of its mixer behind one projection, its feed-forward, its norms."""

    def __init__(self, spec: LayerSpec, w: dict, i: int, H: int, norm: NormSpec, dtype, device):
        self.index, self.spec = i, spec
        t = Tensors(w, f"l{i}.", dtype, device)
        self.pre1, self.norm1 = (t.gain(n, H, norm) for n in norm.names(1))
        m, mix = spec.mixer, t.at("mix.")
        self.gain_a = self.gain_b = None
        if isinstance(m, ParallelSpec):
            self.parts = [AttentionPart(m.left, mix.at("left."), H, norm), StateSpacePart(m.right, mix.at("right."), H, norm)]
            self.gain_a, self.gain_b = mix.f32("left.out", H), mix.f32("right.out", H)
        else:
            kinds = {AttentionSpec: AttentionPart, LinearAttentionSpec: LinearAttentionPart, StateSpaceSpec: StateSpacePart}
            self.parts = [kinds[type(m)](m, mix, H, norm)]
        self._project(H, dtype, device)
        self.ff = self.pre2 = self.norm2 = None
        if spec.mlp is not None:
            self.ff = (MoeFF if isinstance(spec.mlp, MoeSpec) else DenseFF)(spec.mlp, t.at("mlp."), H)
            self.pre2, self.norm2 = (t.gain(n, H, norm) for n in norm.names(2))

    def _project(self, H: int, dtype, device) -> None:
        """The parts' rows one below the other, element-type columns first.  An attention part's q, k, v are
        one run; otherwise every block of columns starts at a multiple of 8 (vector loads)."""
        rows, biases, at = [], [], 0
        any_bias = any(p.biases is not None for p in self.parts)

        def pad(n: int) -> None:
            nonlocal at
            if n:
                rows.append(torch.zeros(n, H, dtype=torch.bfloat16, device=device))
                biases.append(torch.zeros(n, device=device))
                at += n

        for p in self.parts:
            pad(-at % 8)
            p.col = at
            for i, m in enumerate(p.main):
                if isinstance(p, StateSpacePart):
                    pad(-at % 8)
                rows.append(m)
                biases.append(torch.zeros(m.shape[0], device=device) if p.biases is None else p.biases[i].float())
                at += m.shape[0]
        self.n_main, self.n_tail = at, 0
        for p in self.parts:
            p.tcol = self.n_tail
            for m in p.tail:
                rows.append(m)
                biases.append(torch.zeros(m.shape[0], device=device))
                self.n_tail += m.shape[0]
            p.main = p.tail = []
        self.proj = padded(torch.cat(rows), dtype, device)
        self.proj_b = torch.cat(biases).float().contiguous() if any_bias else None

    def tensors(self) -> list[torch.Tensor]:
        holders = [self, *self.parts] + ([self.ff] if self.ff is not None else [])
        return [t for h in holders for t in vars(h).values() if isinstance(t, torch.Tensor)]
