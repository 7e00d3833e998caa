"""Paged KV pool: pages of 64 positions shared by all sequences of a batch.

The cache protocol of ``ShardKVCache`` (rows, ``offsets``, ``pos``, trim / reset / copy_row) over a
pool whose size is given in tokens, not rows x longest sequence: a row owns the pages its tokens
need, through a page table on the device, and gives them back when it is trimmed, reset or
released.  One table serves every layer.  Recurrent layers keep their fixed-size states in slots beside
the pages (``state_pool``); a row then cannot be cut back to an earlier position, only to none.

Per layer with keys of its own (layers that use another layer's keys have no storage):
  k[i]  [pages, G, 64, ldk]   keys as attention uses them (normalised)
  v[i]  [pages, G, ldv, 64]   values, transposed inside the page (matrix-core operand order)
with ldk, ldv the head sizes rounded up to 32; the padding stays zero.  Latent attention keeps one "key" per
position - the normed latent, and behind it the shared rotated key part - and no values.
"""

from __future__ import annotations

import torch

from .cache import LayerKV
from .state_pool import StatePool, StateShape

PAGE = 64


class PoolExhausted(RuntimeError):
    """No free page for a token that is about to be appended."""


def pages_for(tokens: int) -> int:
    return -(-tokens // PAGE)


class PagedKVCache(list):
    """list[LayerKV] (one per layer with keys of its own and per recurrent state) plus the pools."""

    def __init__(self, layers: list[tuple[int, int, int]], rows: int, max_seq: int, device, dtype=torch.bfloat16,
                 pool_tokens: int | None = None, states: list[StateShape] = ()):
        """``layers``: (kv heads, key size, value size) per storing layer.  ``max_seq``: the longest
        sequence a row may hold; ``pool_tokens``: tokens all rows hold together, each row's count
        rounded up to whole pages (default: every row at ``max_seq``); ``states``: the recurrent layers'."""
        super().__init__(LayerKV(self, i) for i in range(len(layers) + len(states)))
        self.batch, self.max_seq, self.shapes = rows, max_seq, list(layers)
        self.n_pages = rows * pages_for(max_seq) if pool_tokens is None else pages_for(pool_tokens)
        self.max_pages = min(pages_for(max_seq), self.n_pages)
        pad = lambda d: -(-d // 32) * 32  # noqa: E731
        z = dict(dtype=dtype, device=device)
        self.k = [torch.zeros(self.n_pages, g, PAGE, pad(d), **z) for g, d, _ in layers]
        self.v = [torch.zeros(self.n_pages, g, pad(e), PAGE, **z) for g, _, e in layers]
        self.states = StatePool(states, rows, device, dtype)
        self.table = torch.zeros(rows, self.max_pages, dtype=torch.int32, device=device)
        self.pos = torch.zeros(rows, dtype=torch.int32, device=device)
        self.offsets = [0] * rows
        self.pages: list[list[int]] = [[] for _ in range(rows)]
        self._free = list(range(self.n_pages - 1, -1, -1))
        self._last_trim = 0

    # -- recurrent states
    @property
    def trimmable(self) -> bool:
        """Whether a row can go back to an earlier position (a recurrent state cannot)."""
        return not len(self.states)

    def save_states(self, rows) -> list[torch.Tensor]:
        return self.states.read(rows)

    def load_states(self, rows, saved: list[torch.Tensor]) -> None:
        self.states.write(rows, saved)

    # -- pages
    @property
    def free_tokens(self) -> int:
        return len(self._free) * PAGE

    def reserve(self, rows, n: int) -> None:
        """Pages for ``n`` more tokens in each of ``rows``; raises before anything changes if a row
        or the pool cannot hold them."""
        self.reserve_each([(r, n) for r in rows])

    def reserve_each(self, wants: list[tuple[int, int]]) -> None:
        need = []
        for r, n in wants:
            if self.offsets[r] + n > self.max_seq:
                raise ValueError(f"KV cache overflow: {self.offsets[r]}+{n} > {self.max_seq}")
            need.append(max(0, pages_for(self.offsets[r] + n) - len(self.pages[r])))
        if sum(need) > len(self._free):
            raise PoolExhausted(f"{sum(need)} pages of {PAGE} tokens wanted, {len(self._free)} free")
        for (r, _), k in zip(wants, need):
            if k:
                new = [self._free.pop() for _ in range(k)]
                at = len(self.pages[r])
                self.pages[r] += new
                self.table[r, at : at + k].copy_(torch.tensor(new, dtype=torch.int32))

    def _give_back(self, row: int, keep_tokens: int) -> None:
        keep = pages_for(keep_tokens)
        self._free += reversed(self.pages[row][keep:])
        del self.pages[row][keep:]

    # -- fill level (ShardKVCache's protocol)
    def advance_host(self, t: int, rows=None) -> None:
        for r in (range(self.batch) if rows is None else rows):
            self.offsets[r] += t

    def sync_pos(self) -> None:
        self.pos.copy_(torch.tensor(self.offsets, dtype=torch.int32), non_blocking=False)

    def trim(self, n: int, rows=None) -> int:
        rows = range(self.batch) if rows is None else rows
        n = min([n] + [self.offsets[r] for r in rows])
        if n and not self.trimmable and any(self.offsets[r] != n for r in rows):
            raise ValueError("a recurrent state cannot be cut back to an earlier position")
        for r in rows:
            self.offsets[r] -= n
            self._give_back(r, self.offsets[r])
        self.sync_pos()
        return n

    def reset(self, rows=None) -> None:
        for r in (range(self.batch) if rows is None else rows):
            self.offsets[r] = 0
            self._give_back(r, 0)
        self.sync_pos()

    def release(self, row: int) -> None:
        """The row's sequence is finished: its pages go back to the pool."""
        self.reset(rows=[row])

    def copy_row(self, src: int, dst: int) -> None:
        """Move one sequence to another row (slot compaction): pages and state slot change hands,
        no key or state moves."""
        self._give_back(dst, 0)
        self.pages[dst], self.pages[src] = self.pages[src], []
        self.table[dst].copy_(self.table[src])
        self.offsets[dst], self.offsets[src] = self.offsets[src], 0
        self.states.swap(src, dst)
        self.sync_pos()

    def swap_rows(self, a: int, b: int) -> None:
        if a == b:
            return
        self.pages[a], self.pages[b] = self.pages[b], self.pages[a]
        self.offsets[a], self.offsets[b] = self.offsets[b], self.offsets[a]
        self.table[[a, b]] = self.table[[b, a]]
        self.states.swap(a, b)
        self.sync_pos()

    def nbytes(self) -> int:
        return sum(t.numel() * t.element_size() for t in self.k + self.v) + self.states.nbytes()

    # -- one row's contents as [n, G, size] tensors (prefix cache, wire)
    def _row_pages(self, row: int, lo: int, hi: int) -> torch.Tensor:
        return torch.tensor(self.pages[row][lo // PAGE : pages_for(hi)], dtype=torch.int64, device=self.pos.device)

    def read_nhd(self, layer: int, row: int, start: int, n: int) -> tuple[torch.Tensor, torch.Tensor]:
        """Keys [n, G, D] and values [n, G, E] of positions [start, start + n)."""
        g, d, e = self.shapes[layer]
        idx, off = self._row_pages(row, start, start + n), start % PAGE
        rows = len(idx) * PAGE
        k = self.k[layer][idx].permute(0, 2, 1, 3).reshape(rows, g, self.k[layer].shape[-1])
        v = self.v[layer][idx].permute(0, 3, 1, 2).reshape(rows, g, self.v[layer].shape[2])
        return k[off : off + n, :, :d].contiguous(), v[off : off + n, :, :e].contiguous()

    def write_nhd(self, layer: int, row: int, start: int, k: torch.Tensor, v: torch.Tensor) -> None:
        """Positions [start, start + n) from keys [n, G, D] and values [n, G, E]; the row must own
        their pages (``reserve``)."""
        n = k.shape[0]
        g, d, e = self.shapes[layer]
        if tuple(k.shape[1:]) != (g, d) or tuple(v.shape) != (n, g, e):
            raise ValueError(f"keys {tuple(k.shape)} / values {tuple(v.shape)} do not fit layer {layer} ({g}, {d}, {e})")
        at = torch.arange(start, start + n, device=self.pos.device)
        page = self._row_pages(row, 0, start + n)[at // PAGE]
        self.k[layer][page, :, at % PAGE, :d] = k.to(self.k[layer].dtype)
        self.v[layer][page, :, :e, at % PAGE] = v.to(self.v[layer].dtype)

    def snapshot(self, row: int) -> list[tuple[torch.Tensor, torch.Tensor]]:
        """Detached copy of the row's positions, per layer (keys, values), then the recurrent
        states (one entry of all of them, if there are any)."""
        kv = [self.read_nhd(i, row, 0, self.offsets[row]) for i in range(len(self.k))]
        return kv + ([tuple(self.states.read([row]))] if len(self.states) else [])

    def restore(self, row: int, layers: list[tuple[torch.Tensor, torch.Tensor]], length: int) -> None:
        self.reset(rows=[row])
        self.reserve([row], length)
        if len(self.states):
            self.states.write([row], list(layers[-1]))
        for i, (k, v) in enumerate(layers[: len(self.k)]):
            self.write_nhd(i, row, 0, k[:length], v[:length])
        self.offsets[row] = length
        self.sync_pos()
