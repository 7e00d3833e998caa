"""Configuration of layer-list decoders: models whose ``config.json`` spells out every layer.

A layer is a mixer and a feed-forward, each described by a small record of the mechanisms it
uses and their constants.  The records carry no design's name: a design is a reader that turns
its ``config.json`` into them (``READERS``), and the model (``stack_model.StackModel``) runs
whatever they describe.  Tensor names of these checkpoints: ``embed``, ``head``, ``final.norm``
and ``l<i>.<...>`` for layer i.
"""

from __future__ import annotations

import copy
import json
from dataclasses import dataclass
from pathlib import Path


@dataclass(frozen=True)
class AttentionSpec:
    heads: int
    kv_heads: int
    dim: int                     # query / key size per head
    vdim: int                    # value size per head
    scale: float
    window: int | None = None    # keys seen: fewer than this many positions back (None: all)
    keep_first: int = 0          # ... and the sequence's first positions, however far
    unit_qk: bool = False        # queries and keys divided by their RMS, per head
    slopes: tuple[float, ...] | None = None  # per query head: score lowered by slope * distance
    bias: bool = False           # projections have biases
    kv_from: int | None = None   # keys and values of that layer instead of own ones


@dataclass(frozen=True)
class ExpertSpec:
    """g = min(gate, limit), u = clamp(up, +-limit): g sigmoid(alpha g) (u + shift)."""

    ff: int
    limit: float
    alpha: float = 1.702
    shift: float = 1.0


@dataclass(frozen=True)
class RouterSpec:
    """softmax over experts + identity outputs; the ``top`` largest of score + correction; weight
    = score * scale.  An identity expert returns its input."""

    experts: int
    identity: int
    top: int
    scale: float

    @property
    def outputs(self) -> int:
        return self.experts + self.identity


@dataclass(frozen=True)
class MoeSpec:
    router: RouterSpec
    expert: ExpertSpec
    shared: ExpertSpec | None = None  # for every token, times sigmoid of one number per token


@dataclass(frozen=True)
class LayerSpec:
    mixer: AttentionSpec
    mlp: MoeSpec | None


@dataclass
class StackConfig:
    architecture: str
    vocab_size: int
    hidden_size: int
    eps: float
    layers: tuple[LayerSpec, ...]
    raw: dict                    # config.json as read

    def __post_init__(self):
        if min(self.vocab_size, self.hidden_size, len(self.layers)) <= 0:
            raise ValueError(f"{self.architecture}: vocab, width and the layer list must not be empty")
        for i, L in enumerate(self.layers):
            m, f = L.mixer, L.mlp
            if min(m.heads, m.kv_heads, m.dim, m.vdim) <= 0 or m.heads % m.kv_heads:
                raise ValueError(f"layer {i}: {m.heads} query heads over {m.kv_heads} key/value heads")
            if (m.window is not None and m.window <= 0) or m.keep_first < 0:
                raise ValueError(f"layer {i}: window {m.window} with {m.keep_first} kept positions")
            if m.kv_from is not None:
                src = self.layers[m.kv_from].mixer if 0 <= m.kv_from < i else None
                if src is None or src.kv_from is not None:
                    raise ValueError(f"layer {i}: kv_from {m.kv_from} is no earlier layer with keys of its own")
                if (src.kv_heads, src.dim, src.vdim) != (m.kv_heads, m.dim, m.vdim):
                    raise ValueError(f"layer {i}: head sizes differ from those of layer {m.kv_from}")
            if f is not None and not 0 < f.router.top <= f.router.outputs:
                raise ValueError(f"layer {i}: top {f.router.top} of {f.router.outputs} experts")

    # -- what the engine asks of any configuration
    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def model_type(self) -> str:
        return self.architecture

    @staticmethod
    def layer_of(key: str) -> int | None:
        """Layer index of a tensor name, None for the layer-independent ones."""
        head = key.split(".", 1)[0]
        return int(head[1:]) if head[:1] == "l" and head[1:].isdigit() else None

    def wants(self, key: str, start_layer: int, end_layer: int) -> bool:
        """Whether the shard [start_layer, end_layer) needs the tensor."""
        li = self.layer_of(key)
        if li is not None:
            return start_layer <= li < end_layer
        if key == "embed":
            return start_layer == 0
        return key in ("head", "final.norm") and end_layer == self.num_hidden_layers

    def to_dict(self) -> dict:
        return copy.deepcopy(self.raw)

    @staticmethod
    def from_dict(d: dict) -> "StackConfig":
        name = d.get("architecture")
        if name not in READERS:
            raise ValueError(f"architecture {name!r} not supported (have {tuple(READERS)})")
        return READERS[name](d)

    @staticmethod
    def from_path(model_dir: str | Path) -> "StackConfig":
        with open(Path(model_dir) / "config.json") as f:
            return StackConfig.from_dict(json.load(f))


# ------------------------------------------------------------------------------ designs


def distance_slopes(heads: int) -> tuple[float, ...]:
    """The geometric series 2^(-8/heads), 2^(-16/heads), ..., 2^-8."""
    return tuple(2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads))


def _gekazen(d: dict) -> StackConfig:
    """Gekazen: attention over a window with kept first tokens, linear distance penalty, unit-RMS
    queries and keys, biased projections, keys and values shared between layers; mixture of
    clamped gated experts with a choice correction, identity experts and a gated shared expert;
    norms on the sublayers' outputs."""

    def expert(e: dict) -> ExpertSpec:
        return ExpertSpec(ff=int(e["ff"]), limit=float(e["limit"]))

    layers = []
    for i, L in enumerate(d["layers"]):
        if L.get("type", "attention") != "attention":
            raise ValueError(f"layer {i}: mixer type {L['type']!r} not supported (have 'attention')")
        m, f = L["mixer"], L.get("mlp")
        mask = m.get("mask") or {}
        mixer = AttentionSpec(
            heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
            scale=float(m["scale"]), window=None if mask.get("size") is None else int(mask["size"]),
            keep_first=int(mask.get("keep_first") or 0), unit_qk=True,
            slopes=distance_slopes(int(m["heads"])), bias=True,
            kv_from=None if m.get("kv_from") is None else int(m["kv_from"]))
        mlp = None
        if f is not None:
            if f.get("kind", "moe") != "moe":
                raise ValueError(f"layer {i}: feed-forward kind {f['kind']!r} not supported (have 'moe')")
            r = f["router"]
            mlp = MoeSpec(
                RouterSpec(int(r["experts"]), int(r.get("identity") or 0), int(r["top"]), float(r["scale"])),
                expert(f["expert"]), expert(f["shared"]) if f.get("shared") else None)
        layers.append(LayerSpec(mixer, mlp))
    return StackConfig("Gekazen", int(d["vocab"]), int(d["width"]), float(d["norm"]["eps"]), tuple(layers),
                       copy.deepcopy(d))


READERS = {"Gekazen": _gekazen}


def gekazen_dict(width: int, vocab: int, layers: int, *, heads: int, kv_heads: int, dim: int, vdim: int, experts: int,
                 identity: int, top: int, ff: int, shared_ff: int | None = None, window: int | None = 4096,
                 keep_first: int = 4, router_scale: float = 1.0, limit: float = 7.0, eps: float = 1e-6,
                 kv_from: dict[int, int] | None = None) -> dict:
    """A ``config.json`` of the design with equal layers (benchmarks); ``kv_from``: layer -> the
    layer whose keys and values it uses."""
    out = []
    for i in range(layers):
        mixer = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=dim ** -0.5,
                     mask=dict(size=window, keep_first=keep_first))
        if kv_from and i in kv_from:
            mixer["kv_from"] = kv_from[i]
        mlp = dict(kind="moe", expert=dict(ff=ff, limit=limit),
                   router=dict(experts=experts, identity=identity, top=top, scale=router_scale))
        if shared_ff:
            mlp["shared"] = dict(ff=shared_ff, limit=limit)
        out.append(dict(type="attention", mixer=mixer, mlp=mlp))
    return dict(architecture="Gekazen", vocab=vocab, width=width, norm=dict(eps=eps), layers=out)
