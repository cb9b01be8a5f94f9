"""Configuration of the hybrid decoder designs.

A design is a list of layers, each with a mixer (softmax attention or the gated delta rule)
and an optional dense feed-forward that reads the same norm (a parallel layer), a norm whose
weight is stored around an offset, a residual multiplier, and an optional looped section:
layers ``start .. stop-1`` run ``times`` times with the same weights, each pass on its own
cache, entered through a projection of [x ; embedding] plus a per-pass vector.

``from_config`` reads the ``config.json`` of a named design; what a design fixes (sink,
normalised queries and keys, output gate, activation) is set there as parameters of the
mechanism.
"""
from __future__ import annotations

import json
from dataclasses import dataclass, field
from pathlib import Path


@dataclass(frozen=True)
class Rotary:
    """Interleaved partial rotary positions: neighbours (2i, 2i+1) of the first ``dims``
    dimensions turn by p * base^(-2i/dims)."""
    dims: int
    base: float


@dataclass(frozen=True)
class AttentionMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Rotary | None
    qk_norm: bool = True   # q, k / rms over the head, after the rotation
    sink: bool = True      # one extra exp(0) in the softmax denominator
    gated: bool = True     # heads * sigmoid(W_g h) before the output projection
    kind = "attention"


@dataclass(frozen=True)
class DeltaMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    taps: int
    kind = "delta"


@dataclass(frozen=True)
class DenseMlp:
    ff: int
    act: str = "gelu"      # exact (erf)


@dataclass(frozen=True)
class Layer:
    mixer: AttentionMixer | DeltaMixer
    mlp: DenseMlp | None


@dataclass(frozen=True)
class Loop:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class Run:
    """One execution of a layer in a token step (a looped layer has one per pass)."""
    index: int             # cache / state index
    layer: int
    enter: int | None      # pass entered right before this run


@dataclass
class HybridConfig:
    name: str
    vocab_size: int
    hidden_size: int
    layers: list[Layer]
    eps: float
    residual_mult: float = 1.0
    norm_offset: float = 1.0
    loop: Loop | None = None
    bos_token_id: int | None = None
    eos_token_id: list[int] = field(default_factory=list)

    def __post_init__(self):
        n, lp = len(self.layers), self.loop
        if n == 0 or self.hidden_size < 1 or self.vocab_size < 1:
            raise ValueError("a model needs layers, a width and a vocabulary")
        if lp is not None and not (0 <= lp.start < lp.stop <= n and lp.times >= 1):
            raise ValueError(f"loop {lp} does not fit {n} layers")

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @property
    def width_padded(self) -> int:
        """Row length of residual rows and of the weights' input side."""
        return -(-self.hidden_size // 8) * 8

    def runs(self) -> list[Run]:
        n, lp = len(self.layers), self.loop
        order: list[tuple[int, int | None]] = []
        for i in range(n):
            if lp is None or i < lp.start or i >= lp.stop:
                order.append((i, None))
            elif i == lp.start:
                order += [(j, t if j == lp.start else None)
                          for t in range(lp.times) for j in range(lp.start, lp.stop)]
        return [Run(k, i, t) for k, (i, t) in enumerate(order)]


def _eos(d: dict) -> list[int]:
    e = d.get("eos_token_id")
    return [] if e is None else [int(x) for x in e] if isinstance(e, list) else [int(e)]


def _fonapel_layer(d: dict) -> Layer:
    m = d["mixer"]
    sizes = dict(heads=int(m["heads"]), kv_heads=int(m["kv_heads"]), dim=int(m["dim"]),
                 vdim=int(m["vdim"]))
    if d["type"] == "attention":
        rot = m.get("rot")
        mixer = AttentionMixer(**sizes, scale=float(m["scale"]),
                               rot=Rotary(int(rot["dims"]), float(rot["base"])) if rot else None)
    elif d["type"] == "delta":
        mixer = DeltaMixer(**sizes, taps=int(m["conv"]))
    else:
        raise ValueError(f"unknown mixer type {d['type']!r}")
    mlp = d.get("mlp")
    if mlp is not None and mlp.get("kind", "dense") != "dense":
        raise ValueError(f"unknown feed-forward kind {mlp['kind']!r}")
    return Layer(mixer, None if mlp is None else DenseMlp(int(mlp["ff"])))


def fonapel(d: dict) -> HybridConfig:
    """The Fonapel design: parallel layers, attention with a sink, normalised rotated queries
    and keys and a sigmoid output gate, gated delta layers, erf-GELU feed-forwards."""
    lp = d.get("loop")
    return HybridConfig(
        name="fonapel", vocab_size=int(d["vocab"]), hidden_size=int(d["width"]),
        layers=[_fonapel_layer(x) for x in d["layers"]], eps=float(d["norm"]["eps"]),
        residual_mult=float(d.get("residual_mult", 1.0)), norm_offset=1.0,
        loop=Loop(int(lp["start"]), int(lp["stop"]), int(lp["times"])) if lp else None,
        bos_token_id=d.get("bos_token_id"), eos_token_id=_eos(d))


DESIGNS = {"Fonapel": fonapel}   # config.json "architecture" -> reader


def from_config(d: dict) -> HybridConfig:
    try:
        read = DESIGNS[d["architecture"]]
    except KeyError:
        raise ValueError(f"unknown hybrid design {d.get('architecture')!r}") from None
    return read(d)


def from_path(path: str | Path) -> HybridConfig:
    p = Path(path)
    return from_config(json.loads((p / "config.json" if p.is_dir() else p).read_text()))
