"""Weights of the hybrid designs, laid out for the kernels.

A parallel layer reads one norm and sums its two sublayers, so it has two matrices:

* ``w_in``  [mixer projections | feed-forward up, width padded to 8] — rows q | k | v | gate
  (delta: then a | b) and the feed-forward's up rows;
* ``w_out`` [width, mixer output | feed-forward down] — the columns of both output
  projections side by side (each padded to 8 with zero columns).

Input columns past the width are zero.  Constants that enter 32-bit computations (norm
weights, convolution taps, decays) are kept in f32.

Tensor names: ``embed``, ``head``, ``final.norm``, ``loop.in``, ``loop.step``, and per layer
``l<i>.norm1``, ``l<i>.mix.*``, ``l<i>.mlp.{up,down}``; linear weights are [out, in].
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Callable

import torch

from ...ops.mixers import AttnShape, DeltaShape, pad_to
from .config import AttentionMixer, DeltaMixer, HybridConfig, Layer

Getter = Callable[[str], torch.Tensor]


def _shaped(get: Getter, name: str, shape: tuple) -> torch.Tensor:
    t = get(name)
    if tuple(t.shape) != shape:
        raise ValueError(f"{name}: shape {tuple(t.shape)} != {shape}")
    return t


def mixer_shape(m: AttentionMixer | DeltaMixer) -> AttnShape | DeltaShape:
    if isinstance(m, AttentionMixer):
        return AttnShape(m.heads, m.kv_heads, m.dim, m.vdim, m.rot.dims // 2 if m.rot else 0)
    return DeltaShape(m.heads, m.kv_heads, m.dim, m.vdim, m.taps)


def tensor_shapes(cfg: HybridConfig) -> dict[str, tuple]:
    """Every tensor of a checkpoint of this configuration."""
    W, V = cfg.hidden_size, cfg.vocab_size
    out: dict[str, tuple] = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    if cfg.loop is not None:
        out["loop.in"] = (W, 2 * W)
        out["loop.step"] = (cfg.loop.times, W)
    for i, L in enumerate(cfg.layers):
        m, p = L.mixer, f"l{i}.mix."
        rows = {"q": (m.heads if m.kind == "attention" else m.kv_heads) * m.dim,
                "k": m.kv_heads * m.dim,
                "v": (m.kv_heads if m.kind == "attention" else m.heads) * m.vdim}
        out[f"l{i}.norm1"] = (W,)
        for k, n in rows.items():
            out[p + k] = (n, W)
        out[p + "o"] = (W, m.heads * m.vdim)
        if m.kind == "attention":
            if m.gated:
                out[p + "g"] = (m.heads * m.vdim, W)
        else:
            for k, n in rows.items():
                out[p + k + ".conv"] = (n, m.taps)
            out.update({p + "g": (m.heads * m.vdim, W), p + "a": (m.heads, W),
                        p + "b": (m.heads, W), p + "A_log": (m.heads,), p + "dt_bias": (m.heads,),
                        p + "norm": (m.vdim,)})
        if L.mlp is not None:
            out[f"l{i}.mlp.up"] = (L.mlp.ff, W)
            out[f"l{i}.mlp.down"] = (W, L.mlp.ff)
    return out


@dataclass
class LayerWeights:
    norm: torch.Tensor      # [Wp] storage dtype
    norm32: torch.Tensor    # [Wp] f32
    w_in: torch.Tensor      # [n_main (+ n_ab) + ff, Wp]
    w_out: torch.Tensor     # [W, mix_cols + ff_cols]
    n_main: int             # q | k | v | gate rows
    n_ab: int               # delta: a | b rows
    ff: int
    mix_cols: int           # columns of w_out before the feed-forward's
    shape: AttnShape | DeltaShape
    consts: dict            # delta: f32 convolution taps, decay constants, read-out norm

    @property
    def n_raw(self) -> int:
        return self.n_main + self.n_ab

    @property
    def out_cols(self) -> int:
        return self.w_out.shape[1]

    @classmethod
    def load(cls, get: Getter, i: int, cfg: HybridConfig, device, dtype) -> "LayerWeights":
        L, shapes, p = cfg.layers[i], tensor_shapes(cfg), f"l{i}.mix."
        Wp = cfg.width_padded

        def t(name, dt=dtype):
            return _shaped(get, name, shapes[name]).to(device=device, dtype=dt)
        m, sh = L.mixer, mixer_shape(L.mixer)
        main = ["q", "k", "v"] + (["g"] if m.kind == "delta" or m.gated else [])
        ab = ["a", "b"] if m.kind == "delta" else []
        ff = L.mlp.ff if L.mlp is not None else 0
        rows = [t(p + k) for k in main + ab] + ([t(f"l{i}.mlp.up")] if ff else [])
        n_main = sum(r.shape[0] for r in rows[:len(main)])
        n_ab = sum(r.shape[0] for r in rows[len(main):len(main) + len(ab)])
        w_in = torch.zeros((sum(r.shape[0] for r in rows), Wp), device=device, dtype=dtype)
        torch.cat(rows, 0, out=w_in) if Wp == cfg.hidden_size else \
            w_in[:, :cfg.hidden_size].copy_(torch.cat(rows, 0))
        mix_cols = pad_to(sh.out_cols, 8)
        w_out = torch.zeros((cfg.hidden_size, mix_cols + pad_to(ff, 8)), device=device,
                            dtype=dtype)
        w_out[:, :sh.out_cols] = t(p + "o")
        if ff:
            w_out[:, mix_cols:mix_cols + ff] = t(f"l{i}.mlp.down")
        norm32 = torch.zeros(Wp, device=device, dtype=torch.float32)
        norm32[:cfg.hidden_size] = t(f"l{i}.norm1", torch.float32)
        consts = {}
        if m.kind == "delta":
            f32 = torch.float32
            conv = torch.cat([t(p + k + ".conv", f32) for k in ("q", "k", "v")], 0)
            consts = dict(conv=conv.t().contiguous(), a_log=t(p + "A_log", f32).contiguous(),
                          dt_bias=t(p + "dt_bias", f32).contiguous(),
                          norm_w=t(p + "norm", f32).contiguous())
        return cls(norm32.to(dtype), norm32, w_in, w_out, n_main, n_ab, ff, mix_cols, sh, consts)


@dataclass
class ModelWeights:
    """Embedding, final norm, head and the looped section's entry."""
    embed: torch.Tensor           # [V, Wp]
    norm: torch.Tensor
    norm32: torch.Tensor
    lm_head: torch.Tensor         # [V, Wp]
    loop_in: torch.Tensor | None  # [W, 2 W padded to 8]
    loop_step: torch.Tensor | None  # [times, W] f32

    @classmethod
    def load(cls, get: Getter, cfg: HybridConfig, device, dtype) -> "ModelWeights":
        shapes, W, Wp = tensor_shapes(cfg), cfg.hidden_size, cfg.width_padded

        def t(name, dt=dtype):
            return _shaped(get, name, shapes[name]).to(device=device, dtype=dt)

        def padded(name, cols):
            src = t(name)
            out = torch.zeros((src.shape[0], cols), device=device, dtype=dtype)
            out[:, :src.shape[1]] = src
            return out
        norm32 = torch.zeros(Wp, device=device, dtype=torch.float32)
        norm32[:W] = t("final.norm", torch.float32)
        lp = cfg.loop is not None
        return cls(padded("embed", Wp), norm32.to(dtype), norm32, padded("head", Wp),
                   padded("loop.in", pad_to(2 * W, 8)) if lp else None,
                   t("loop.step", torch.float32).contiguous() if lp else None)


def random_tensors(cfg: HybridConfig, device="cpu", dtype=torch.bfloat16, seed: int = 0,
                   gain: float = 1.0) -> Getter:
    """A getter of seeded random tensors (one generator per tensor, so any rank or order of
    loading gives the same values), scaled to keep activations of order one."""
    shapes = tensor_shapes(cfg)
    order = {n: k for k, n in enumerate(shapes)}

    def get(name: str) -> torch.Tensor:
        shape = shapes[name]
        g = torch.Generator(device=device)
        g.manual_seed(seed * 1000003 + order[name])
        t = torch.empty(shape, device=device, dtype=torch.float32)
        leaf = name.rsplit(".", 1)[-1]
        if leaf == "A_log":
            t.uniform_(-4.0, 1.0, generator=g)
        elif leaf == "dt_bias":
            t.uniform_(-3.0, 1.0, generator=g)
        elif leaf == "norm1" or name == "final.norm":
            t.normal_(0.0, 0.1, generator=g)
        elif leaf == "norm":
            t.normal_(1.0, 0.1, generator=g)
        elif leaf == "conv":
            t.normal_(0.0, shape[1] ** -0.5, generator=g)
        elif name == "embed":
            t.normal_(0.0, 1.0, generator=g)
        elif leaf == "step":
            t.normal_(0.0, 0.3, generator=g)
        else:
            t.normal_(0.0, gain * shape[1] ** -0.5, generator=g)
        return t.to(dtype)
    return get


__all__ = ["LayerWeights", "ModelWeights", "mixer_shape", "random_tensors", "tensor_shapes",
           "Layer"]
