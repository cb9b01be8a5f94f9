"""Text model families: config.json -> loader, generator and the kernel libraries it needs.

A family is picked by ``config.json``: one that carries ``architecture`` names a design of
:mod:`.hybrid`; anything else is a Llama checkpoint (HF layout).
"""
from __future__ import annotations

import json
import logging
from dataclasses import dataclass
from pathlib import Path
from typing import Callable

log = logging.getLogger("cake.models")


@dataclass(frozen=True)
class Family:
    name: str
    load_model: Callable      # (model_dir, device, dtype, max_seq) -> model with open_sequence / step
    load_generator: Callable  # (Context) -> TextGenerator
    libs: tuple[str, ...]     # kernel libraries of a step (build.ensure_text)
    distributed: bool         # layers can be placed on workers / ranks


def _llama_model(model_dir, device, dtype, max_seq):
    from .llama3.factory import load_model
    return load_model(model_dir, device, dtype, max_seq=max_seq)


def _llama_generator(ctx):
    """The native engine when it can serve this context (a GPU, 16-bit weights, graphs;
    topology workers through its TCP client), else the Python generator (CPU, f32,
    --no-graph, CAKE_NATIVE=0)."""
    from .llama3.native_generator import NativeLLM, native_eligible
    if native_eligible(ctx):
        topo = getattr(ctx, "topology", None)
        if topo is not None and getattr(topo, "nodes", None):
            log.info("text model on the native engine, TCP workers %s",
                     [f"{n.name}@{n.host}" for n in topo.nodes])
        else:
            log.info("text model on the native engine (libcake_engine.so)")
        return NativeLLM.load(ctx)
    from .llama3.generator import LLamaGenerator
    return LLamaGenerator.load(ctx)


def _hybrid_model(model_dir, device, dtype, max_seq):
    from .hybrid.model import HybridModel
    return HybridModel.load(model_dir, device, dtype, max_seq)


def _hybrid_generator(ctx):
    from .hybrid.generator import HybridGenerator
    return HybridGenerator.load(ctx)


LLAMA = Family("llama3", _llama_model, _llama_generator, ("gemm", "kernels"), True)
HYBRID = Family("hybrid", _hybrid_model, _hybrid_generator, ("gemm", "mixers"), False)


def family_of(model_dir: str | Path) -> Family:
    p = Path(model_dir) / "config.json"
    if not p.exists():
        return LLAMA  # its loader reports what is missing
    d = json.loads(p.read_text())
    if "architecture" not in d:
        return LLAMA
    from .hybrid.config import DESIGNS
    if d["architecture"] not in DESIGNS:
        raise ValueError(f"{p}: unknown architecture {d['architecture']!r} "
                         f"(known: {', '.join(DESIGNS)})")
    return HYBRID


def check_placement(ctx) -> None:
    """Refuse a worker role, a rank group or a topology with workers for a family whose layers
    cannot be placed apart (a looped section visits its layers several times per token)."""
    fam = family_of(ctx.model_path)
    if fam.distributed:
        return
    topo = getattr(ctx, "topology", None)
    if ctx.mode == "worker" or getattr(ctx.args, "transport", "tcp") != "tcp" or \
            (topo is not None and getattr(topo, "nodes", None)):
        raise ValueError(f"{fam.name} models run on one GPU: no workers, no --transport "
                         "rccl / loopback, no topology nodes")
