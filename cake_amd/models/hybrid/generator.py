"""Text generator of the hybrid designs: the framework's generator over a HybridModel.

Prompt template, sampling, repeat penalty, streaming and the captured decode loop are those
of every text model (:class:`~cake_amd.models.llama3.generator.LLamaGenerator`,
:class:`~cake_amd.models.decoder.DeviceDecoder`); 32-bit models decode through the step
function without a graph.
"""
from __future__ import annotations

from ..llama3.generator import LLamaGenerator, load_tokenizer


class HybridGenerator(LLamaGenerator):
    MODEL_NAME = "hybrid"

    @classmethod
    def load(cls, ctx) -> "HybridGenerator":
        from .model import HybridModel
        model = HybridModel.load(ctx.model_path, ctx.device, ctx.dtype, ctx.max_seq_len)
        tok, eos = load_tokenizer(ctx.model_path, model.cfg.eos_token_id)
        gen = cls(model, tok, eos, ctx.sampling, use_graph=not ctx.no_graph)
        gen.MODEL_NAME = model.cfg.name
        return gen
