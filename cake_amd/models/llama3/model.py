"""Master-side Llama-3 model: embedding → placed blocks → ln_f → lm_head.

Counterpart of ``LLama::forward`` (cake-core/src/models/llama3/llama.rs:72-138).
Blocks are placed per the topology: a layer named on a worker is reached
through a remote :class:`~cake_amd.parallel.forwarder.Forwarder`; every other
layer runs in this process's :class:`LayerStack`.  Consecutive layers with the
same owner form one *run* and cost one hop (contiguous-block batching,
llama.rs:95-114) — planned once at load time by :func:`plan_runs`.

For the all-local HIP case, :class:`~cake_amd.models.decoder.DeviceDecoder` captures the whole decode
step (embedding, 32/80 layers, ln_f + lm_head, repeat penalty, argmax, next
token/position bookkeeping) into ONE hipGraph; the host reads 4 bytes per token,
one step behind the GPU.
"""
from __future__ import annotations

from dataclasses import dataclass
from functools import partial

import torch

from ...ops import reference as R
from ..base import StepEntry
from ..decoder import DeviceDecoder  # noqa: F401  (the all-local decoder of this family)
from .blocks import DecodeBuffers, LayerStack
from .config import LlamaConfig
from .weights import HeadWeights, layer_name


@dataclass
class Run:
    ident: str                 # "local" or the worker identity
    layers: list[int]
    forwarder: object | None = None   # parallel.forwarder.Forwarder for remote runs

    @property
    def local(self) -> bool:
        return self.ident == "local"


def plan_runs(num_layers: int, remote: dict[int, object]) -> list[Run]:
    """Group consecutive layers with equal owner identity (llama.rs:95-114)."""
    runs: list[Run] = []
    for li in range(num_layers):
        fwd = remote.get(li)
        ident = "local" if fwd is None else fwd.ident()
        if runs and runs[-1].ident == ident:
            runs[-1].layers.append(li)
        else:
            runs.append(Run(ident=ident, layers=[li], forwarder=fwd))
    return runs


class LlamaModel:
    def __init__(self, cfg: LlamaConfig, head: HeadWeights, stack: LayerStack,
                 remote: dict[int, object] | None = None):
        self.cfg = cfg
        self.head = head
        self.stack = stack
        self.remote = dict(remote or {})
        self.runs = plan_runs(cfg.num_hidden_layers, self.remote)
        missing = [li for r in self.runs if r.local for li in r.layers if li not in stack.weights]
        if missing:
            raise ValueError(f"local layers without weights: {missing[:8]}")
        self.device = stack.device
        self.dtype = stack.dtype
        self.backend = stack.backend
        self.session = 0
        self._seq_pos: dict[int, int] = {}  # open sequences (step) -> tokens fed

    @property
    def all_local(self) -> bool:
        return all(r.local for r in self.runs)

    # ------------------------------------------------------------------ generic path
    def embed(self, tokens: list[int]) -> torch.Tensor:
        ids = torch.tensor(tokens, dtype=torch.int32, device=self.device)
        if self.backend == "hip":
            from ...ops import hip as K
            out = torch.empty((len(tokens), self.cfg.hidden_size), device=self.device,
                              dtype=torch.float32)
            K.embed(self.head.embed, ids, out)
            return out
        return self.head.embed[ids.long()].float()

    def forward_hidden(self, hidden: torch.Tensor, pos0: int) -> torch.Tensor:
        for run in self.runs:
            if run.local:
                self.stack.forward(hidden, run.layers, pos0, self.session)
            else:
                batch = [(layer_name(li), pos0, li) for li in run.layers]
                hidden = run.forwarder.forward_batch(hidden, batch, self.session)
                if hidden.device != self.device:
                    hidden = hidden.to(self.device)
                hidden = hidden.float().contiguous()
        return hidden

    def head_logits(self, last: torch.Tensor, out: torch.Tensor | None = None) -> torch.Tensor:
        """ln_f + lm_head on one f32 row -> f32 logits (llama.rs:119-137)."""
        if self.backend == "hip":
            from ...ops import hip as K
            if out is None:
                out = torch.empty(self.cfg.vocab_size, device=self.device, dtype=torch.float32)
            K.norm_gemv_f32(last.contiguous(), self.head.norm, self.cfg.rms_norm_eps,
                            self.head.lm_head, out)
            return out
        x = R.rms_norm(last, self.head.norm, self.cfg.rms_norm_eps).to(self.dtype)
        return (x @ self.head.lm_head.t()).float()

    def forward(self, tokens: list[int], pos0: int) -> torch.Tensor:
        """Logits (f32 [V]) of the last of `tokens`, fed at positions pos0.."""
        h = self.embed(tokens)
        h = self.forward_hidden(h, pos0)
        return self.head_logits(h[-1])

    def reset(self) -> None:
        self.stack.reset(self.session)
        for run in self.runs:
            if not run.local and hasattr(run.forwarder, "reset"):
                run.forwarder.reset(self.session)

    # ------------------------------------------------------------------ decode hooks
    # (DeviceDecoder, models/decoder.py)
    @property
    def max_seq(self) -> int:
        return self.stack.max_seq

    @property
    def device_decode(self) -> bool:
        return self.backend == "hip" and self.all_local

    @property
    def decode_version(self) -> int:
        return 0

    @property
    def num_decode_layers(self) -> int:
        return self.cfg.num_hidden_layers

    def decode_buffers(self) -> DecodeBuffers:
        return self.stack.decode_buffers(with_head=True)

    def decode_state(self, b: DecodeBuffers) -> list[torch.Tensor]:
        """What a step changes besides the KV rows and the token history."""
        return [b.tok, b.pos, b.hist_len, b.resid]

    def decode_embed(self, b: DecodeBuffers) -> None:
        from ...ops import hip as K
        K.embed(self.head.embed, b.tok, b.resid)

    def decode_layers(self, b: DecodeBuffers, layers: list[int]) -> None:
        self.stack.decode_step(b, layers, self.session)

    def decode_head(self, b: DecodeBuffers) -> None:
        from ...ops import hip as K
        K.norm_gemv_f32(b.resid, self.head.norm, self.cfg.rms_norm_eps, self.head.lm_head,
                        b.logits)

    def decode_head_select(self, b: DecodeBuffers, last_n: int, penalty: float) -> None:
        from ...ops import hip as K
        K.head_select(b.resid, self.head.norm, self.cfg.rms_norm_eps, self.head.lm_head, b.logits,
                      b.hist, b.hist_len, last_n, penalty, b.slot, b.sel_ticket, b.tok, b.pos,
                      embed=self.head.embed)

    def decode_buckets(self) -> list:
        """(key, context factory) of the graphs that cover every live length: the key is
        compared with :meth:`decode_need`."""
        from ...ops import hip as K
        out = [(cap, partial(K.attn_split_cap, cap)) for cap in K.attn_split_caps(self.max_seq)]
        # bucket "1 split": attention and o_proj as one launch per layer (attn_oproj.hip),
        # for the live lengths whose attention is a single split
        if self.stack.attn_oproj_ok() and not self.stack.mk_enabled():
            out.append((1, K.attn_oproj_fused))
        return out

    def decode_need(self, tk: int) -> int:
        from ...ops import hip as K
        return K.attn_splits(tk)

    def decode_eager(self, pos: int):
        """Context of an ungraphed step at device position `pos`."""
        from ...ops import hip as K
        return K.attn_oproj_fused(K.attn_oproj_short(pos))

    def decode_check(self, b: DecodeBuffers) -> None:
        if self.backend == "hip":
            self.stack.mk_check(b)

    def prefill_logits(self, prompt: list[int], out: torch.Tensor) -> None:
        """The whole prompt from position 0; logits of its last token into `out`."""
        self.stack.reset(self.session)
        h = self.forward_hidden(self.embed(prompt), 0)
        self.head_logits(h[-1], out=out)

    # ------------------------------------------------------------------ ragged steps
    def open_sequence(self) -> int:
        """A new sequence for :meth:`step` (its own KV cache)."""
        used = self._seq_pos
        sid = next(i for i in range(1, len(used) + 2) if i not in used)
        self.stack.max_sessions = max(self.stack.max_sessions, len(used) + 2)
        used[sid] = 0
        return sid

    def close_sequence(self, sid: int) -> None:
        del self._seq_pos[sid]
        self.stack.drop(sid)

    def step(self, entries: list[StepEntry]) -> list[torch.Tensor]:
        """Feed each sequence its next tokens; logits [len(want), V] per entry.  The Llama
        kernels hold one sequence at a time, so the entries run one after another."""
        out = []
        for e in entries:
            pos = self._seq_pos[e.seq]
            keep, self.session = self.session, e.seq
            try:
                h = self.forward_hidden(self.embed(e.tokens), pos)
            finally:
                self.session = keep
            self._seq_pos[e.seq] = pos + len(e.tokens)
            rows = [self.head_logits(h[w]).clone() for w in e.want]
            out.append(torch.stack(rows) if rows else h.new_zeros((0, self.cfg.vocab_size)))
        return out
