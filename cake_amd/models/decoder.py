"""Whole-step hipGraph decoder shared by the text model families.

A model family plugs in through a few hooks (``decode_*`` and ``prefill_logits`` of
:class:`~cake_amd.models.llama3.model.LlamaModel` or
:class:`~cake_amd.models.hybrid.model.HybridModel`); capture, replay by position bucket,
token selection and the token history are the same for all of them.
"""
from __future__ import annotations

import os

import torch


class DeviceDecoder:
    """Whole-step hipGraph decoder for an all-local model on the HIP backend.

    Device state (the model's ``decode_buffers()``): tok, pos, hist, hist_len, slot.  A step:
    embed(tok) → layers(pos) → ln_f/lm_head → [repeat penalty] → token
    selection → finalize (tok ← selected, hist.append, pos += 1).  Selection is
    argmax (greedy) or, with ``sampling`` (temperature > 0), a seeded device draw
    (top-k / top-p threshold + Gumbel-max, sampling.hip) — both inside the graph.
    ``greedy=False`` without ``sampling`` keeps the host-sampler mode: the graph
    stops after the penalty and the caller pushes the token.
    """

    def __init__(self, model, repeat_penalty: float = 1.0, repeat_last_n: int = 128,
                 greedy: bool = True, use_graph: bool = True, steps_per_graph: int = 1,
                 sampling=None):
        if not model.device_decode:
            raise ValueError("DeviceDecoder needs an all-local model on the hip backend")
        self.sampling = sampling if sampling is not None and not sampling.greedy else None
        if self.sampling is not None:
            greedy = True  # token chosen on the device: no host input between steps
        # device-selected decode needs no host input between steps, so several steps
        # can share one graph launch (fewer host round trips); host-sampled mode is 1
        self.k = max(1, int(steps_per_graph)) if greedy and use_graph else 1
        self.m = model
        self.penalty = float(repeat_penalty)
        self.last_n = int(repeat_last_n)
        self.greedy = greedy
        self.use_graph = use_graph
        self.bufs = model.decode_buffers()
        self.params: torch.Tensor | None = None  # device SampleParams (set_sampling)
        self.graph: torch.cuda.CUDAGraph | None = None
        # one graph per attention split cap (position buckets), see capture()
        self.graphs: dict[int, torch.cuda.CUDAGraph] = {}
        self._version = model.decode_version
        self.host_pos = 0  # device position of the next step (tracked on the host)
        self._layers = list(range(model.num_decode_layers))
        # CAKE_FUSED_HEAD=0 keeps the four-launch tail (A/B)
        self._fuse_tail = os.environ.get("CAKE_FUSED_HEAD", "1") != "0"

    # the captured body
    def _step_body(self) -> None:
        from ..ops import hip as K
        b, m = self.bufs, self.m
        fused = self._fused_select()
        if not fused:
            m.decode_embed(b)
        m.decode_layers(b, self._layers)
        if fused:
            # greedy: lm_head + penalty + argmax + finalize + the next step's embedding
            # row in ONE launch (the step's input was embedded by the previous one, or
            # by _select_first)
            m.decode_head_select(b, self.last_n if self.penalty != 1.0 else 0, self.penalty)
            return
        m.decode_head(b)
        if self.penalty != 1.0:
            K.repeat_penalty(b.logits, b.hist, b.hist_len, self.last_n, self.penalty)
        if self.greedy:
            K.select_token(b.logits, b.slot, b.hist, b.hist_len, b.tok, b.pos, self.sampling,
                           b.thr, params=self.params)

    def _fused_select(self) -> bool:
        """Greedy argmax with no device parameter block: the fused head_select tail."""
        from ..ops import hip as K
        return (self.greedy and self.sampling is None and self.params is None
                and (self.penalty == 1.0 or self.last_n <= K.HEAD_SELECT_MAX_LAST_N)
                and self._fuse_tail)

    def set_sampling(self, sampling) -> None:
        """Per-request sampling configuration (None / temperature <= 0 = greedy).  The
        first call switches the selection to a device parameter block (one recapture);
        later calls only rewrite that block, so the captured graph is reused."""
        from ..ops import hip as K
        if self.params is None:
            self.params = torch.zeros(K.SAMPLE_PARAMS_WORDS, dtype=torch.int32,
                                      device=self.m.device)
            self.graph = None
            self.graphs = {}
            self.greedy = True
        self.sampling = sampling if sampling is not None and not sampling.greedy else None
        self.params.copy_(K.pack_sample_params(sampling))

    def profile_layers(self, reps: int = 3) -> list[float]:
        """Per-layer decode kernel time (ms): each layer's five launches
        captured as its own small graph and replayed between timing events, at the
        current device position (the K/V row it writes is the next step's, which that
        step rewrites).  Run between generations (--metrics)."""
        b, m = self.bufs, self.m
        if getattr(self, "_layer_graphs", None) is None:
            m.decode_embed(b)
            torch.cuda.synchronize()
            gs = []
            for li in self._layers:
                g = torch.cuda.CUDAGraph()
                with torch.cuda.graph(g):
                    m.decode_layers(b, [li])
                gs.append(g)
            self._layer_graphs = gs
        m.decode_embed(b)
        state = m.decode_state(b)  # a recurrent layer's replay advances its state
        saved = [t.clone() for t in state]
        out = [0.0] * len(self._layer_graphs)
        for _ in range(reps):
            evs = [torch.cuda.Event(enable_timing=True) for _ in range(len(out) + 1)]
            evs[0].record()
            for i, g in enumerate(self._layer_graphs):
                g.replay()
                evs[i + 1].record()
            evs[-1].synchronize()
            for i in range(len(out)):
                out[i] += evs[i].elapsed_time(evs[i + 1]) / reps
        for t, v in zip(state, saved):
            t.copy_(v)
        return out

    def capture(self) -> None:
        if not self.use_graph or self.graph is not None:
            return
        s = torch.cuda.Stream()
        s.wait_stream(torch.cuda.current_stream())
        # warm the kernels once outside capture on scratch state, then restore
        state = self.m.decode_state(self.bufs)
        saved = [t.clone() for t in state]
        hist = self.bufs.hist.clone()
        with torch.cuda.stream(s):
            self._step_body()
        torch.cuda.current_stream().wait_stream(s)
        torch.cuda.synchronize()
        for t, v in zip(state, saved):
            t.copy_(v)
        self.bufs.hist.copy_(hist)
        self.bufs.slot.zero_()
        # Position buckets: the decode-attention grid is sized by its split cap, and
        # a max_seq-sized grid's idle workgroups cost every layer (8B, max_seq 4096:
        # 353 -> 368 tok/s at short context).  One graph per bucket; launch() replays
        # the smallest that covers the live length.
        self.graphs = {}
        for key, scope in self.m.decode_buckets():
            g = torch.cuda.CUDAGraph()
            with scope(), torch.cuda.graph(g):
                for _ in range(self.k):
                    self._step_body()
            self.graphs[key] = g
        self.graph = self.graphs[max(self.graphs)]
        torch.cuda.synchronize()

    def graph_set(self):
        """The bucket graphs as the native decode loop's GraphSet (built once)."""
        gs = getattr(self, "_graph_set", None)
        if gs is None or gs.graphs[-1] is not self.graphs[max(self.graphs)]:
            from ..ops import graph_loop as GL
            caps = sorted(self.graphs)
            index = {c: i for i, c in enumerate(caps)}
            by_graph = {id(self.graphs[c]): index[c] for c in caps}
            gs = self._graph_set = GL.GraphSet(
                [self.graphs[c] for c in caps], lambda t: by_graph[id(self._graph_for(t))],
                self.m.max_seq)
        return gs

    def _graph_for(self, tk: int) -> torch.cuda.CUDAGraph:
        need = self.m.decode_need(tk)
        for cap in sorted(self.graphs):
            if cap >= need:
                return self.graphs[cap]
        return self.graph

    def start(self, prompt: list[int]) -> int:
        """Prefill `prompt` at position 0 and select the first token (returned)."""
        m, b = self.m, self.bufs
        if m.decode_version != self._version:  # the model's buffers moved: capture again
            self.graph, self.graphs, self._graph_set = None, {}, None
            self._layer_graphs, self._version = None, m.decode_version
        T = len(prompt)
        if T + 1 > m.max_seq:
            raise ValueError("prompt longer than max_seq")
        m.prefill_logits(prompt, b.logits)
        ids = torch.tensor(prompt, dtype=torch.int32)
        b.hist[:T].copy_(ids.to(m.device))
        b.hist_len.fill_(T)
        b.pos.fill_(T - 1)
        b.slot.zero_()
        self.host_pos = T - 1
        return self._select_first()

    def _select_first(self) -> int:
        from ..ops import hip as K
        b = self.bufs
        if self.penalty != 1.0:
            K.repeat_penalty(b.logits, b.hist, b.hist_len, self.last_n, self.penalty)
        if self.greedy:
            K.select_token(b.logits, b.slot, b.hist, b.hist_len, b.tok, b.pos, self.sampling,
                           b.thr, params=self.params)
            if self._fused_select():  # the fused step body starts from the embedded token
                self.m.decode_embed(b)
            self.host_pos += 1
            return int(b.tok.item())
        raise RuntimeError("sampled mode: caller pushes the first token")

    def push(self, token: int) -> None:
        from ..ops import hip as K
        b = self.bufs
        src = torch.tensor([token], dtype=torch.int32, device=self.m.device)
        K.push_token(src, b.tok, b.hist, b.hist_len, b.pos)
        self.host_pos += 1

    def launch(self) -> None:
        """Enqueue `self.k` decode steps (one graph replay; async).  Raises instead of
        writing past the KV cache / token history (max_seq)."""
        if self.host_pos + self.k >= self.m.max_seq:
            raise ValueError(f"decode step at position {self.host_pos} (+{self.k}) overruns "
                             f"max_seq {self.m.max_seq}")
        if self.graph is not None:
            # live length of the last step of this replay (+1: sampled mode pushes)
            self._graph_for(self.host_pos + self.k + 1).replay()
        else:
            with self.m.decode_eager(self.host_pos + self.k - 1):
                self._step_body()
        if self.greedy:  # greedy steps advance pos on the device; sampled ones via push()
            self.host_pos += self.k

    def logits(self) -> torch.Tensor:
        return self.bufs.logits
