"""Greedy generation for decoders whose single-token step runs from device state (token, position, history), so that it can
be captured in a HIP graph once and replayed."""
from __future__ import annotations

import time
from typing import List, Optional, Sequence

import torch

from . import _lib


class GreedyDecoder:
    """Mixin.  The model provides ``cfg.ctx``, ``cfg.vocab``, ``device``, ``L``, ``forward`` and ``_decode_step_dev``; the hooks below may be
    overridden."""

    def _init_greedy(self, ctx: int) -> None:
        i32 = dict(dtype=torch.int32, device=self.device)
        self.token_dev = torch.zeros(1, **i32)
        self.pos_dev = torch.zeros(1, **i32)
        self.counter_dev = torch.zeros(1, **i32)
        self.history_dev = torch.zeros(ctx, **i32)
        self.argmax_ws = torch.zeros(1024, dtype=torch.uint8, device=self.device)      # CQ_NN_ARGMAX_WORKSPACE
        self._graph = None
        self._graph_key = None

    def _chain_embedding(self, max_kv_len: int) -> bool:
        """Whether a step starts from an embedding row that the previous arg-max left in place."""
        return False

    def _argmax_dev(self, logits_ptr: int, embed: bool, sp) -> None:
        """Sampling::ArgMax into token_dev / history_dev, the position advanced."""
        _lib.check("cq_nn_argmax", self.L.cq_nn_argmax(logits_ptr, self.cfg.vocab, self.token_dev.data_ptr(), self.history_dev.data_ptr(),
                                                      self.counter_dev.data_ptr(), self.pos_dev.data_ptr(), self.argmax_ws.data_ptr(), sp))

    def _step_state(self) -> List[torch.Tensor]:
        """Everything a step changes and the next one reads (the warm-up before a capture runs a step and puts it back)."""
        return [self.token_dev, self.pos_dev, self.counter_dev]

    def _graph_key_for(self, max_kv: int):
        return max_kv

    def _steps_done(self, prompt: int, steps: int) -> None:
        """The decode steps of a generation have been enqueued."""

    def _steps_failed(self) -> bool:
        """Whether the steps of a generation have to be run again another way (which the model has switched to)."""
        return False

    def generate_greedy(self, prompt: Sequence[int], n_new: int, use_graph: bool = True, max_kv: Optional[int] = None) -> dict:
        """The loop of candle-examples/examples/quantized/main.rs:616-690 with temperature <= 0 (Sampling::ArgMax):
        prefill the prompt in one forward, pick the arg-max token, then n_new - 1 single-token steps.
        Returns the generated tokens and the wall-clock split prompt / decode, as the example prints them.
        max_kv: the number of cache positions the captured step is laid out for (its attention split count follows from
        it); by default exactly prompt + n_new, a server that captures one step for every request passes the context."""
        cfg = self.cfg
        prompt = [int(t) for t in prompt]
        if len(prompt) + n_new > cfg.ctx:
            raise ValueError("prompt + generated tokens exceed the context")
        if max_kv is not None and not len(prompt) + n_new <= max_kv <= cfg.ctx:
            raise ValueError("max_kv must cover prompt + generated tokens and fit the context")
        dev = self.device
        torch.cuda.synchronize(dev)
        t0 = time.perf_counter()
        logits = self.forward(torch.tensor([prompt], dtype=torch.int32, device=dev), 0)
        stream = torch.cuda.current_stream(dev)
        self.counter_dev.zero_()
        self.pos_dev.fill_(len(prompt) - 1)       # argmax advances it to the position of the token it emits
        steps = n_new - 1
        if max_kv is None:
            max_kv = len(prompt) + n_new
        self._argmax_dev(logits.data_ptr(), steps > 0 and self._chain_embedding(max_kv), stream.cuda_stream)
        torch.cuda.synchronize(dev)
        t1 = time.perf_counter()
        prompt_seconds = t1 - t0
        if steps > 0:
            if use_graph:
                key = self._graph_key_for(max_kv)
                if self._graph is None or self._graph_key != key:
                    side = torch.cuda.Stream(device=dev)
                    # capture must not disturb the live decode state: save and restore it around the warm-up run
                    state = self._step_state()
                    saved = [t.clone() for t in state]
                    torch.cuda.synchronize(dev)
                    with torch.cuda.stream(side):
                        self._decode_step_dev(max_kv, side.cuda_stream)
                        side.synchronize()
                        g = torch.cuda.CUDAGraph()
                        with torch.cuda.graph(g, stream=side):
                            self._decode_step_dev(max_kv, torch.cuda.current_stream(dev).cuda_stream)
                    torch.cuda.synchronize(dev)
                    for t, s in zip(state, saved):
                        t.copy_(s)
                    torch.cuda.synchronize(dev)
                    self._graph, self._graph_key = g, key
                t1 = time.perf_counter()
                for _ in range(steps):
                    self._graph.replay()
            else:
                for _ in range(steps):
                    self._decode_step_dev(max_kv, stream.cuda_stream)
        torch.cuda.synchronize(dev)
        t2 = time.perf_counter()
        if self._steps_failed():
            return self.generate_greedy(prompt, n_new, use_graph)
        self._steps_done(len(prompt), max(steps, 0))
        tokens = self.history_dev[:n_new].cpu().tolist()
        return {"tokens": tokens, "prompt_seconds": prompt_seconds, "decode_seconds": t2 - t1, "decode_steps": steps}
