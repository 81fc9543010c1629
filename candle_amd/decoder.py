"""Decoders made of the parts in ``mixers.py``: pre-norm layers over a f32 residual stream whose mixers and feed-forwards config.json lists layer by layer.
A design is a subclass of ``Decoder`` that names its norm and which class each configured mixer and feed-forward means; layers may run more than
once, and a layer may attend to the cache of an earlier one.

Everything that is computed is a call into libcandle_hip_mixer.so.
"""
from __future__ import annotations

import dataclasses
import json
import os
from typing import Callable, ClassVar, Dict, List, Optional, Sequence

import torch

from . import mixers
from ._lib import check
from .cache import SequenceCache
from .generation import GreedyDecoder
from .mixers import Dense, Runtime, pad_to
from .safetensors_file import SafetensorsFile

DTYPES = {"bfloat16": mixers.BF16, "float32": mixers.F32}


@dataclasses.dataclass
class Config:
    vocab: int
    width: int
    eps: float
    layers: List[dict]                # per layer: type, mixer (its sizes and constants), mlp (or None)
    order: List[tuple]                # layer runs: (layer, whether the embedding output is added before it)
    ctx: int = 4096
    embed_scale: float = 1.0          # factor on the embedding output

    # what the entries of a design mean; a design's configuration sets its own
    MIXERS: ClassVar[Dict[str, type]] = {}
    FEED_FORWARDS: ClassVar[Dict[str, type]] = {}

    @classmethod
    def from_dict(cls, d: dict, ctx: int = 4096) -> "Config":
        layers = d["layers"]
        for i, layer in enumerate(layers):
            if layer["type"] not in cls.MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if layer.get("mlp") and layer["mlp"]["kind"] not in cls.FEED_FORWARDS:
                raise ValueError(f"layer {i}: unknown feed-forward {layer['mlp']['kind']!r}")
        return cls(vocab=int(d["vocab"]), width=int(d["width"]), eps=float(d["norm"]["eps"]), layers=layers, order=cls.layer_runs(d), ctx=int(ctx),
                   embed_scale=float(d.get("embedding", {}).get("scale", 1.0)))

    @classmethod
    def layer_runs(cls, d: dict) -> List[tuple]:
        return [(i, False) for i in range(len(d["layers"]))]


class Layer:
    def __init__(self, rt: Runtime, cfg: Config, norm: type, i: int, get: Callable[[str], torch.Tensor]):
        entry, pre = cfg.layers[i], f"l{i}."
        self.norm1 = norm(rt, get, pre + "norm1", cfg.eps)
        self.mixer = cfg.MIXERS[entry["type"]](rt, entry["mixer"], lambda n: get(pre + "mix." + n), cfg.eps)
        self.norm2 = self.mlp = None
        if entry.get("mlp"):
            self.norm2 = norm(rt, get, pre + "norm2", cfg.eps)
            self.mlp = cfg.FEED_FORWARDS[entry["mlp"]["kind"]](rt, entry["mlp"], lambda n: get(pre + "mlp." + n), cfg.eps)


    def parts(self) -> list:
        return [self.mixer] + ([self.mlp] if self.mlp else [])


def token_bytes(part) -> int:
    """Weight bytes that a single-token step of a mixer or feed-forward streams: all of its matrices, unless it says otherwise."""
    return part.token_bytes() if hasattr(part, "token_bytes") else sum(d.nbytes() for d in part.denses())


class Decoder(GreedyDecoder):
    """One sequence on one GPU.  ``forward`` for the logits of the last token, ``step`` for those at chosen places, ``generate_greedy``."""

    CONFIG = Config
    NORM: type = mixers.RmsNorm
    MAX_ROWS = 4096                   # tokens per pass; longer calls run as several

    def __init__(self, cfg: Config, get: Callable[[str], torch.Tensor], device="cuda:0", dtype: str = "bfloat16"):
        if dtype not in DTYPES:
            raise ValueError(f"dtype {dtype!r}: expected one of {sorted(DTYPES)}")
        self.cfg, self.device = cfg, torch.device(device)
        self.rt = rt = Runtime(device, DTYPES[dtype], cfg.ctx)
        self.L = rt.L
        self.ld = pad_to(cfg.width, 64)               # row stride of the residual stream
        table = torch.zeros((cfg.vocab, self.ld), dtype=torch.float32, device=self.device)
        table[:, :cfg.width] = get("embed").to(self.device)
        if cfg.embed_scale != 1.0:
            table *= cfg.embed_scale
        self.embed = table
        self.layers = [Layer(rt, cfg, self.NORM, i, get) for i in range(len(cfg.layers))]
        self.final_norm = self.NORM(rt, get, "final.norm", cfg.eps)
        self.head = Dense(rt, [get("head")])
        self.cache = SequenceCache(self.device)
        self.kept, of_layer = [], {}                  # per layer run; of the last run of each layer
        for i, _ in cfg.order:
            source = self.layers[i].mixer.kv_from
            if source is not None and source not in of_layer:
                raise ValueError(f"layer {i} attends to the cache of layer {source}, which has not run before it")
            of_layer[i] = self.layers[i].mixer.new_cache(self.cache) if source is None else of_layer[source]
            self.kept.append(of_layer[i])
        self.loops = any(again for _, again in cfg.order)
        # single-token steps use the fused matvecs unless an input row is too long for them
        self.fuse_decode = max(d.kp for d in self.denses()) <= mixers.MATVEC_MAX_K
        self.tap: Optional[Callable[[int, torch.Tensor], None]] = None      # tests: residual stream after each layer run of several rows
        self._init_greedy(cfg.ctx)
        self._graph_generation = -1

    # ------------------------------------------------------------------------------------------ construction
    @classmethod
    def from_pretrained(cls, path: str, device="cuda:0", dtype: str = "bfloat16", ctx: int = 4096) -> "Decoder":
        with open(os.path.join(path, "config.json")) as f:
            cfg = cls.CONFIG.from_dict(json.load(f), ctx)
        return cls(cfg, SafetensorsFile(os.path.join(path, "model.safetensors")).tensor, device, dtype)

    @staticmethod
    def tensor_shapes(cfg: Config) -> Dict[str, tuple]:
        """{name: shape} of the checkpoint a configuration describes."""
        raise NotImplementedError

    @classmethod
    def random_vector(cls, name: str, n: int) -> torch.Tensor:
        """A one-dimensional tensor of a random model."""
        return torch.ones(n)

    @classmethod
    def random_init(cls, cfg: Config, seed: int = 0, device="cuda:0", dtype: str = "bfloat16") -> "Decoder":
        """Random weights of the configured shapes, made on the device (benchmarks)."""
        gen = torch.Generator(device=device)
        gen.manual_seed(seed)
        shapes = cls.tensor_shapes(cfg)

        def get(name: str) -> torch.Tensor:
            shape = shapes[name]
            if len(shape) == 1:
                return cls.random_vector(name, shape[0]).to(device)
            std = 1.0 if name == "embed" else shape[-1] ** -0.5
            return (torch.randn(shape, generator=gen, device=device) * std).to(torch.bfloat16)
        return cls(cfg, get, device, dtype)

    def denses(self) -> List[Dense]:
        out = [self.head]
        for layer in self.layers:
            out += [d for part in layer.parts() for d in part.denses()]
        return out

    def weight_bytes_per_token(self) -> int:
        """Weight bytes one decode step streams (a layer counts once per run)."""
        per_layer = [sum(token_bytes(part) for part in la.parts()) for la in self.layers]
        return sum(per_layer[i] for i, _ in self.cfg.order) + self.head.nbytes()

    # ------------------------------------------------------------------------------------------ kernels of a step
    def _embed(self, ids: int, dst: int, rows: int, sp) -> None:
        check("cq_nn_embedding", self.L.cq_nn_embedding(self.embed.data_ptr(), ids, dst, rows, self.ld, self.cfg.vocab, None, sp))

    def _enqueue_rows(self, ids: int, rows: int, pos: int, sp) -> int:
        """`rows` new tokens through all layers; returns the residual stream."""
        rt, ld = self.rt, self.ld
        x = rt.scratch("x", rows * ld)
        emb = rt.scratch("embedding", rows * ld) if self.loops else None
        self._embed(ids, x, rows, sp)
        if self.loops:
            self._embed(ids, emb, rows, sp)
        for run, (i, again) in enumerate(self.cfg.order):
            layer = self.layers[i]
            h = rt.normed(layer.mixer.INPUT, rows * ld)
            layer.norm1.rows(x, ld, h, ld, rows, sp, delta=emb if again else None)
            layer.mixer.prefill(h, ld, x, ld, self.kept[run], pos, rows, sp)
            if layer.mlp:
                h = rt.normed(layer.mlp.INPUT, rows * ld)
                layer.norm2.rows(x, ld, h, ld, rows, sp)
                layer.mlp.prefill(h, ld, x, ld, rows, sp)
            if self.tap:
                self.tap(run, rt._scratch["x"][:rows * ld].view(rows, ld)[:, :self.cfg.width])
        return x

    def _enqueue_token(self, ids: int, pos_dev: Optional[int], pos: int, sp) -> int:
        """One new token, its position in device memory if pos_dev is given (then a step may be captured); returns the residual row."""
        rt, order = self.rt, self.cfg.order
        x = rt.scratch("x", self.ld)
        emb = rt.scratch("embedding", self.ld) if self.loops else None
        self._embed(ids, x, 1, sp)
        if self.loops:
            self._embed(ids, emb, 1, sp)
        for run, (i, _) in enumerate(order):
            layer = self.layers[i]
            # the last matvec of a pass over the repeated layers also adds the embedding output for the next pass
            add = emb if run + 1 < len(order) and order[run + 1][1] else None
            layer.mixer.step(x, layer.norm1, self.kept[run], pos_dev, pos, None if layer.mlp else add, sp)
            if layer.mlp:
                layer.mlp.step(x, layer.norm2, add, sp)
        return x

    def _logits_row(self, x: int, dst: int, sp) -> None:
        self.head.row(x, dst, sp, self.final_norm.prologue, self.final_norm.vec, self.final_norm.eps)

    # ------------------------------------------------------------------------------------------ public steps
    def step(self, tokens: Sequence[int], want: Sequence[int], pos: Optional[int] = None) -> torch.Tensor:
        """Runs the next tokens of the sequence (from position `pos`, by default where the last call ended) and returns the logits
        [len(want), vocab] at the given places among them."""
        cfg, rt = self.cfg, self.rt
        n = len(tokens)
        pos = self.cache.length if pos is None else pos
        want = [int(w) for w in want]
        if n == 0 or pos < 0 or pos + n > cfg.ctx:
            raise ValueError(f"positions {pos}..{pos + n} outside the context of {cfg.ctx}")
        if any(not 0 <= w < n for w in want):
            raise ValueError("a wanted place outside the step's tokens")
        ids_host = torch.as_tensor(tokens, dtype=torch.int32).reshape(-1)
        if int(ids_host.min()) < 0 or int(ids_host.max()) >= cfg.vocab:
            raise ValueError(f"token ids must be in [0, {cfg.vocab})")
        self.cache.begin(pos)
        ids = ids_host.to(self.device)
        sp = torch.cuda.current_stream(self.device).cuda_stream
        out = torch.empty((len(want), cfg.vocab), dtype=torch.float32, device=self.device)
        for lo in range(0, n, self.MAX_ROWS):
            rows = min(self.MAX_ROWS, n - lo)
            at = [j for j, w in enumerate(want) if lo <= w < lo + rows]
            if rows == 1 and self.fuse_decode:
                x = self._enqueue_token(ids.data_ptr() + 4 * lo, None, pos + lo, sp)
                for j in at:
                    self._logits_row(x, out[j].data_ptr(), sp)
            else:
                x = self._enqueue_rows(ids.data_ptr() + 4 * lo, rows, pos + lo, sp)
                if at:
                    index = torch.tensor([want[j] - lo for j in at], dtype=torch.int32).to(self.device)
                    h = rt.normed(mixers.AS_F32, len(at) * self.ld)
                    ldl = pad_to(cfg.vocab, 4)
                    logits = rt.scratch("logits", len(at) * ldl)
                    self.final_norm.rows(x, self.ld, h, self.ld, len(at), sp, index=index.data_ptr())
                    self.head.rows(h.f32, self.ld, logits, ldl, len(at), sp)
                    out[at] = rt._scratch["logits"][:len(at) * ldl].view(len(at), ldl)[:, :cfg.vocab]
        self.cache.length = pos + n
        return out

    def forward(self, x: torch.Tensor, index_pos: int) -> torch.Tensor:
        """Token ids [1, seq_len] at positions index_pos.. -> logits [1, vocab] of the last token."""
        if x.dim() != 2 or x.shape[0] != 1:
            raise ValueError(f"expected token ids of shape (1, seq_len), got {tuple(x.shape)}")
        return self.step(x[0].cpu(), [x.shape[1] - 1], index_pos)

    def reset(self) -> None:
        """Give the sequence back; the next call starts at position 0."""
        self.cache.reset()

    # ------------------------------------------------------------------------------------------ greedy decode (generation.py)
    def _decode_step_dev(self, max_kv_len: int, sp) -> None:
        rt = self.rt
        logits = rt.scratch("logits", pad_to(self.cfg.vocab, 4))
        if self.fuse_decode:
            x = self._enqueue_token(self.token_dev.data_ptr(), self.pos_dev.data_ptr(), 0, sp)
            self._logits_row(x, logits, sp)
        else:
            raise RuntimeError(f"input rows longer than {mixers.MATVEC_MAX_K} have no single-token step from device state")
        self._argmax_dev(logits, False, sp)

    def _step_state(self) -> List[torch.Tensor]:
        return super()._step_state() + self.cache.states

    def _graph_key_for(self, max_kv: int):
        return self.rt.generation                     # the launches are laid out for the whole context; buffers must be the captured ones

    def _steps_done(self, prompt: int, steps: int) -> None:
        self.cache.length = prompt + steps
