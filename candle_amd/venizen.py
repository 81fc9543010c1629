"""The Venizen decoder: pre-norm layers over a f32 residual stream whose mixers and feed-forwards config.json lists layer by layer, with a range of
layers that runs several times on the same weights (each run with its own cache and state), the embedding output added before every run but the first.

Everything that is computed is a call into libcandle_hip_mixer.so; the layers' parts are those of ``mixers.py``.
"""
from __future__ import annotations

import dataclasses
import json
import os
from typing import Callable, Dict, List, Optional, Sequence

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

    @staticmethod
    def from_dict(d: dict, ctx: int = 4096) -> "Config":
        layers = d["layers"]
        n, loop = len(layers), d.get("loop")
        order = [(i, False) for i in range(n)]
        if loop:
            start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
            if not 0 <= start < stop <= n or times < 1:
                raise ValueError(f"loop {loop} does not fit {n} layers")
            again = [(i, i == start) for i in range(start, stop)]
            order = order[:stop] + again * (times - 1) + order[stop:]
        for i, layer in enumerate(layers):
            if layer["type"] not in mixers.MIXERS:
                raise ValueError(f"layer {i}: unknown mixer {layer['type']!r}")
            if layer.get("mlp") and layer["mlp"]["kind"] not in mixers.FEED_FORWARDS:
                raise ValueError(f"layer {i}: unknown feed-forward {layer['mlp']['kind']!r}")
        return Config(vocab=int(d["vocab"]), width=int(d["width"]), eps=float(d["norm"]["eps"]), layers=layers, order=order, ctx=int(ctx))


def tensor_shapes(cfg: Config) -> Dict[str, tuple]:
    """{name: shape} of the checkpoint a configuration describes.  The rank of a delta mixer's decay is the tensors' own choice: a quarter of
    its head size here, at least 16."""
    w = cfg.width
    out = {"embed": (cfg.vocab, w), "final.norm": (w,), "head": (cfg.vocab, w)}
    for i, layer in enumerate(cfg.layers):
        pre, m = f"l{i}.", layer["mixer"]
        out[pre + "norm1"] = (w,)
        if layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            H, G, d, e = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            out.update({pre + "mix.left." + n: s for n, s in (("q", (H * d, w)), ("k", (G * d, w)), ("v", (G * e, w)), ("q.norm", (d,)), ("k.norm", (d,)),
                                                              ("talk", (H, H)), ("o", (w, H * e)))})
            d, e = r["heads"] * r["dim"], r["heads"] * r["vdim"]
            out.update({pre + "mix.right." + n: s for n, s in (("q", (d, w)), ("k", (d, w)), ("v", (e, w)), ("g", (e, w)), ("o", (w, e)))})
        else:
            d, rank = m["heads"] * m["dim"], max(16, m["dim"] // 4)
            out.update({pre + "mix." + n: (d, w) for n in "rkvga"})
            out.update({pre + "mix." + n: s for n, s in (("a.b", (d,)), ("w0", (d,)), ("norm", (d,)), ("w1", (rank, w)), ("w2", (d, rank)), ("o", (w, d)))})
        if layer.get("mlp"):
            ff = layer["mlp"]["ff"]
            out.update({pre + "norm2": (w,), pre + "mlp.up": (ff, w), pre + "mlp.down": (w, ff), pre + "mlp.act": (4,)})
    return out


class Layer:
    def __init__(self, rt: Runtime, cfg: Config, i: int, get: Callable[[str], torch.Tensor]):
        entry, pre = cfg.layers[i], f"l{i}."
        self.norm1 = rt.vector(get(pre + "norm1"))
        self.mixer = mixers.MIXERS[entry["type"]](rt, entry["mixer"], lambda n: get(pre + "mix." + n), cfg.eps)
        self.norm2 = self.mlp = None
        if entry.get("mlp"):
            self.norm2 = rt.vector(get(pre + "norm2"))
            self.mlp = mixers.FEED_FORWARDS[entry["mlp"]["kind"]](rt, entry["mlp"], lambda n: get(pre + "mlp." + n), cfg.eps)


class Model(GreedyDecoder):
    """One sequence on one GPU.  ``forward`` for the logits of the last token, ``step`` for those at chosen places, ``generate_greedy``."""

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
        self.embed = table
        self.layers = [Layer(rt, cfg, i, get) for i in range(len(cfg.layers))]
        self.final_norm = rt.vector(get("final.norm"))
        self.head = Dense(rt, [get("head")])
        self.cache = SequenceCache(self.device)
        self.kept = [self.layers[i].mixer.new_cache(self.cache) for i, _ in cfg.order]
        self.loops = any(again for _, again in cfg.order)
        # single-token steps use the fused matvecs unless an input row is too long for them
        self.fuse_decode = max(d.kp for d in self.denses()) <= mixers.MATVEC_MAX_K
        self.tap: Optional[Callable[[int, torch.Tensor], None]] = None      # tests: residual stream after each layer run of several rows
        self._init_greedy(cfg.ctx)
        self._graph_generation = -1

    # ------------------------------------------------------------------------------------------ construction
    @classmethod
    def from_pretrained(cls, path: str, device="cuda:0", dtype: str = "bfloat16", ctx: int = 4096) -> "Model":
        with open(os.path.join(path, "config.json")) as f:
            cfg = Config.from_dict(json.load(f), ctx)
        return cls(cfg, SafetensorsFile(os.path.join(path, "model.safetensors")).tensor, device, dtype)

    @classmethod
    def random_init(cls, cfg: Config, seed: int = 0, device="cuda:0", dtype: str = "bfloat16") -> "Model":
        """Random weights of the configured shapes, made on the device (benchmarks)."""
        gen = torch.Generator(device=device)
        gen.manual_seed(seed)
        shapes = tensor_shapes(cfg)

        def get(name: str) -> torch.Tensor:
            shape = shapes[name]
            if name.endswith("act"):
                return torch.tensor([0.7, 0.2, 0.1, 0.0], device=device)
            if len(shape) == 1:
                return torch.ones(shape, device=device)
            std = 1.0 if name == "embed" else shape[-1] ** -0.5
            return (torch.randn(shape, generator=gen, device=device) * std).to(torch.bfloat16)
        return cls(cfg, get, device, dtype)

    def denses(self) -> List[Dense]:
        out = [self.head]
        for layer in self.layers:
            out += layer.mixer.denses() + (layer.mlp.denses() if layer.mlp else [])
        return out

    def weight_bytes_per_token(self) -> int:
        """Weight bytes one decode step streams (a layer counts once per run)."""
        per_layer = [sum(d.nbytes() for d in la.mixer.denses() + (la.mlp.denses() if la.mlp else [])) for la in self.layers]
        return sum(per_layer[i] for i, _ in self.cfg.order) + self.head.nbytes()

    # ------------------------------------------------------------------------------------------ kernels of a step
    def _embed(self, ids: int, dst: int, rows: int, sp) -> None:
        check("cq_nn_embedding", self.L.cq_nn_embedding(self.embed.data_ptr(), ids, dst, rows, self.ld, self.cfg.vocab, None, sp))

    def _norm_rows(self, x: int, delta: Optional[int], weight: torch.Tensor, out: int, rows: int, sp, index: Optional[int] = None) -> None:
        check("cq_mix_rms_norm_rows", self.L.cq_mix_rms_norm_rows(x, self.ld, index, delta, self.ld, weight.data_ptr(), out, self.ld, rows, self.cfg.width, self.cfg.eps, sp))

    def _enqueue_rows(self, ids: int, rows: int, pos: int, sp) -> int:
        """`rows` new tokens through all layers; returns the residual stream."""
        rt, ld = self.rt, self.ld
        x, h = rt.scratch("x", rows * ld), rt.scratch("h", rows * ld)
        emb = rt.scratch("embedding", rows * ld) if self.loops else None
        self._embed(ids, x, rows, sp)
        if self.loops:
            self._embed(ids, emb, rows, sp)
        for run, (i, again) in enumerate(self.cfg.order):
            layer = self.layers[i]
            self._norm_rows(x, emb if again else None, layer.norm1, h, rows, sp)
            layer.mixer.prefill(h, ld, x, ld, self.kept[run], pos, rows, sp)
            if layer.mlp:
                self._norm_rows(x, None, layer.norm2, h, rows, sp)
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
        self.head.row(x, dst, sp, mixers.NORM, self.final_norm, self.cfg.eps)

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
                    h = rt.scratch("h", len(at) * self.ld)
                    ldl = pad_to(cfg.vocab, 4)
                    logits = rt.scratch("logits", len(at) * ldl)
                    self._norm_rows(x, None, self.final_norm, h, len(at), sp, index=index.data_ptr())
                    self.head.rows(h, self.ld, logits, ldl, len(at), sp)
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
