"""Building blocks of decoders with bfloat16 weights, over include/candle_hip_mixer.h: dense layers, sequence mixers and
feed-forwards.  A block takes its sizes and constants from its configuration entry, registers what it keeps of a sequence
with the SequenceCache once per run of its layer, and enqueues its kernels for several rows (``prefill``) or for one row whose position
lives in device memory (``step``).  PyTorch only provides memory and the stream.

Several rows: norm -> one product for all projections of a mixer -> head packing (norm, rotation, cache append) -> the mixer's
kernels -> one product back to the residual stream.  One row: the norm is the prologue of the projection matvec, the residual add the
epilogue of the last one, and the state kernels do their packing and gating themselves.
"""
from __future__ import annotations

import ctypes
import math
from typing import Callable, Dict, List, Optional

import numpy as np
import torch

from . import _lib
from ._lib import MixHeads
from .cache import SequenceCache

BF16, F32 = 0, 1                                     # enum cq_dense_precision
PLAIN, NORM, POLY = 0, 1, 2                          # enum cq_dense_prologue
SILU, SIGMOID = 0, 1                                 # enum cq_gate
MATVEC_MAX_K = 32768                                 # CQ_DENSE_MATVEC_MAX_K

check = _lib.check


def pad_to(n: int, m: int) -> int:
    return (n + m - 1) // m * m


class Runtime:
    """What the blocks of one model share: the library, device, product precision, rotation tables and grow-only scratch buffers.

    Scratch is zeroed when it is allocated and only ever holds finite values, so the padding of rows (which meets zero weights) never
    produces a NaN."""

    def __init__(self, device, precision: int, ctx: int):
        self.L = _lib.mixer_lib()
        self.device = torch.device(device)
        self.precision = precision
        self.ctx = ctx
        self.generation = 0                          # counts reallocations: a captured step holds the old addresses
        self._scratch: Dict[str, torch.Tensor] = {}
        self._tables: Dict[tuple, tuple] = {}

    def scratch(self, name: str, floats: int) -> int:
        """Address of the scratch buffer ``name`` with room for ``floats`` f32."""
        t = self._scratch.get(name)
        if t is None or t.numel() < floats:
            if torch.cuda.is_current_stream_capturing():
                raise RuntimeError(f"scratch buffer {name} would have to grow while a step is being captured")
            if t is not None:
                torch.cuda.synchronize(self.device)
            t = torch.zeros(pad_to(max(floats, 1), 64), dtype=torch.float32, device=self.device)
            self._scratch[name] = t
            self.generation += 1
        return t.data_ptr()

    def rotation(self, base: float, dims: int) -> tuple:
        """cos / sin [ctx, dims / 2] of t * base^(-2 i / dims), evaluated in double and rounded once."""
        key = (float(base), int(dims))
        if key not in self._tables:
            ang = np.arange(self.ctx, dtype=np.float64)[:, None] * np.float64(base) ** (-2.0 * np.arange(dims // 2, dtype=np.float64) / dims)
            self._tables[key] = tuple(torch.from_numpy(f(ang).astype(np.float32)).to(self.device) for f in (np.cos, np.sin))
        return self._tables[key]

    def vector(self, t: torch.Tensor) -> torch.Tensor:
        return t.to(device=self.device, dtype=torch.float32).contiguous()


class Dense:
    """One or several weights [out, in] stacked along `out` (they read the same input) or along `in` (their inputs are concatenated),
    rows padded with zeros to a multiple of 64."""

    def __init__(self, rt: Runtime, weights: List[torch.Tensor], along: str = "out"):
        for w in weights:
            if w.dtype != torch.bfloat16 or w.dim() != 2:
                raise ValueError(f"expected bfloat16 matrices, got {w.dtype} {tuple(w.shape)}")
        self.rt = rt
        self.n = sum(w.shape[0] for w in weights) if along == "out" else weights[0].shape[0]
        self.k = weights[0].shape[1] if along == "out" else sum(w.shape[1] for w in weights)
        self.kp = pad_to(self.k, 64)
        self.w = torch.zeros((self.n, self.kp), dtype=torch.bfloat16, device=rt.device)
        at = 0
        for w in weights:
            if along == "out":
                if w.shape[1] != self.k:
                    raise ValueError("stacked weights must read the same input")
                self.w[at:at + w.shape[0], :self.k] = w.to(rt.device)
                at += w.shape[0]
            else:
                if w.shape[0] != self.n:
                    raise ValueError("weights side by side must write the same output")
                self.w[:, at:at + w.shape[1]] = w.to(rt.device)
                at += w.shape[1]

    def nbytes(self) -> int:
        return self.w.numel() * 2

    def rows(self, x: int, ldx: int, dst: int, ldd: int, rows: int, sp, accumulate: bool = False) -> None:
        rt = self.rt
        need = rt.L.cq_dense_matmul_workspace_bytes(rt.precision, rows, self.n, self.kp)
        ws = rt.scratch("dense_planes", need // 4) if need else None
        check("cq_dense_matmul", rt.L.cq_dense_matmul(rt.precision, self.w.data_ptr(), self.kp, x, ldx, dst, ldd, None, 0, int(accumulate), rows, self.n, self.kp,
                                                      ws, need, sp))

    def row(self, x: int, dst: int, sp, prologue: int = PLAIN, vec: Optional[torch.Tensor] = None, eps: float = 0.0, accumulate: bool = False,
            add: Optional[int] = None) -> None:
        check("cq_dense_matvec", self.rt.L.cq_dense_matvec(self.w.data_ptr(), self.kp, x, prologue, vec.data_ptr() if vec is not None else None, eps, self.k, dst,
                                                          add, int(accumulate), self.n, self.kp, sp))


def _heads(src_off: int, heads: int, dim: int, *, dim_pad: int = 0, dst: Optional[int] = None, row_stride: int = 0, head_stride: int = 0,
           norm: Optional[torch.Tensor] = None, tables: Optional[tuple] = None, rot_dims: int = 0, by_position: bool = False, ctx: int = 0,
           factor: float = 1.0) -> MixHeads:
    return MixHeads(norm.data_ptr() if norm is not None else None, tables[0].data_ptr() if tables else None, tables[1].data_ptr() if tables else None,
                    dst, src_off, row_stride, head_stride, heads, dim, dim_pad or dim, rot_dims, int(by_position), ctx, factor, 0)


def _group_array(groups: List[MixHeads]):
    return (MixHeads * len(groups))(*groups)


class Rotation:
    def __init__(self, rt: Runtime, cfg: Optional[dict]):
        self.dims = int(cfg["dims"]) if cfg else 0
        self.tables = rt.rotation(cfg["base"], self.dims) if self.dims else None

    def args(self) -> dict:
        return dict(tables=self.tables, rot_dims=self.dims)


class TalkingAttention:
    """Grouped-query softmax attention with q/k head norms, rotary positions, scores mixed across heads before the softmax, and a sliding window
    that keeps the first tokens.  One side of ``Parallel``."""

    def __init__(self, rt: Runtime, cfg: dict, get: Callable[[str], torch.Tensor], eps: float):
        self.rt, self.eps = rt, eps
        self.heads, self.kv_heads, self.dim, self.vdim = (int(cfg[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
        if self.heads % self.kv_heads:
            raise ValueError("heads must be a multiple of kv_heads")
        self.scale = float(cfg["scale"])
        mask = cfg.get("mask") or {"size": rt.ctx}   # no mask: every earlier key
        self.window, self.keep_first = int(mask["size"]), int(mask.get("keep_first", 0))
        self.rot = Rotation(rt, cfg.get("rot"))
        self.dp, self.vp = pad_to(self.dim, 16), pad_to(self.vdim, 16)
        self.projections = [get("q"), get("k"), get("v")]
        self.q_norm, self.k_norm = rt.vector(get("q.norm")), rt.vector(get("k.norm"))
        self.talk = rt.vector(get("talk"))
        self.o = get("o")
        self.q_off = 0

    def width_in(self) -> int:
        return self.heads * self.dim + self.kv_heads * (self.dim + self.vdim)

    def width_out(self) -> int:
        return self.heads * self.vdim

    def new_cache(self, cache: SequenceCache):
        return cache.add_kv(self.kv_heads, self.rt.ctx, self.dp, self.vp)

    def groups(self, kv, off: int, q_dst: Optional[int]) -> List[MixHeads]:
        """q, k and v at column `off` of a projection row; k and v go to the caches."""
        ctx = self.rt.ctx
        k_off = off + self.heads * self.dim
        v_off = k_off + self.kv_heads * self.dim
        return [_heads(off, self.heads, self.dim, dim_pad=self.dp, dst=q_dst, row_stride=self.heads * self.dp, head_stride=self.dp, norm=self.q_norm, ctx=ctx,
                       **self.rot.args()),
                _heads(k_off, self.kv_heads, self.dim, dim_pad=self.dp, dst=kv[0].data_ptr(), row_stride=self.dp, head_stride=ctx * self.dp, norm=self.k_norm,
                       by_position=True, ctx=ctx, **self.rot.args()),
                _heads(v_off, self.kv_heads, self.vdim, dim_pad=self.vp, dst=kv[1].data_ptr(), row_stride=self.vp, head_stride=ctx * self.vp, by_position=True,
                       ctx=ctx)]

    def attend(self, q: int, kv, out: int, out_stride: int, out_scale: float, pos: int, rows: int, sp) -> None:
        L = self.rt.L
        need = L.cq_mix_talk_attention_workspace_bytes(rows, self.heads, self.vdim, self.window, self.keep_first, pos)
        ws = self.rt.scratch("attention_splits", need // 4) if need else None
        check("cq_mix_talk_attention", L.cq_mix_talk_attention(
            q, kv[0].data_ptr(), kv[1].data_ptr(), self.talk.data_ptr(), self.scale, self.window, self.keep_first, out_scale, out, out_stride, pos, rows, self.heads,
            self.kv_heads, self.dp, self.vdim, self.vp, self.rt.ctx, ws, need, sp))

    def records(self):
        n = self.rt.L.cq_mix_talk_decode_workspace_bytes(self.heads, self.vdim, self.window, self.keep_first, self.rt.ctx)
        return self.rt.scratch("attention_records", n // 4), n


class Retention:
    """Linear attention with one fixed decay per head, rotary positions, RMS-normalized heads and a silu gate.  One side of ``Parallel``."""

    def __init__(self, rt: Runtime, cfg: dict, get: Callable[[str], torch.Tensor], eps: float):
        self.rt, self.eps = rt, eps
        self.heads, self.dim, self.vdim = (int(cfg[k]) for k in ("heads", "dim", "vdim"))
        decay = np.asarray(cfg["decay"], dtype=np.float64)
        if decay.shape != (self.heads,):
            raise ValueError("one decay per head")
        self.decay = rt.vector(torch.from_numpy(decay))
        with np.errstate(divide="ignore"):           # a decay of 0: finite, so that gamma^0 stays 1
            self.log2_decay = rt.vector(torch.from_numpy(np.maximum(np.log2(decay), -1e30)))
        self.rot = Rotation(rt, cfg.get("rot"))
        self.dp = pad_to(self.dim, 16)
        self.projections = [get("q"), get("k"), get("v"), get("g")]
        self.o = get("o")

    def width_in(self) -> int:
        return 2 * self.heads * (self.dim + self.vdim)

    def width_out(self) -> int:
        return self.heads * self.vdim

    def new_cache(self, cache: SequenceCache) -> torch.Tensor:
        return cache.add_state(self.heads, self.vdim, self.rt.L.cq_mix_state_pad(self.dim))

    def offsets(self, off: int):
        """Columns of v and of the gate in a projection row."""
        v = off + 2 * self.heads * self.dim
        return v, v + self.heads * self.vdim

    def groups(self, off: int, q_dst: Optional[int], k_dst: Optional[int]) -> List[MixHeads]:
        common = dict(dim_pad=self.dp, row_stride=self.heads * self.dp, head_stride=self.dp, ctx=self.rt.ctx, **self.rot.args())
        return [_heads(off, self.heads, self.dim, dst=q_dst, **common),
                _heads(off + self.heads * self.dim, self.heads, self.dim, dst=k_dst, factor=1.0 / math.sqrt(self.dim), **common)]

    def attend(self, q: int, k: int, row: int, row_stride: int, off: int, state: torch.Tensor, out: int, out_stride: int, out_scale: float, rows: int, sp) -> None:
        rt, L = self.rt, self.rt.L
        v_off, g_off = self.offsets(off)
        need = L.cq_mix_retention_workspace_bytes(rows, self.heads, self.dim, self.vdim)
        ws = rt.scratch("retention_segments", need // 4) if need else None
        raw, w = rt.scratch("mixer_raw", rows * self.width_out()), self.width_out()
        check("cq_mix_retention", L.cq_mix_retention(q, k, row + 4 * v_off, row_stride, self.log2_decay.data_ptr(), state.data_ptr(), raw, w, rows, self.heads, self.dim,
                                                     self.dp, self.vdim, ws, need, sp))
        check("cq_mix_head_norm_gate", L.cq_mix_head_norm_gate(raw, w, row + 4 * g_off, row_stride, None, SILU, out_scale, out, out_stride, rows, self.heads, self.vdim,
                                                               self.eps, sp))


class Mixer:
    """A layer's first sublayer: x <- x + mixer(norm(x)).  ``norm_rows`` has left norm(x) in `h` for ``prefill``; ``step`` applies it itself."""

    def denses(self) -> List[Dense]:
        raise NotImplementedError

    def new_cache(self, cache: SequenceCache):
        raise NotImplementedError

    def prefill(self, h: int, ldh: int, x: int, ldx: int, kept, pos: int, rows: int, sp) -> None:
        raise NotImplementedError

    def step(self, x: int, norm: torch.Tensor, kept, pos_dev: Optional[int], pos: int, add: Optional[int], sp) -> None:
        raise NotImplementedError


class Parallel(Mixer):
    """Attention and retention side by side on the same input, left_scale * left + right_scale * right.  One product projects for both, one takes
    their outputs, side by side and already scaled, back to the residual stream."""

    def __init__(self, rt: Runtime, cfg: dict, get: Callable[[str], torch.Tensor], eps: float):
        self.rt, self.eps = rt, eps
        self.left = TalkingAttention(rt, cfg["left"], lambda n: get("left." + n), eps)
        self.right = Retention(rt, cfg["right"], lambda n: get("right." + n), eps)
        self.left_scale, self.right_scale = float(cfg["left_scale"]), float(cfg["right_scale"])
        self.w_in = Dense(rt, self.left.projections + self.right.projections)
        self.w_out = Dense(rt, [self.left.o, self.right.o], along="in")
        self.off = self.left.width_in()              # the right side's first column
        if self.w_in.n != self.off + self.right.width_in() or self.w_out.k != self.left.width_out() + self.right.width_out():
            raise ValueError("projection sizes do not match the mixer's configuration")
        del self.left.projections, self.right.projections, self.left.o, self.right.o

    def denses(self) -> List[Dense]:
        return [self.w_in, self.w_out]

    def new_cache(self, cache: SequenceCache):
        return self.left.new_cache(cache), self.right.new_cache(cache)

    def prefill(self, h, ldh, x, ldx, kept, pos, rows, sp):
        rt, lt, rg = self.rt, self.left, self.right
        kv, state = kept
        ldp, ldo = pad_to(self.w_in.n, 4), self.w_out.kp
        row = rt.scratch("projection", rows * ldp)
        q = rt.scratch("attention_q", rows * lt.heads * lt.dp)
        rq, rk = rt.scratch("retention_q", rows * rg.heads * rg.dp), rt.scratch("retention_k", rows * rg.heads * rg.dp)
        out = rt.scratch("mixer_out", rows * ldo)
        self.w_in.rows(h, ldh, row, ldp, rows, sp)
        groups = _group_array(lt.groups(kv, 0, q) + rg.groups(self.off, rq, rk))
        check("cq_mix_pack_heads", rt.L.cq_mix_pack_heads(row, ldp, groups, len(groups), self.eps, None, pos, rows, sp))
        lt.attend(q, kv, out, ldo, self.left_scale, pos, rows, sp)
        rg.attend(rq, rk, row, ldp, self.off, state, out + 4 * lt.width_out(), ldo, self.right_scale, rows, sp)
        self.w_out.rows(out, ldo, x, ldx, rows, sp, accumulate=True)

    def step(self, x, norm, kept, pos_dev, pos, add, sp):
        rt, lt, rg = self.rt, self.left, self.right
        kv, state = kept
        row, out = rt.scratch("projection", self.w_in.n), rt.scratch("mixer_out", self.w_out.kp)
        rec, rec_bytes = lt.records()
        self.w_in.row(x, row, sp, NORM, norm, self.eps)
        check("cq_mix_talk_decode", rt.L.cq_mix_talk_decode(row, _group_array(lt.groups(kv, 0, None)), self.eps, lt.talk.data_ptr(), lt.scale, lt.window,
                                                            lt.keep_first, pos_dev, pos, rec, rec_bytes, sp))
        v_off, g_off = rg.offsets(self.off)
        check("cq_mix_talk_merge_retention_step", rt.L.cq_mix_talk_merge_retention_step(
            rec, lt.heads, lt.vdim, lt.window, lt.keep_first, rt.ctx, self.left_scale, out, row, _group_array(rg.groups(self.off, None, None)), v_off, g_off,
            rg.decay.data_ptr(), state.data_ptr(), rg.heads, rg.vdim, self.eps, self.right_scale, out + 4 * lt.width_out(), pos_dev, pos, sp))
        self.w_out.row(out, x, sp, accumulate=True, add=add)


class GeneralDelta(Mixer):
    """The generalized delta rule: a decay and a removal rate per head and key channel, the decay through a low-rank projection."""

    def __init__(self, rt: Runtime, cfg: dict, get: Callable[[str], torch.Tensor], eps: float):
        self.rt, self.eps = rt, eps
        self.heads, self.dim = int(cfg["heads"]), int(cfg["dim"])
        self.width = self.heads * self.dim
        low = get("w1")
        self.rank = low.shape[0]
        self.w_in = Dense(rt, [get(n) for n in ("r", "k", "v", "g", "a")] + [low])
        self.w2 = Dense(rt, [get("w2")])
        self.w_out = Dense(rt, [get("o")])
        self.w0, self.a_bias, self.norm = (rt.vector(get(n)) for n in ("w0", "a.b", "norm"))
        if self.w_in.n != 5 * self.width + self.rank or self.w2.k != self.rank or self.w2.n != self.width:
            raise ValueError("projection sizes do not match the mixer's configuration")
        self.r_off, self.k_off, self.v_off, self.g_off, self.a_off, self.low_off = (i * self.width for i in range(6))

    def denses(self) -> List[Dense]:
        return [self.w_in, self.w2, self.w_out]

    def new_cache(self, cache: SequenceCache) -> torch.Tensor:
        return cache.add_state(self.heads, self.dim, self.rt.L.cq_mix_state_pad(self.dim))

    def prefill(self, h, ldh, x, ldx, kept, pos, rows, sp):
        rt, L, w = self.rt, self.rt.L, self.width
        ldp, ldw, ldo = pad_to(self.w_in.n, 4), pad_to(w, 4), self.w_out.kp
        row = rt.scratch("projection", rows * ldp)
        low, wl = rt.scratch("delta_low", rows * self.w2.kp), rt.scratch("delta_decay", rows * ldw)
        packed = rt.scratch("delta_packed", rows * self.heads * (4 * L.cq_mix_state_pad(self.dim) + 1))
        raw, out = rt.scratch("mixer_raw", rows * w), rt.scratch("mixer_out", rows * ldo)
        self.w_in.rows(h, ldh, row, ldp, rows, sp)
        check("cq_mix_tanh", L.cq_mix_tanh(row + 4 * self.low_off, ldp, low, self.w2.kp, rows, self.rank, sp))
        self.w2.rows(low, self.w2.kp, wl, ldw, rows, sp)
        check("cq_mix_delta_prep", L.cq_mix_delta_prep(row, ldp, self.r_off, self.k_off, self.a_off, wl, ldw, self.w0.data_ptr(), self.a_bias.data_ptr(), packed, rows,
                                                       self.heads, self.dim, sp))
        check("cq_mix_delta_scan", L.cq_mix_delta_scan(packed, row + 4 * self.v_off, ldp, kept.data_ptr(), raw, w, rows, self.heads, self.dim, sp))
        check("cq_mix_head_norm_gate", L.cq_mix_head_norm_gate(raw, w, row + 4 * self.g_off, ldp, self.norm.data_ptr(), SIGMOID, 1.0, out, ldo, rows, self.heads,
                                                               self.dim, self.eps, sp))
        self.w_out.rows(out, ldo, x, ldx, rows, sp, accumulate=True)

    def step(self, x, norm, kept, pos_dev, pos, add, sp):
        rt = self.rt
        row, out = rt.scratch("projection", self.w_in.n), rt.scratch("mixer_out", self.w_out.kp)
        self.w_in.row(x, row, sp, NORM, norm, self.eps)
        check("cq_mix_delta_step", rt.L.cq_mix_delta_step(row, self.r_off, self.k_off, self.v_off, self.g_off, self.a_off, self.low_off, self.w2.w.data_ptr(), self.w2.kp,
                                                          self.rank, self.w0.data_ptr(), self.a_bias.data_ptr(), self.norm.data_ptr(), kept.data_ptr(), out,
                                                          self.heads, self.dim, self.eps, sp))
        self.w_out.row(out, x, sp, accumulate=True, add=add)


class PolyFeedForward:
    """down(PolyNorm(up(norm(x)))): the activation is a polynomial whose powers are each divided by the row's root mean square."""

    def __init__(self, rt: Runtime, cfg: dict, get: Callable[[str], torch.Tensor], eps: float):
        self.rt, self.eps = rt, eps
        self.up, self.down = Dense(rt, [get("up")]), Dense(rt, [get("down")])
        self.coef = rt.vector(get("act"))
        self.ff = int(cfg["ff"])
        if self.up.n != self.ff or self.down.k != self.ff or self.coef.numel() != 4:
            raise ValueError("feed-forward sizes do not match the configuration")

    def denses(self) -> List[Dense]:
        return [self.up, self.down]

    def prefill(self, h, ldh, x, ldx, rows, sp):
        rt, ld = self.rt, self.down.kp
        z = rt.scratch("feed_forward", rows * ld)
        self.up.rows(h, ldh, z, ld, rows, sp)
        check("cq_mix_poly_norm", rt.L.cq_mix_poly_norm(z, ld, self.coef.data_ptr(), z, ld, rows, self.ff, self.eps, sp))
        self.down.rows(z, ld, x, ldx, rows, sp, accumulate=True)

    def step(self, x, norm, add, sp):
        z = self.rt.scratch("feed_forward", self.down.kp)
        self.up.row(x, z, sp, NORM, norm, self.eps)
        self.down.row(z, x, sp, POLY, self.coef, self.eps, accumulate=True, add=add)


MIXERS = {"parallel": Parallel, "general_delta": GeneralDelta}
FEED_FORWARDS = {"dense": PolyFeedForward}
