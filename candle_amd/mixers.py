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
from typing import Callable, Dict, List, NamedTuple, Optional

import numpy as np
import torch

from . import _lib
from ._lib import DenseArgs, Latent, MixHeads, Moe
from .cache import SequenceCache

BF16, F32 = 0, 1                                     # enum cq_dense_precision
PLAIN, NORM, POLY, LAYER_NORM, RELU2 = 0, 1, 2, 3, 4  # enum cq_dense_prologue
ACT_NONE, ACT_RELU2, ACT_SWIGLU = 0, 1, 2            # enum cq_dense_act
SILU, SIGMOID = 0, 1                                 # enum cq_gate
MATVEC_MAX_K = 32768                                 # CQ_DENSE_MATVEC_MAX_K

check = _lib.check


def pad_to(n: int, m: int) -> int:
    return (n + m - 1) // m * m


def frequencies(base: float, dims: int, scaling: Optional[dict] = None) -> tuple:
    """Angle per position of each pair of dimensions, base^(-2 i / dims), and a factor on cos and sin (1 without scaling).

    YaRN scaling: pairs that turn more than ``fast`` times over ``original`` positions keep their frequency, those that turn less than ``slow``
    times are slowed down by ``factor``, those between are blended linearly in i; cos and sin grow by 0.1 ln(factor) + 1."""
    i = np.arange(dims // 2, dtype=np.float64)
    freq = np.float64(base) ** (-2.0 * i / dims)
    if not scaling:
        return freq, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])
    pair = lambda turns: dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(pair(float(scaling["fast"]))), 0), min(math.ceil(pair(float(scaling["slow"]))), dims - 1)
    slowed = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return freq * (1.0 - slowed) + freq / factor * slowed, 0.1 * math.log(factor) + 1.0


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

    @property
    def t_bf16(self) -> bool:
        """Whether intermediate values that only feed matrix products are kept in bfloat16."""
        return self.precision == BF16

    def typed(self, name: str, count: int) -> int:
        """Scratch for ``count`` values of the products' input type.  A name is used either for these or for f32 (one read as the other
        need not be finite)."""
        return self.scratch(name, (count + 1) // 2 if self.t_bf16 else count)

    def normed(self, kinds: tuple, count: int) -> Normed:
        """Scratch for normed rows.  Without reduced precision both kinds are one buffer."""
        f32, typed = kinds
        if not self.t_bf16:
            p = self.scratch("h", count)
            return Normed(p, p)
        return Normed(self.scratch("h", count) if f32 else None, self.typed("h_typed", count) if typed else None)

    def rotation(self, base: float, dims: int, scaling: Optional[dict] = None) -> tuple:
        """cos / sin [ctx, dims / 2] of t * frequency, evaluated in double and rounded once (see ``frequencies``)."""
        key = (float(base), int(dims), tuple(sorted(scaling.items())) if scaling else None)
        if key not in self._tables:
            freq, factor = frequencies(base, dims, scaling)
            ang = np.arange(self.ctx, dtype=np.float64)[:, None] * freq
            self._tables[key] = tuple(torch.from_numpy((factor * f(ang)).astype(np.float32)).to(self.device) for f in (np.cos, np.sin))
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

    def rows(self, x: int, ldx: int, dst: int, ldd: int, rows: int, sp, accumulate: bool = False, precision: Optional[int] = None, **options) -> None:
        """Several rows; `options` are further fields of cq_dense_args."""
        rt = self.rt
        precision = rt.precision if precision is None else precision
        need = rt.L.cq_dense_matmul_workspace_bytes(precision, rows, self.n, self.kp)
        dense_product(rt, precision, sp, rt.scratch("dense_planes", need // 4) if need else None, need, w_dev=self.w.data_ptr(), ldw=self.kp, x_dev=x, ldx=ldx, dst_dev=dst,
                      ldd=ldd, m=rows, n=self.n, k=self.kp, batch=1, accumulate=int(accumulate), **options)

    def row(self, x: int, dst: int, sp, prologue: int = PLAIN, vec: Optional[torch.Tensor] = None, eps: float = 0.0, accumulate: bool = False,
            add: Optional[int] = None) -> None:
        check("cq_dense_matvec", self.rt.L.cq_dense_matvec(self.w.data_ptr(), self.kp, x, prologue, vec.data_ptr() if vec is not None else None, eps, self.k, dst,
                                                          add, int(accumulate), self.n, self.kp, sp))


def dense_product(rt: Runtime, precision: int, sp, workspace=None, workspace_bytes: int = 0, **fields) -> None:
    check("cq_dense_product", rt.L.cq_dense_product(precision, DenseArgs(**fields), workspace, workspace_bytes, sp))


def alternate(gate: torch.Tensor, up: torch.Tensor) -> torch.Tensor:
    """Rows gate 0, up 0, gate 1, up 1, ...: what the gated activation of a product takes."""
    return torch.stack([gate, up], dim=1).reshape(2 * gate.shape[0], gate.shape[1])


class Normed(NamedTuple):
    """Normed rows as a block asks for them (``INPUT``): f32, the type of the products' inputs, or both.  Row strides are the same in elements."""

    f32: Optional[int] = None
    typed: Optional[int] = None


AS_F32, AS_TYPED, AS_BOTH = (True, False), (False, True), (True, True)


class RmsNorm:
    """x / rms(x) * weight, over rows or as the prologue of a single-row product."""

    prologue = NORM

    def __init__(self, rt: Runtime, get: Callable[[str], torch.Tensor], name: str, eps: float):
        self.rt, self.eps = rt, eps
        self.vec = rt.vector(get(name))
        self.dim = self.vec.numel()

    def rows(self, x: int, ldx: int, out: Normed, ldo: int, rows: int, sp, index: Optional[int] = None, delta: Optional[int] = None) -> None:
        """Rows of x (those that `index` names) into out; `delta` [rows, ldx] is added to x first."""
        if out.f32 is None or (out.typed is not None and out.typed != out.f32):
            raise ValueError("this norm writes f32 only")
        check("cq_mix_rms_norm_rows", self.rt.L.cq_mix_rms_norm_rows(x, ldx, index, delta, ldx, self.vec.data_ptr(), out.f32, ldo, rows, self.dim, self.eps, sp))


class LayerNorm:
    """(x - mean) / standard deviation * weight + bias; the bias is the tensor of the same name with '.b' added."""

    prologue = LAYER_NORM

    def __init__(self, rt: Runtime, get: Callable[[str], torch.Tensor], name: str, eps: float):
        self.rt, self.eps = rt, eps
        self.vec = torch.cat([rt.vector(get(name)), rt.vector(get(name + ".b"))])
        self.dim = self.vec.numel() // 2

    def rows(self, x: int, ldx: int, out: Normed, ldo: int, rows: int, sp, index: Optional[int] = None, delta: Optional[int] = None) -> None:
        if delta is not None:
            raise ValueError("this norm adds nothing to its input")
        f32, bf16 = (out.f32, out.typed) if self.rt.t_bf16 else (out.f32 or out.typed, None)
        check("cq_mix_layer_norm_rows", self.rt.L.cq_mix_layer_norm_rows(x, ldx, index, self.vec.data_ptr(), f32, bf16, ldo, rows, self.dim, self.eps, sp))


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
        self.tables = rt.rotation(cfg["base"], self.dims, cfg.get("scaling")) if self.dims else None

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
    """A layer's first sublayer: x <- x + mixer(norm(x)).  ``prefill`` finds norm(x) in `h`; ``step`` applies the norm itself."""

    INPUT = AS_F32                                   # how `prefill` wants its normed rows
    kv_from: Optional[int] = None                    # a layer whose cache this one attends to instead of having its own

    def denses(self) -> List[Dense]:
        raise NotImplementedError

    def new_cache(self, cache: SequenceCache):
        raise NotImplementedError

    def prefill(self, h: Normed, ldh: int, x: int, ldx: int, kept, pos: int, rows: int, sp) -> None:
        raise NotImplementedError

    def step(self, x: int, norm, kept, pos_dev: Optional[int], pos: int, add: Optional[int], sp) -> None:
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
        self.w_in.rows(h.f32, ldh, row, ldp, rows, sp)
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
        self.w_in.row(x, row, sp, norm.prologue, norm.vec, norm.eps)
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
        self.w_in.rows(h.f32, ldh, row, ldp, rows, sp)
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
        self.w_in.row(x, row, sp, norm.prologue, norm.vec, norm.eps)
        check("cq_mix_delta_step", rt.L.cq_mix_delta_step(row, self.r_off, self.k_off, self.v_off, self.g_off, self.a_off, self.low_off, self.w2.w.data_ptr(), self.w2.kp,
                                                          self.rank, self.w0.data_ptr(), self.a_bias.data_ptr(), self.norm.data_ptr(), kept.data_ptr(), out,
                                                          self.heads, self.dim, self.eps, sp))
        self.w_out.row(out, x, sp, accumulate=True, add=add)


class FeedForward:
    """A layer's second sublayer, like ``Mixer`` without anything kept."""

    INPUT = AS_F32

    def denses(self) -> List[Dense]:
        raise NotImplementedError

    def prefill(self, h: Normed, ldh: int, x: int, ldx: int, rows: int, sp) -> None:
        raise NotImplementedError

    def step(self, x: int, norm, add: Optional[int], sp) -> None:
        raise NotImplementedError


class PolyFeedForward(FeedForward):
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
        self.up.rows(h.f32, ldh, z, ld, rows, sp)
        check("cq_mix_poly_norm", rt.L.cq_mix_poly_norm(z, ld, self.coef.data_ptr(), z, ld, rows, self.ff, self.eps, sp))
        self.down.rows(z, ld, x, ldx, rows, sp, accumulate=True)

    def step(self, x, norm, add, sp):
        z = self.rt.scratch("feed_forward", self.down.kp)
        self.up.row(x, z, sp, norm.prologue, norm.vec, norm.eps)
        self.down.row(z, x, sp, POLY, self.coef, self.eps, accumulate=True, add=add)


class LatentAttention(Mixer):
    """Causal softmax attention whose keys and values are linear in a cached latent: per position one normed latent and one rotated key part for all
    heads.  Heads are gated by a sigmoid of their own.  With ``kv_from`` the layer has no latent of its own and attends to another layer's cache.

    Many rows: keys and values of all heads are computed from the cache rows, then attended to head by head.  Few rows and single tokens: the key matrix is
    applied to the query and the value matrix to the attended latent, so that the heads attend to the cache rows themselves."""

    INPUT = AS_TYPED
    MAX_RANK, MAX_HEAD, MAX_VALUE = 512, 320, 256    # CQ_LATENT_MAX_*; rotated parts of more than 64 (up to 192) with latents up to 256

    def __init__(self, rt: Runtime, cfg: dict, get: Callable[[str], torch.Tensor], eps: float):
        self.rt, self.eps = rt, eps
        self.heads, self.dim, self.rot_dim, self.vdim, self.rank = (int(cfg[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
        self.kv_from = None if cfg.get("kv_from") is None else int(cfg["kv_from"])
        H, r = self.heads, self.rank
        self.rank_pad, self.rot_pad, self.dim_pad, self.v_pad = pad_to(r, 64), pad_to(self.rot_dim, 8), pad_to(self.dim, 8), pad_to(self.vdim, 8)
        self.ld = self.rank_pad + self.rot_pad
        if self.rot_pad > 192 or self.rank_pad > (256 if self.rot_pad > 64 else self.MAX_RANK):
            raise ValueError(f"latents of {r} + {self.rot_dim} values: at most {self.MAX_RANK} + 64 or 256 + 192")
        rot = Rotation(rt, cfg.get("rot"))
        if rot.dims != self.rot_dim:
            raise ValueError("the rotated part of a head is rotated as a whole")
        own = self.kv_from is None
        self.w_in = Dense(rt, [get("q")] + ([get("dkv")] if own else []) + [get("g")])
        self.kv_off = H * (self.dim + self.rot_dim) if own else -1
        self.g_off = self.w_in.n - H
        if self.w_in.n != H * (self.dim + self.rot_dim + 1) + (r + self.rot_dim if own else 0):
            raise ValueError("projection sizes do not match the mixer's configuration")
        uk, uv = get("uk").to(rt.device), get("uv").to(rt.device)
        if uk.shape != (H * self.dim, r) or uv.shape != (H * self.vdim, r):
            raise ValueError("key and value sizes do not match the mixer's configuration")
        self.ukt = torch.zeros((H, r, pad_to(self.dim, 64)), dtype=torch.bfloat16, device=rt.device)
        self.ukt[..., :self.dim] = uk.view(H, self.dim, r).transpose(1, 2)
        self.uv = Dense(rt, [uv])
        self.w_out = Dense(rt, [get("o")])
        self.expand = None
        if self.dim_pad + self.rot_pad <= self.MAX_HEAD and self.v_pad <= self.MAX_VALUE:
            padded = lambda w, d, dp: torch.nn.functional.pad(w.view(H, d, r), (0, 0, 0, dp - d)).reshape(H * dp, r)
            self.expand = Dense(rt, [padded(uk, self.dim, self.dim_pad), padded(uv, self.vdim, self.v_pad)])
        norm = rt.vector(get("dkv.norm")) if own else None
        self.norm, self.tables = norm, rot.tables
        self.shape = Latent(norm.data_ptr() if own else None, rot.tables[0].data_ptr() if rot.dims else None, rot.tables[1].data_ptr() if rot.dims else None, H, self.dim,
                            self.rot_dim, self.vdim, r, self.rank_pad, self.rot_pad, rt.ctx, int(rt.t_bf16), float(cfg["scale"]), eps, 0)

    def denses(self) -> List[Dense]:
        return [self.w_in, self.uv, self.w_out]

    def token_bytes(self) -> int:
        """Weight bytes of a single-token step."""
        return sum(d.nbytes() for d in self.denses()) + self.ukt.numel() * 2

    def new_cache(self, cache: SequenceCache) -> torch.Tensor:
        return cache.add_rows(self.rt.ctx, self.ld, torch.bfloat16 if self.rt.t_bf16 else torch.float32)

    def expands(self, rows: int) -> bool:
        """Whether computing keys and values per head costs less than attending to latents with `rows` queries (whose longer products run at about half the
        rate)."""
        d = self.dim + self.vdim
        return self.expand is not None and 2 * rows * (2 * self.rank - d) > self.rank * d

    def prefill(self, h, ldh, x, ldx, kept, pos, rows, sp):
        rt, L, H = self.rt, self.rt.L, self.heads
        ldp, ldo, bf = pad_to(self.w_in.n, 4), self.w_out.kp, int(rt.t_bf16)
        row, out = rt.scratch("projection", rows * ldp), rt.typed("mixer_out_typed", rows * ldo)
        gate = row + 4 * self.g_off
        self.w_in.rows(h.typed, ldh, row, ldp, rows, sp, x_bf16=bf)
        if self.expands(rows):
            head, keys = self.dim_pad + self.rot_pad, pos + rows
            ldkv = self.expand.n + (0 if self.expand.n // 128 % 2 else 128)     # rows an odd number of 256 bytes apart fall on all memory channels
            q, kv = rt.typed("latent_q", rows * H * head), rt.typed("latent_kv", keys * ldkv)
            check("cq_mix_latent_pack", L.cq_mix_latent_pack(self.shape, row, ldp, self.kv_off, kept.data_ptr(), None, 0, q, head, self.dim_pad, pos, rows, sp))
            self.expand.rows(kept.data_ptr(), self.ld, kv, ldkv, keys, sp, x_bf16=bf, dst_bf16=bf)
            check("cq_mix_latent_expanded", L.cq_mix_latent_expanded(self.shape, q, self.dim_pad, kv, ldkv, H * self.dim_pad, self.v_pad, kept.data_ptr(), gate, ldp, out, ldo,
                                                                     pos, rows, sp))
        else:
            kp = self.ukt.shape[2]
            plain, q, lat = rt.scratch("latent_plain", rows * H * kp), rt.typed("latent_q", rows * H * self.ld), rt.scratch("latent_out", rows * H * self.rank_pad)
            check("cq_mix_latent_pack", L.cq_mix_latent_pack(self.shape, row, ldp, self.kv_off, kept.data_ptr(), plain, kp, q, self.ld, self.rank_pad, pos, rows, sp))
            dense_product(rt, rt.precision, sp, w_dev=self.ukt.data_ptr(), ldw=kp, w_batch=self.rank * kp, x_dev=plain, ldx=H * kp, x_batch=kp, dst_dev=q, ldd=H * self.ld,
                          dst_batch=self.ld, dst_bf16=bf, m=rows, n=self.rank, k=kp, batch=H)
            need = L.cq_mix_latent_absorbed_workspace_bytes(self.shape, rows, pos, 0)
            ws = rt.scratch("attention_splits", need // 4) if need else None
            check("cq_mix_latent_absorbed", L.cq_mix_latent_absorbed(self.shape, q, kept.data_ptr(), gate, ldp, lat, pos, rows, ws, need, sp))
            dense_product(rt, rt.precision, sp, w_dev=self.uv.w.data_ptr(), ldw=self.uv.kp, w_batch=self.vdim * self.uv.kp, x_dev=lat, ldx=H * self.rank_pad,
                          x_batch=self.rank_pad, dst_dev=out, ldd=ldo, dst_batch=self.vdim, dst_bf16=bf, m=rows, n=self.vdim, k=self.uv.kp, batch=H)
        self.w_out.rows(out, ldo, x, ldx, rows, sp, accumulate=True, x_bf16=bf)

    def step(self, x, norm, kept, pos_dev, pos, add, sp):
        rt, L = self.rt, self.rt.L
        row, out, q = rt.scratch("projection", self.w_in.n), rt.scratch("mixer_out", self.w_out.kp), rt.typed("latent_q", self.heads * self.ld)
        need = L.cq_mix_latent_absorbed_workspace_bytes(self.shape, 1, 0, 1)
        ws = rt.scratch("attention_records", need // 4)
        self.w_in.row(x, row, sp, norm.prologue, norm.vec, norm.eps)
        check("cq_mix_latent_step", L.cq_mix_latent_step(self.shape, row, self.kv_off, kept.data_ptr(), self.ukt.data_ptr(), self.ukt.shape[2], self.uv.w.data_ptr(), self.uv.kp,
                                                         self.g_off, q, out, pos_dev, pos, ws, need, sp))
        self.w_out.row(out, x, sp, accumulate=True, add=add)


class ReluSquaredFeedForward(FeedForward):
    """down(relu(up(norm(x)))^2)."""

    INPUT = AS_TYPED

    def __init__(self, rt: Runtime, cfg: dict, get: Callable[[str], torch.Tensor], eps: float):
        self.rt = rt
        self.up, self.down = Dense(rt, [get("up")]), Dense(rt, [get("down")])
        if self.up.n != int(cfg["ff"]) or self.down.k != int(cfg["ff"]):
            raise ValueError("feed-forward sizes do not match the configuration")

    def denses(self) -> List[Dense]:
        return [self.up, self.down]

    def prefill(self, h, ldh, x, ldx, rows, sp):
        rt, ld, bf = self.rt, self.down.kp, int(self.rt.t_bf16)
        z = rt.typed("activation", rows * ld)
        self.up.rows(h.typed, ldh, z, ld, rows, sp, act=ACT_RELU2, x_bf16=bf, dst_bf16=bf)
        self.down.rows(z, ld, x, ldx, rows, sp, accumulate=True, x_bf16=bf)

    def step(self, x, norm, add, sp):
        z = self.rt.scratch("feed_forward", self.down.kp)
        self.up.row(x, z, sp, norm.prologue, norm.vec, norm.eps)
        self.down.row(z, x, sp, RELU2, accumulate=True, add=add)


class GatedExperts(FeedForward):
    """A mixture of small feed-forwards down(silu(gate(h)) * up(h)), weighted by the softmax over the chosen router logits, and optionally one that every token
    takes, weighted by a sigmoid.  The choice and everything after it stay on the device."""

    INPUT = AS_BOTH                                  # the router reads f32

    def __init__(self, rt: Runtime, cfg: dict, get: Callable[[str], torch.Tensor], eps: float):
        self.rt = rt
        self.experts, self.top, self.ff = int(cfg["router"]["experts"]), int(cfg["router"]["top"]), int(cfg["expert"]["ff"])
        router = get("router")
        self.width = router.shape[1]
        if not 1 <= self.top <= self.experts or router.shape[0] != self.experts:
            raise ValueError("router sizes do not match the configuration")
        shared = cfg.get("shared")
        self.shared_ff = int(shared["ff"]) if shared else 0
        self.router = Dense(rt, [router] + ([get("shared.sg")] if shared else []))
        self.kp, self.ffp = pad_to(self.width, 64), pad_to(self.ff, 64)
        self.up = torch.zeros((self.experts, 2 * self.ff, self.kp), dtype=torch.bfloat16, device=rt.device)
        self.down = torch.zeros((self.experts, self.width, self.ffp), dtype=torch.bfloat16, device=rt.device)
        for e in range(self.experts):
            gate, up, down = (get(f"e{e}.{n}").to(rt.device) for n in ("gate", "up", "down"))
            if gate.shape != (self.ff, self.width) or up.shape != gate.shape or down.shape != (self.width, self.ff):
                raise ValueError("expert sizes do not match the configuration")
            self.up[e, :, :self.width] = alternate(gate, up)
            self.down[e, :, :self.ff] = down
        self.shared_up = self.shared_down = None
        if shared:
            self.shared_up, self.shared_down = Dense(rt, [alternate(get("shared.gate"), get("shared.up"))]), Dense(rt, [get("shared.down")])
            if self.shared_up.n != 2 * self.shared_ff or self.shared_down.k != self.shared_ff:
                raise ValueError("shared expert sizes do not match the configuration")
        self.sizes = Moe(self.up.data_ptr(), self.down.data_ptr(), self.shared_up.w.data_ptr() if shared else None, self.shared_down.w.data_ptr() if shared else None,
                         self.up[0].numel(), self.down[0].numel(), self.experts, self.top, self.kp, self.ff, self.ffp, self.shared_ff, self.shared_down.kp if shared else 0, 0)
        self.fused = bool(rt.L.cq_mix_moe_step_fits(self.sizes))

    def denses(self) -> List[Dense]:
        return [self.router]

    def token_bytes(self) -> int:
        """Weight bytes of a single-token step."""
        shared = self.shared_up.nbytes() + self.shared_down.nbytes() if self.shared_ff else 0
        return self.router.nbytes() + shared + 2 * self.top * (self.up[0].numel() + self.down[0].numel())

    def prefill(self, h, ldh, x, ldx, rows, sp):
        rt, L, E, top, bf = self.rt, self.rt.L, self.experts, self.top, int(self.rt.t_bf16)
        ldl, pairs = pad_to(self.router.n, 4), rows * top
        logits = rt.scratch("router_logits", rows * ldl)
        ids, weights, shared = rt.scratch("expert_ids", pairs), rt.scratch("expert_weights", pairs), rt.scratch("shared_weights", rows)
        self.router.rows(h.f32, ldh, logits, ldl, rows, sp, precision=F32)
        check("cq_mix_moe_select", L.cq_mix_moe_select(logits, ldl, rows, E, top, ids, weights, shared if self.shared_ff else None, sp))
        if self.shared_ff:
            ld = self.shared_down.kp
            z = rt.typed("shared_activation", rows * ld)
            self.shared_up.rows(h.typed, ldh, z, ld, rows, sp, act=ACT_SWIGLU, row_scale_dev=shared, x_bf16=bf, dst_bf16=bf)
            self.shared_down.rows(z, ld, x, ldx, rows, sp, accumulate=True, x_bf16=bf)
        per_expert = pairs / E
        tile = 64 if not bf else (128 if per_expert >= 96 else (64 if per_expert >= 24 else 32))
        max_tiles = L.cq_mix_moe_max_tiles(rows, E, top, tile)
        src, dst, scale = (rt.scratch("pair_" + n, pairs) for n in ("src", "dst", "scale"))
        tiles, n_tiles = rt.scratch("pair_tiles", 4 * max_tiles), rt.scratch("pair_n_tiles", 1)
        check("cq_mix_moe_plan", L.cq_mix_moe_plan(ids, weights, rows, E, top, tile, src, dst, scale, tiles, n_tiles, sp))
        z, ldy = rt.typed("expert_activation", pairs * self.ffp), pad_to(self.width, 4)
        y = rt.scratch("expert_out", pairs * ldy)
        grouped = dict(tiles_dev=tiles, n_tiles_dev=n_tiles, max_tiles=max_tiles, tile_rows=tile, m=pairs, batch=1)
        dense_product(rt, rt.precision, sp, w_dev=self.up.data_ptr(), ldw=self.kp, w_batch=self.up[0].numel(), x_dev=h.typed, ldx=ldh, dst_dev=z, ldd=self.ffp,
                      n=2 * self.ff, k=self.kp, src_rows_dev=src, row_scale_dev=scale, act=ACT_SWIGLU, x_bf16=bf, dst_bf16=bf, **grouped)
        dense_product(rt, rt.precision, sp, w_dev=self.down.data_ptr(), ldw=self.ffp, w_batch=self.down[0].numel(), x_dev=z, ldx=self.ffp, dst_dev=y, ldd=ldy, n=self.width,
                      k=self.ffp, dst_rows_dev=dst, x_bf16=bf, **grouped)
        check("cq_mix_moe_add", L.cq_mix_moe_add(y, ldy, top, x, ldx, rows, self.width, sp))

    def step(self, x, norm, add, sp):
        rt = self.rt
        if not self.fused:                           # sizes beyond the two launches: the several-row path with one row
            if add is not None:
                raise ValueError("no addend on this path")
            h = rt.normed(self.INPUT, self.kp)
            norm.rows(x, self.kp, h, self.kp, 1, sp)
            self.prefill(h, self.kp, x, self.kp, 1, sp)
            return
        logits, ids = rt.scratch("router_logits", pad_to(self.router.n, 4)), rt.scratch("expert_ids", self.top)
        act = rt.scratch("feed_forward", self.top * self.ffp + (self.shared_down.kp if self.shared_ff else 0))
        self.router.row(x, logits, sp, norm.prologue, norm.vec, norm.eps)
        check("cq_mix_moe_step", rt.L.cq_mix_moe_step(self.sizes, x, norm.prologue, norm.vec.data_ptr(), norm.eps, self.width, logits, act, ids, add, sp))
