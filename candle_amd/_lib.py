"""ctypes binding of libcandle_hip_quant.so (the C ABI declared in include/candle_hip_quant.h and
include/candle_hip_nn.h) and of libcandle_hip_mixer.so (include/candle_hip_mixer.h, plus the glue of candle_hip_nn.h).

The library must be built first (``python -m candle_amd.build`` or ``__graft_entry__.build()``);
loading fails loudly when it is missing — there is no CPU or PyTorch fallback.
"""
from __future__ import annotations

import ctypes
import os

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "libcandle_hip_quant.so")
MIXER_LIB_PATH = os.path.join(_HERE, "libcandle_hip_mixer.so")

_i64 = ctypes.c_int64
_int = ctypes.c_int
_vp = ctypes.c_void_p
_f32 = ctypes.c_float

# name -> (restype, argtypes); mirrors the two headers under include/ one to one
SIGNATURES = {
    "cq_status_string": (ctypes.c_char_p, [_int]),
    "cq_block_size": (_i64, [_int]),
    "cq_type_size": (_i64, [_int]),
    "cq_storage_bytes": (_i64, [_int, _i64]),
    "cq_dequantize": (_int, [_int, _vp, _vp, _i64, _int, _vp]),
    "cq_embedding": (_int, [_int, _vp, _vp, _vp, _i64, _i64, _i64, _vp]),
    "cq_quantize": (_int, [_int, _vp, _vp, _i64, _vp]),
    "cq_act_scratch_bytes": (_i64, [_int, _i64, _i64]),
    "cq_quantize_act": (_int, [_int, _vp, _int, _vp, _i64, _i64, _vp]),
    "cq_matvec": (_int, [_int, _vp, _vp, _vp, _int, _i64, _i64, _i64, _i64, _vp]),
    "cq_matmul": (_int, [_int, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _vp]),
    "cq_qmatmul_workspace_bytes": (_i64, [_int, _i64, _i64, _i64]),
    "cq_qmatmul_stream_step_bytes": (_i64, [_int, _i64, _i64]),
    "cq_qmatmul_forward": (_int, [_int, _vp, _vp, _int, _vp, _int, _i64, _i64, _i64, _vp, _i64, _vp]),
    "cq_static_workspace_bytes": (_i64, []),
    "cq_qmatmul_forward_static": (_int, [_int, _vp, _vp, _int, _vp, _int, _i64, _i64, _i64, _vp]),
    "cq_indexed_moe_workspace_bytes": (_i64, [_int, _i64, _i64, _i64, _i64, _i64, _i64]),
    "cq_indexed_moe_forward": (_int, [_int, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _i64, _i64, _vp, _i64, _vp]),
    "cq_moe_gemm_workspace_bytes": (_i64, [_int, _i64, _i64, _i64, _i64, _i64, _int]),
    "cq_moe_gemm_gguf_swiglu": (_int, [_int, _vp, _vp, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _i64, _vp]),
    "cq_moe_gemm_gguf_down_after_pair": (_int, [_int, _vp, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _i64, _i64, _vp, _i64, _vp]),
    "cq_moe_direct_pairs": (_int, [_int, _i64, _i64, _i64]),
    "cq_moe_gemm_gguf_pair": (_int, [_int, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _i64, _int, _vp, _i64, _vp]),
    "cq_moe_gemm_gguf": (_int, [_int, _vp, _vp, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _i64, _int, _vp, _i64, _vp]),
    # include/candle_hip_nn.h
    "cq_nn_embedding": (_int, [_vp, _vp, _vp, _i64, _i64, _i64, _vp, _vp]),
    "cq_nn_qmatmul_norm": (_int, [_int, _vp, _vp, _vp, _vp, _f32, _vp, _i64, _i64, _vp]),
    "cq_nn_qmatmul_residual": (_int, [_int, _vp, _vp, _vp, _vp, _vp, _i64, _i64, _vp]),
    "cq_nn_qmatmul_norm_swiglu": (_int, [_int, _vp, _vp, _vp, _vp, _vp, _f32, _vp, _i64, _i64, _vp]),
    "cq_nn_qmatmul_norm_pair": (_int, [_int, _vp, _i64, _vp, _int, _vp, _i64, _vp, _vp, _vp, _vp, _f32, _i64, _vp]),
    "cq_nn_qmatmul_split_planes": (_i64, [_int, _i64]),
    "cq_nn_qmatmul_split": (_int, [_int, _vp, _vp, _vp, _vp, _i64, _i64, _vp]),
    "cq_nn_qmatmul_norm_merge": (_int, [_int, _vp, _vp, _vp, _i64, _vp, _f32, _vp, _i64, _i64, _vp]),
    "cq_nn_qmatmul_norm_pair_merge": (_int, [_int, _vp, _i64, _vp, _int, _vp, _i64, _vp, _vp, _vp, _i64, _vp, _f32, _i64, _vp]),
    "cq_nn_qmatmul_residual_merge": (_int, [_int, _vp, _vp, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _vp]),
    "cq_nn_qmatmul_residual_attn_merge": (_int, [_int, _vp, _vp, _i64, _i64, _vp, _vp, _vp, _i64, _i64, _i64, _vp]),
    "cq_nn_qmatmul_residual_attn": (_int, [_int, _vp, _vp, _i64, _i64, _vp, _vp, _i64, _i64, _vp]),
    "cq_nn_moe_route": (_int, [_vp, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _int, _vp]),
    "cq_nn_moe_sort": (_int, [_vp, _vp, _vp, _i64, _i64, _vp]),
    "cq_nn_moe_sum": (_int, [_vp, _vp, _i64, _i64, _i64, _vp]),
    "cq_nn_rms_norm": (_int, [_vp, _vp, _vp, _vp, _vp, _i64, _i64, _f32, _vp]),
    "cq_nn_rope_i_kv": (_int, [_vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _i64, _i64, _i64, _i64, _i64, _vp]),
    "cq_nn_attention_workspace_bytes": (_i64, [_i64, _i64, _i64, _i64]),
    "cq_nn_attention": (_int, [_vp, _i64, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _i64, _i64, _i64, _f32, _vp, _i64, _vp]),
    "cq_nn_attention_decode_workspace_bytes": (_i64, [_i64, _i64, _i64]),
    "cq_nn_attention_decode_splits": (_i64, [_i64]),
    "cq_nn_attention_decode": (_int, [_vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _i64, _i64, _f32, _vp, _i64, _vp, _i64,
                                      _i64, _vp]),
    "cq_nn_coop_sync_bytes": (_i64, []),
    "cq_nn_decode_mlp": (_int, [_int, _vp, _vp, _int, _vp, _vp, _vp, _vp, _f32, _vp, _i64, _i64, _vp, _vp]),
    "cq_nn_silu_mul": (_int, [_vp, _vp, _vp, _i64, _i64, _i64, _i64, _vp]),
    "cq_nn_qmatmul_swiglu_rows": (_int, [_int, _vp, _vp, _vp, _i64, _i64, _vp, _i64, _i64, _i64, _vp, _i64, _vp]),
    "cq_nn_argmax": (_int, [_vp, _i64, _vp, _vp, _vp, _vp, _vp, _vp]),
    "cq_nn_argmax_embed": (_int, [_vp, _i64, _vp, _vp, _vp, _vp, _vp, _vp, _vp, _i64, _i64, _vp, _vp]),
}



class MixHeads(ctypes.Structure):
    """cq_mix_heads of include/candle_hip_mixer.h."""
    _fields_ = [("norm_dev", _vp), ("cos_dev", _vp), ("sin_dev", _vp), ("dst_dev", _vp), ("src_off", _i64), ("dst_row_stride", _i64),
                ("dst_head_stride", _i64), ("heads", ctypes.c_int32), ("dim", ctypes.c_int32), ("dim_pad", ctypes.c_int32),
                ("rot_dims", ctypes.c_int32), ("by_position", ctypes.c_int32), ("ctx", ctypes.c_int32), ("factor", _f32),
                ("reserved", ctypes.c_int32)]


_heads = ctypes.POINTER(MixHeads)


class DenseArgs(ctypes.Structure):
    """cq_dense_args of include/candle_hip_mixer.h."""
    _fields_ = [(n, _vp) for n in ("w_dev", "x_dev", "dst_dev", "add_dev", "row_scale_dev", "src_rows_dev", "dst_rows_dev", "n_tiles_dev", "tiles_dev")] + \
               [(n, _i64) for n in ("ldw", "ldx", "ldd", "ld_add", "m", "n", "k", "batch", "w_batch", "x_batch", "dst_batch", "max_tiles", "tile_rows")] + \
               [(n, ctypes.c_int32) for n in ("x_bf16", "dst_bf16", "accumulate", "act")]


class Latent(ctypes.Structure):
    """cq_latent of include/candle_hip_mixer.h."""
    _fields_ = [(n, _vp) for n in ("norm_dev", "cos_dev", "sin_dev")] + \
               [(n, ctypes.c_int32) for n in ("heads", "dim", "rot_dim", "vdim", "rank", "rank_pad", "rot_pad", "ctx", "bf16")] + \
               [("scale", _f32), ("eps", _f32), ("reserved", ctypes.c_int32)]


class Moe(ctypes.Structure):
    """cq_moe of include/candle_hip_mixer.h."""
    _fields_ = [(n, _vp) for n in ("up_dev", "down_dev", "shared_up_dev", "shared_down_dev")] + [("up_stride", _i64), ("down_stride", _i64)] + \
               [(n, ctypes.c_int32) for n in ("experts", "top", "kp", "ff", "ffp", "shared_ff", "shared_ffp", "reserved")]


_dense, _latent, _moe = ctypes.POINTER(DenseArgs), ctypes.POINTER(Latent), ctypes.POINTER(Moe)

# include/candle_hip_mixer.h
MIXER_SIGNATURES = {
    "cq_dense_matmul_workspace_bytes": (_i64, [_int, _i64, _i64, _i64]),
    "cq_dense_matmul": (_int, [_int, _vp, _i64, _vp, _i64, _vp, _i64, _vp, _i64, _int, _i64, _i64, _i64, _vp, _i64, _vp]),
    "cq_dense_product": (_int, [_int, _dense, _vp, _i64, _vp]),
    "cq_dense_matvec": (_int, [_vp, _i64, _vp, _int, _vp, _f32, _i64, _vp, _vp, _int, _i64, _i64, _vp]),
    "cq_mix_rms_norm_rows": (_int, [_vp, _i64, _vp, _vp, _i64, _vp, _vp, _i64, _i64, _i64, _f32, _vp]),
    "cq_mix_layer_norm_rows": (_int, [_vp, _i64, _vp, _vp, _vp, _vp, _i64, _i64, _i64, _f32, _vp]),
    "cq_mix_poly_norm": (_int, [_vp, _i64, _vp, _vp, _i64, _i64, _i64, _f32, _vp]),
    "cq_mix_tanh": (_int, [_vp, _i64, _vp, _i64, _i64, _i64, _vp]),
    "cq_mix_pack_heads": (_int, [_vp, _i64, _heads, _int, _f32, _vp, _i64, _i64, _vp]),
    "cq_mix_head_norm_gate": (_int, [_vp, _i64, _vp, _i64, _vp, _int, _f32, _vp, _i64, _i64, _i64, _i64, _f32, _vp]),
    "cq_mix_talk_attention_workspace_bytes": (_i64, [_i64, _i64, _i64, _i64, _i64, _i64]),
    "cq_mix_talk_attention": (_int, [_vp, _vp, _vp, _vp, _f32, _i64, _i64, _f32, _vp, _i64, _i64, _i64, _i64, _i64, _i64, _i64, _i64, _i64, _vp, _i64, _vp]),
    "cq_mix_talk_decode_workspace_bytes": (_i64, [_i64, _i64, _i64, _i64, _i64]),
    "cq_mix_talk_decode": (_int, [_vp, _heads, _f32, _vp, _f32, _i64, _i64, _vp, _i64, _vp, _i64, _vp]),
    "cq_mix_state_pad": (_i64, [_i64]),
    "cq_mix_retention_workspace_bytes": (_i64, [_i64, _i64, _i64, _i64]),
    "cq_mix_retention": (_int, [_vp, _vp, _vp, _i64, _vp, _vp, _vp, _i64, _i64, _i64, _i64, _i64, _i64, _vp, _i64, _vp]),
    "cq_mix_talk_merge_retention_step": (_int, [_vp, _i64, _i64, _i64, _i64, _i64, _f32, _vp, _vp, _heads, _i64, _i64, _vp, _vp, _i64, _i64, _f32, _f32,
                                                _vp, _vp, _i64, _vp]),
    "cq_mix_delta_prep": (_int, [_vp, _i64, _i64, _i64, _i64, _vp, _i64, _vp, _vp, _vp, _i64, _i64, _i64, _vp]),
    "cq_mix_delta_scan": (_int, [_vp, _vp, _i64, _vp, _vp, _i64, _i64, _i64, _i64, _vp]),
    "cq_mix_delta_step": (_int, [_vp, _i64, _i64, _i64, _i64, _i64, _i64, _vp, _i64, _i64, _vp, _vp, _vp, _vp, _vp, _i64, _i64, _f32, _vp]),
}
MIXER_SIGNATURES.update({
    "cq_mix_latent_pack": (_int, [_latent, _vp, _i64, _i64, _vp, _vp, _i64, _vp, _i64, _i64, _i64, _i64, _vp]),
    "cq_mix_latent_expanded": (_int, [_latent, _vp, _i64, _vp, _i64, _i64, _i64, _vp, _vp, _i64, _vp, _i64, _i64, _i64, _vp]),
    "cq_mix_latent_absorbed_workspace_bytes": (_i64, [_latent, _i64, _i64, _int]),
    "cq_mix_latent_absorbed": (_int, [_latent, _vp, _vp, _vp, _i64, _vp, _i64, _i64, _vp, _i64, _vp]),
    "cq_mix_latent_step": (_int, [_latent, _vp, _i64, _vp, _vp, _i64, _vp, _i64, _i64, _vp, _vp, _vp, _i64, _vp, _i64, _vp]),
    "cq_mix_moe_select": (_int, [_vp, _i64, _i64, _i64, _i64, _vp, _vp, _vp, _vp]),
    "cq_mix_moe_max_tiles": (_i64, [_i64, _i64, _i64, _i64]),
    "cq_mix_moe_plan": (_int, [_vp, _vp, _i64, _i64, _i64, _i64, _vp, _vp, _vp, _vp, _vp, _vp]),
    "cq_mix_moe_add": (_int, [_vp, _i64, _i64, _vp, _i64, _i64, _i64, _vp]),
    "cq_mix_moe_step_fits": (_int, [_moe]),
    "cq_mix_moe_step": (_int, [_moe, _vp, _int, _vp, _f32, _i64, _vp, _vp, _vp, _vp, _vp]),
})
# glue that the mixer library carries as well
_MIXER_GLUE = ("cq_status_string", "cq_nn_embedding", "cq_nn_argmax")

_lib = None


class CqError(RuntimeError):
    """A C-ABI entry point returned a non-zero status."""

    def __init__(self, fn: str, status: int, text: str):
        super().__init__(f"{fn} failed: {text} (status {status})")
        self.fn = fn
        self.status = status


def _load(path: str, signatures: dict) -> ctypes.CDLL:
    if not os.path.exists(path):
        raise ImportError(
            f"{path} is missing: build the HIP extension first (python -m candle_amd.build). "
            "There is no fallback path."
        )
    L = ctypes.CDLL(path)
    for name, (res, args) in signatures.items():
        fn = getattr(L, name)
        fn.restype = res
        fn.argtypes = args
    return L


def lib() -> ctypes.CDLL:
    global _lib
    if _lib is None:
        _lib = _load(LIB_PATH, SIGNATURES)
    return _lib


_mixer = None


def mixer_lib() -> ctypes.CDLL:
    """libcandle_hip_mixer.so: what models with bfloat16 weights and other sequence mixers run on, complete in itself."""
    global _mixer
    if _mixer is None:
        _mixer = _load(MIXER_LIB_PATH, {**MIXER_SIGNATURES, **{n: SIGNATURES[n] for n in _MIXER_GLUE}})
    return _mixer


BENCH_LIB_PATH = os.path.join(_HERE, "libcq_bench.so")
_bench = None


def bench_lib():
    """libcq_bench.so, the benchmark's plain-read yardstick kernel (candle_amd/csrc/cq_bench.hip): a measurement aid that is
    not part of the C ABI.  None when it has not been built."""
    global _bench
    if _bench is None and os.path.exists(BENCH_LIB_PATH):
        B = ctypes.CDLL(BENCH_LIB_PATH)
        B.cq_bench_read.restype = _int
        B.cq_bench_read.argtypes = [_vp, _i64, _vp, _vp]
        B.cq_bench_read_best.restype = _int
        B.cq_bench_read_best.argtypes = [_vp, _i64, _vp, _vp]
        _bench = B
    return _bench


def status_string(status: int) -> str:
    return (_lib or _mixer or lib()).cq_status_string(status).decode()


def check(fn: str, status: int) -> None:
    if status != 0:
        raise CqError(fn, status, status_string(status))
