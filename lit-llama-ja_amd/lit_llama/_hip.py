"""ctypes binding of the in-tree HIP library `_lljamd.so` (C ABI: include/lit_llama_amd.h).

The library is the only compute path of this package: there is no CPU or eager-PyTorch
fallback. If it is missing or the device is not a ROCm GPU, calls raise.
"""
from __future__ import annotations

import ctypes
import os
from pathlib import Path

import torch

# LLJ_LIB: another build of the same library (experiment variants built by _build.build(out=...,
# defines=...)); the product loads the in-tree _lljamd.so
LIB_PATH = Path(os.environ["LLJ_LIB"]) if os.environ.get("LLJ_LIB") else Path(__file__).resolve().parent / "_lljamd.so"

_P = ctypes.c_void_p
_I = ctypes.c_int
_F = ctypes.c_float
_U64 = ctypes.c_ulonglong


# name -> argtypes (every function returns int: 0 ok, hipError_t, or 1000 = EINVAL)
SIGNATURES = {
    "llj_w4_repack": [_P, _P, _I, _I, _P],
    "llj_w4_unpack": [_P, _P, _I, _I, _P],
    "llj_w4_scale_zero": [_P, _P, _I, _P, _I, _P],
    "llj_w8_repack": [_P, _P, _I, _I, _P],
    "llj_w8_unpack": [_P, _P, _I, _I, _P],
    "llj_i8_repack": [_P, _P, _I, _I, _P],
    "llj_i8_unpack": [_P, _P, _I, _I, _P],
    "llj_w8_scale_zero": [_P, _P, _I, _P, _I, _P],
    "llj_linear": [_I, _P, _I, _P, _P, _P, _P, _I, _I, _I, _I, _P, _I, _P, _P],
    "llj_norm_qkv_rope": [_I, _P, _P, _F, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P, _P, _P, _I,
                          _P],
    "llj_attention_split": [_P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _P],
    "llj_gemm_i8_linear": [_P, _I, _P, _P, _P, _P, _P, _I, _P, _I, _I, _I, _I, _P],
    "llj_gemm_i8_resid": [_P, _I, _P, _P, _P, _P, _P, _I, _P, _I, _I, _I, _I, _P],
    "llj_gemm_i8_silu_mul": [_P, _I, _P, _P, _P, _P, _P, _I, _P, _I, _I, _I, _I, _P],
    "llj_gemm_i8_qkv_rope": [_P, _P, _P, _P, _P, _P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P],
    "llj_i8_gather_act": [_P, _I, _I, _I, _P, _P, _I, _P],
    "llj_i8_gather_weight": [_P, _P, _I, _I, _P, _P, _I, _P],
    "llj_gptq_block": [_P, _I, _I, _P, _I, _P, _P, _I, _P, _P, _P, _P],
    "llj_gptq_block_bs": [_P, _I, _I, _I, _P, _I, _P, _P, _I, _P, _P, _P, _P],
    "llj_colblock_pack": [_P, _I, _I, _P, _P, _I, _P, _P],
    "llj_attention": [_P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P],
    "llj_attention_prefill": [_P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P],
    "llj_linear_resid": [_I, _P, _I, _P, _P, _P, _I, _I, _I, _I, _P, _I, _P, _P],
    "llj_linear_resid_attn": [_I, _P, _I, _I, _P, _P, _P, _I, _I, _I, _P, _P],
    "llj_attention_part": [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _P],
    "llj_norm_swiglu": [_I, _P, _P, _F, _P, _P, _P, _P, _P, _I, _I, _I, _P, _I, _P, _P, _I, _P],
    "llj_norm_linear": [_I, _P, _P, _F, _P, _P, _P, _I, _I, _I, _I, _P, _I, _P, _P, _I, _P],
    "llj_i8_stats": [_P, _I, _I, _I, _F, _P, _P],
    "llj_i8_norm_stats": [_P, _P, _F, _P, _I, _I, _F, _P, _P],
    "llj_i8_quant_weight": [_P, _I, _P, _P, _I, _I, _P],
    "llj_embedding": [_P, _P, _P, _I, _I, _P, _P],
    "llj_rmsnorm": [_P, _P, _F, _P, _I, _I, _P],
    "llj_rmsnorm_rows": [_P, _P, _F, _P, _P, _I, _I, _P],
    "llj_argmax": [_P, _I, _I, _I, _P, _P, _I, _P, _P],
    "llj_sample": [_P, _I, _I, _I, _F, _I, _P, ctypes.c_ulonglong, _P, _P, _I, _P, _P],
    "llj_set_tpw_max": [_I],
    "llj_set_stream_a": [_I],
    "llj_set_option": [_I, _I],
    "llj_attention_i8": [_P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _P, _P, _I, _F, _P],
    "llj_i8_swiglu_stats": [_P, _P, _P, _P, _P, _P, _I, _I, _I, _P, _P, _P, _P, _I, _F, _P],
    "llj_i8_norm_rowstats": [_P, _P, _F, _P, _I, _I, _F, _P, _P, _P],
    "llj_i8_linear_resid": [_P, _I, _P, _P, _P, _I, _I, _I, _I, _P, _P],
    "llj_gemm_linear": [_I, _P, _I, _P, _P, _P, _I, _I, _I, _I, _P],
    "llj_gemm_resid": [_I, _P, _I, _P, _P, _P, _I, _I, _I, _I, _P],
    "llj_gemm_silu_mul": [_I, _P, _I, _P, _P, _P, _I, _I, _I, _I, _P],
    "llj_gemm_swiglu": [_I, _P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _P],
    "llj_gemm_swiglu_ws": [_I, _P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _P, ctypes.c_size_t, _P],
    "llj_gemm_resid_ws": [_I, _P, _I, _P, _P, _P, _I, _I, _I, _I, _P, ctypes.c_size_t, _P],
    "llj_gemm_qkv_rope": [_I, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P],
    "llj_stream_read": [_P, ctypes.c_size_t, _P, _I, _P],
    "llj_g_embedding": [_P, _P, _P, _I, _I, _P, _I, _P],
    "llj_g_rmsnorm": [_P, _I, _P, _F, _P, _I, _I, _I, _I, _P],
    "llj_g_linear": [_I, _P, _I, _I, _I, _P, _P, _P, _I, _I, _I, _P, _I, _P, _I, _I, _P],
    "llj_g_rope_kv": [_P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P],
    "llj_g_attention": [_P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P],
    "llj_g_silu_mul": [_P, _P, _P, ctypes.c_size_t, _I, _P],
    "llj_g_argmax": [_P, _I, _I, _I, _P, _P, _I, _P, _P],
    "llj_g_sample": [_P, _I, _I, _I, _F, _I, _P, ctypes.c_ulonglong, _P, _P, _I, _P, _P],
    "llj_next_token": [_P, _I, _I, _I, _F, _I, _P, _U64, _P, _P, _I, _P, _I, _I, _P],
    "llj_bigram_embed": [_P, _P, _I, _P, _I, _I, _U64, _U64, _P, _F, _P, _P, _P, _P, _P, _P, _I, _P, _I, _I, _I, _I, _P],
    "llj_post_norm": [_P, _I, _P, _F, _P, _I, _P, _I, _P, _P, _I, _I, _I, _P],
    "llj_g_relu2": [_P, ctypes.c_size_t, _I, _P],
    "llj_gla_scan": [_P, _I, _I, _I, _I, _I, _I, _P, _I, _P, _I, _P, _P, _I, _P, _P, _P, _I, _I, _I, _I, _F, _F, _F, _I,
                     _P],
    "llj_rows_linear": [_I, _P, _I, _P, _P, _P, _I, _I, _I, _I, _F, _F, _P],
    "llj_post_linear": [_I, _P, _P, _F, _P, _P, _I, _P, _P, _I, _I, _P],
    "llj_gemm_bf16": [_I, _P, _I, _P, _P, _P, _I, _I, _I, _I, _F, _F, _P, ctypes.c_size_t, _P],
    "llj_gla_chunk_rows": [_I, _I],
    "llj_gla_chunks": [_P, _I, _I, _I, _I, _I, _I, _P, _I, _P, _I, _P, _P, _I, _P, _P, _P, _I, _P, _I, _P, _P, _I, _I, _I,
                       _F, _F, _F, _I, _P],
    "llj_latent_flash_ok": [_I, _I, _I],
    "llj_latent_flash": [_P, _I, _I, _I, _P, _I, _I, _P, _I, _I, _P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F,
                         _P],
    "llj_latent_gather": [_P, _P, _I, _I, _P, _P, _P, _P, _I, _P],
    "llj_latent_decode_ok": [_I, _I, _I, _I],
    "llj_latent_decode": [_P, _I, _I, _I, _I, _P, _P, _P, _P, _P, _P, _P, _I, _I, _P, _P, _I, _P, _I, _I, _I, _I, _I, _I,
                          _I, _I, _I, _F, _F, _P],
    "llj_latent_prep": [_P, _I, _I, _I, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _P],
    "llj_latent_commit": [_P, _P, _I, _I, _P, _P, _P, _P, _I, _I, _P],
    "llj_prev_commit": [_P, _P, _P, _P, _I, _P],
    "llj_latent_rows": [_P, _I, _I, _I, _P, _I, _P, _I, _P, _P, _I, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I,
                        _I, _I, _F, _I, _P],
    "llj_g_bias_act": [_I, _P, _I, _P, _P, _I, _I, _I, _F, _F, _I, _P],
    "llj_streams_embed": [_P, _P, _I, _F, _P, _P, _I, _I, _P, _P, _F, _P, _I, _I, _I, _I, _P],
    "llj_streams_step": [_P, _I, _P, _P, _P, _I, _I, _P, _P, _F, _P, _I, _P, _I, _I, _I, _P],
    "llj_streams_linear_ok": [_I, _I],
    "llj_streams_linear": [_I, _P, _P, _P, _P, _P, _I, _I, _P, _P, _F, _I, _P, _P, _P, _I, _I, _F, _F, _P],
    "llj_gqa_prep": [_P, _I, _I, _I, _I, _P, _I, _I, _F, _P, _P, _P, _P, _I, _I, _P, _P, _I, _I, _I, _I, _I, _I, _I,
                     _P],
    "llj_gqa_rows": [_P, _I, _I, _I, _P, _P, _P, _P, _I, _I, _P, _I, _I, _I, _I, _I, _I, _F, _I, _I, _P],
    "llj_gqa_flash_rows": [_I, _I, _I],
    "llj_gqa_flash": [_P, _I, _I, _I, _P, _I, _I, _P, _P, _P, _I, _I, _P, _I, _I, _I, _I, _I, _I, _F, _I, _P],
    "llj_gqa_decode_ok": [_I, _I],
    "llj_gqa_part_width": [_I],
    "llj_gqa_decode": [_P, _I, _I, _I, _I, _I, _P, _I, _I, _F, _P, _P, _P, _I, _I, _P, _P, _I, _P, _P, _I, _P, _I, _I,
                       _I, _I, _I, _I, _F, _I, _P],
    "llj_g_i8_linear": [_P, _I, _I, _I, _P, _P, _F, _P, _I, _P, _I, _P, _I, _I, _P],
}

# workspace sizes (host functions)
SIZE_SIGNATURES = {
    "llj_i8_ws_bytes": [_I, _I],
    "llj_attention_ws_bytes": [_I, _I, _I, _I],
    "llj_g_i8_ws_bytes": [_I, _I],
    "llj_i8_rowstats_bytes": [_I],
    "llj_gemm_resid_ws_bytes": [_I, _I, _I, _I],
    "llj_gemm_swiglu_ws_bytes": [_I, _I, _I, _I],
    "llj_gemm_bf16_ws_bytes": [_I, _I, _I],
}

_lib = None


class HipError(RuntimeError):
    pass


# llj_set_option indices (include/lit_llama_amd.h LLJ_OPT_*)
WF_I8_ROWSTATS = 0x10000  # wfmt flag: i8ws is a decode hand-off block (include/lit_llama_amd.h)
WF_ZINT = 0x20000  # prefill GEMM wfmt flag: int4 whose zeros are all integers (include/lit_llama_amd.h)
(OPT_ATT_SPEC_FULL, OPT_FLASH_QB, OPT_FLASH_PAIR, OPT_GEMM_GLDS, OPT_GLDS_COST128, OPT_GEMV_LDS_A_KB,
 OPT_ATT_SPEC_BATCH, OPT_GEMM_W4Z) = range(8)


def lib() -> ctypes.CDLL:
    global _lib
    if _lib is None:
        if not LIB_PATH.exists():
            raise HipError(
                f"{LIB_PATH} is missing: build it with `python -c 'import __graft_entry__ as g; g.build()'` "
                "(hipcc --offload-arch=gfx950). There is no fallback path.")
        L = ctypes.CDLL(str(LIB_PATH))
        part = LIB_PATH.name.startswith("_lljamd_")  # a model's own sources only: some entry points are absent
        for name, argt in SIGNATURES.items():
            if part and not hasattr(L, name):
                continue
            f = getattr(L, name)
            f.argtypes = argt
            f.restype = ctypes.c_int
        for name, argt in SIZE_SIGNATURES.items():
            if part and not hasattr(L, name):
                continue
            f = getattr(L, name)
            f.argtypes = argt
            f.restype = ctypes.c_size_t
        _lib = L
    return _lib


def require(stems=None) -> None:
    """Make a library available that holds these csrc/ sources (None: all): the built one, or in a checkout
    without it one compiled from those sources alone."""
    global LIB_PATH
    if _lib is not None or LIB_PATH.exists():
        return
    from . import _build

    LIB_PATH = _build.build() if stems is None else _build.build_part(stems)


def call(name: str, *args) -> None:
    rc = getattr(lib(), name)(*args)
    if rc != 0:
        what = "unsupported shape/argument (EINVAL)" if rc == 1000 else f"hipError {rc}"
        raise HipError(f"{name} failed: {what}")


def stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def require_device(t: torch.Tensor, what: str = "tensor") -> None:
    if t.device.type != "cuda" or torch.version.hip is None:
        raise HipError(
            f"{what} is on {t.device}: this package runs only on a ROCm GPU (MI355X / gfx950); "
            "it has no CPU path")


def ptr(t) -> int | None:
    return None if t is None else t.data_ptr()
