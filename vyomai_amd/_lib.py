"""ctypes binding of libvyom_hip.so (C ABI in include/vyom_hip.h).

The library is built in-tree by ``__graft_entry__.build()`` (hipcc, gfx950) into
``vyomai_amd/lib/``.  There is no fallback: if it is missing or a call fails, the op raises.
"""
from __future__ import annotations

import ctypes as C
import os
from typing import Optional

_HERE = os.path.dirname(os.path.abspath(__file__))
# VY_LIB_PATH: developer knob for A/B runs of two builds of the same ABI on one box (tools/ab_lib.sh)
LIB_PATH = os.environ.get("VY_LIB_PATH") or os.path.join(_HERE, "lib", "libvyom_hip.so")

VY_F32, VY_BF16 = 0, 1
ACT_NONE, ACT_GELU_ERF, ACT_GELU_TANH, ACT_SILU, ACT_RELU2 = 0, 1, 2, 3, 4
ACT_SAVE_DERIV = 0x100   # saved tensor = act'(pre) instead of pre (include/vyom_hip.h)
MOE_CLAMPED, MOE_GELU = 0, 1
SCORE_SOFTMAX, SCORE_SIGMOID = 0, 1
MASK_NONE, MASK_CAUSAL, MASK_KEYPAD, MASK_ADDITIVE = 0, 1, 2, 4

_p, _i64, _i, _f, _u64 = C.c_void_p, C.c_int64, C.c_int, C.c_float, C.c_uint64

# name -> argtypes, exactly the prototypes of include/vyom_hip.h
PROTOTYPES = {
    "vy_linear_fwd": [_p, _i64, _p, _i64, _p, _p, _i64, _p, _i64, _p, _i64, _i64, _i64, _i, _i, _p],
    "vy_linear_softcap_fwd": [_p, _i64, _p, _i64, _p, _i64, _i64, _i64, _i64, _f, _i, _p],
    "vy_qkv_rope_fwd": [_p, _i64, _p, _i64, _p, _p, _p, _i64,
                        _p, _i64, _i64, _i64, _p, _i64, _i64, _i64, _p, _i64, _i64, _i64,
                        _i64, _i64, _i64, _i, _i, _i, _i, _p],
    "vy_attn_fwd": [_p, _i64, _i64, _i64, _p, _i64, _i64, _i64, _p, _i64, _i64, _i64,
                    _p, _i64, _i64, _p, _i, _i64, _p, _i64, _p, _i64, _i64,
                    _i64, _i, _i, _i64, _i64, _i, _f, _i, _p],
    "vy_attn_decode": [_p, _i64, _i64, _p, _i64, _i64, _i64, _p, _i64, _i64, _i64,
                       _p, _i64, _i64, _i, _i, _i64, _i, _f, _i, _p],
    "vy_layernorm_fwd": [_p, _i64, _p, _p, _p, _i64, _p, _p, _i64, _i64, _f, _i, _p],
    "vy_rmsnorm_fwd": [_p, _i64, _p, _p, _i64, _i64, _i64, _f, _f, _i, _p],
    "vy_gated_act_fwd": [_p, _i64, _p, _i64, _i64, _i64, _i, _i, _p],
    "vy_rope_fwd": [_p, _i64, _i64, _i64, _p, _p, _i64, _i64, _i, _i64, _i, _i, _i, _p],
    "vy_linear_dgrad": [_p, _i64, _p, _i64, _p, _i64, _i, _p, _i64, _p, _i64, _p, _i64, _i64, _i64, _i64, _i, _p],
    "vy_linear_wgrad": [_p, _i64, _p, _i64, _p, _i64, _p, _f, _p, _i64, _i64, _i64, _i, _p],
    "vy_linear_wgrad_grouped": [_p, _i, _i, _p],
    "vy_layernorm_bwd": [_p, _i64, _p, _i64, _p, _p, _p, _p, _i64, _p, _p, _f, _p, _i64, _i64, _i, _p],
    "vy_attn_bwd": [_p, _i64, _i64, _i64, _p, _i64, _i64, _i64, _p, _i64, _i64, _i64,
                    _p, _p, _i64, _i64, _p, _p,
                    _p, _i64, _i64, _i64, _p, _i64, _i64, _i64, _p, _i64, _i64, _i64,
                    _i, _i64, _p, _i64, _p, _p, _i64, _i64, _i, _i, _i64, _i64, _i, _f, _i, _p],
    "vy_adamw_step": [_p, _p, _p, _p, _p, _i64, _f, _f, _f, _f, _f, _i64, _f, _p, _p],
    "vy_adamw_step_gated": [_p, _p, _p, _p, _p, _i64, _f, _f, _f, _f, _f, _i64, _f, _p, _p, _p],
    "vy_sumsq": [_p, _i64, _p, _p, _p],
    "vy_linear_dropout_fwd": [_p, _i64, _p, _i64, _p, _p, _i64, _p, _i64, _i64, _i64, _i64, _f, _u64, _u64, _i, _p],
    "vy_dropout": [_p, _i64, _p, _i64, _i64, _i64, _f, _u64, _u64, _i, _p],
    "vy_act_bwd": [_p, _i64, _p, _i64, _p, _i64, _i64, _i64, _i, _i, _p],
    "vy_xent_fwd": [_p, _i64, _p, _i64, _p, _p, _p, _i64, _i64, _p, _i, _p],
    "vy_xent_bwd": [_p, _i64, _p, _i64, _p, _p, _p, _i64, _i64, _i, _p],
    "vy_xent_fused": [_p, _i64, _p, _i64, _p, _p, _p, _p, _i64, _i64, _p, _i, _p],
    "vy_transpose_batched": [_p, _i, _i, _i, _p],
    "vy_embedding_fwd": [_p, _i64, _p, _p, _i64, _i64, _i64, _i64, _p, _i, _p],
    "vy_embedding_bwd": [_p, _i64, _p, _p, _i64, _i64, _i64, _i64, _i64, _i, _p],
    "vy_transpose": [_p, _i64, _p, _i64, _i64, _i64, _i, _p],
    "vy_greedy_step": [_p, _i64, _i64, _i64, _i, _p, _i64, _i64, _p, _i64, _p, _i, _p, _p, _p],
    "vy_sampling_probs": [_p, _i64, _i64, _i64, _i, _f, _i, _f, _p, _i64, _p],
    "vy_decoder_step": [_p, _p, _i64, _p, _p, _p, _i64, _p],
    "vy_gemma_decoder_step": [_p, _p, _i64, _p, _i64, _p],
    "vy_residual_norm": [_p, _i64, _p, _i64, _p, _i64, _p, _i64, _p, _p, _f, _p, _f, _p, _i64, _i64, _i64, _i64, _i, _i, _p],
    "vy_residual_norm_routed": [_p, _i64, _p, _i64, _p, _i64, _p, _i64, _p, _f, _p, _p, _f, _p, _f, _p, _i64, _i64, _i64, _i64, _i,
                                _i, _p],
    "vy_latent_norm": [_p, _i64, _p, _p, _i64, _i, _i, _p, _p, _i64, _i, _i, _p, _i64, _i64, _i, _i, _p, _p, _p, _i64, _i64, _f,
                       _i, _p],
    "vy_rmsnorm_gate": [_p, _i64, _p, _p, _i64, _p, _i64, _i64, _i64, _i64, _f, _i, _p],
    "vy_head_norm_gate": [_p, _i64, _p, _p, _i64, _p, _i64, _i64, _i, _i64, _i64, _f, _i, _p],
    "vy_attn_fwd_ex": [_p, _i64, _i64, _i64, _p, _i64, _i64, _i64, _p, _i64, _i64, _i64, _p, _i64, _i64, _p, _i64, _i64,
                       _p, _p, _i64, _i, _i, _i64, _i64, _i, _i, _f, _p, _i, _p],
    "vy_latent_decode": [_p, _i64, _p, _p, _p, _i64, _i64, _p, _p, _i64, _p, _i64, _p, _i64, _i, _i, _i, _i, _i, _i, _i, _f, _p, _i64,
                         _i, _p],
    "vy_gated_attn": [_p, _i64, _i64, _i64, _i64, _p, _p, _p, _p, _p, _p, _p, _i64, _i64, _i64, _i, _i, _i, _i, _p, _i64, _i, _p],
    "vy_diff_attn_fwd": [_p, _i64, _p, _i64, _i64, _i, _p, _p, _p, _p, _p, _i64, _i64, _i64, _i, _i, _i, _i, _f, _i, _p],
    "vy_decay_attn": [_p, _i64, _i64, _i64, _i64, _p, _p, _p, _p, _p, _p, _i64, _i64, _i64, _i, _i, _i, _i, _p, _i, _i, _f, _p, _i64,
                      _i, _p],
    "vy_window_rows": [_p, _i64, _i64, _i64, _p, _i64, _i64, _i, _i, _p, _i, _i, _i, _i, _p, _p, _p, _i64, _i64, _i, _i, _i, _i, _p],
    "vy_qkv_rows": [_p, _i64, _i64, _i64, _i64, _p, _p, _i64, _i64, _i, _i, _p, _i, _i, _i, _p, _p, _p, _i64, _i64, _i, _i, _i, _i, _i,
                    _p],
    "vy_window_context": [_p, _i64, _i64, _i64, _p, _i64, _i64, _i, _i, _p, _i, _i, _p, _p, _i64, _i64, _i, _i, _i, _i, _p],
    "vy_window_decode": [_p, _i64, _i64, _i64, _i64, _i64, _p, _i64, _i64, _i, _i, _p, _i, _i, _p, _p, _p, _p, _i64, _p, _i64, _i64, _i, _i,
                         _i, _i, _f, _i, _p, _i64, _i, _p],
    "vy_moe_fwd": [_p, _p, _i64, _i64, _p, _i64, _p, _i64, _p, _p, _p, _p, _i64, _i, _p],
    "vy_clamped_act_fwd": [_p, _i64, _p, _i64, _i64, _i64, _f, _f, _i, _p],
    "vy_hybrid_decoder_step": [_p, _p, _p, _p, _i64, _p, _i64, _p],
    "vy_cast": [_p, _p, _i64, _i, _i, _p],
    "vy_ddp_unique_id": [_p],
    "vy_ddp_init": [_p, _i, _i],
    "vy_ddp_all_reduce_async": [_p, _i64, _i, _p],
    "vy_ddp_destroy": [],
    "vy_set_concurrent_chains": [_i],
    "vy_workspace_set": [_p, _p, _i64],
}
OTHER_SYMBOLS = ["vy_last_error", "vy_abi_version", "vy_layernorm_bwd_ws_rows", "vy_decode_ws_bytes",
                 "vy_gemma_ws_bytes", "vy_ddp_world", "vy_ddp_rank", "vy_latent_decode_ws_bytes", "vy_decay_attn_ws_bytes",
                 "vy_hybrid_ws_bytes", "vy_window_decode_ws_bytes", "vy_moe_ws_bytes", "vy_gated_attn_ws_bytes"]
DECAY_CHUNK = 64   # VY_DECAY_CHUNK
ALL_SYMBOLS = list(PROTOTYPES) + OTHER_SYMBOLS


class VyWgradDesc(C.Structure):
    """vy_wgrad_desc of include/vyom_hip.h."""
    _fields_ = [("dy", _p), ("lddy", _i64), ("x", _p), ("ldx", _i64), ("dw", _p), ("lddw", _i64), ("db", _p),
                ("M", _i64), ("N", _i64), ("K", _i64)]


class VyAttnWindow(C.Structure):
    """vy_attn_window of include/vyom_hip.h."""
    _fields_ = [(n, C.c_int32) for n in ("window", "sink", "kv_by_slot", "start_cap")] + \
               [("rope", _p), ("rope_dims", C.c_int32), ("rope_len", C.c_int32), ("keep", C.c_int32), ("gate_heads", C.c_int32)]


class VyQkvPrep(C.Structure):
    """vy_qkv_prep of include/vyom_hip.h."""
    _fields_ = [("q_norm", _p), ("k_norm", _p), ("n_q", C.c_int32), ("n_k", C.c_int32), ("eps", C.c_float), ("lambda_", C.c_float),
                ("v_mix", _p), ("ldm", _i64), ("n_v", C.c_int32), ("m_v", C.c_int32), ("m_vp", C.c_int32), ("v_out", _p), ("ldo", _i64),
                ("group", C.c_int32), ("temp_every", C.c_int32), ("temp_coef", C.c_float)]


class VyDiff(C.Structure):
    """vy_diff of include/vyom_hip.h."""
    _fields_ = [("lambda_", C.c_float), ("out_scale", C.c_float), ("eps", C.c_float), ("n_v", C.c_int32)]


class VyRoutedRows(C.Structure):
    """vy_routed_rows of include/vyom_hip.h."""
    _fields_ = [("rows", _p), ("ld", _i64), ("pos", _p), ("weight", _p), ("top", C.c_int32)]


class VyMoe(C.Structure):
    """vy_moe of include/vyom_hip.h."""
    _fields_ = [(n, C.c_int32) for n in ("experts", "top", "groups", "keep", "width", "ff", "act", "score", "group_best",
                                         "normalize")] + \
               [(n, C.c_float) for n in ("scale", "limit", "alpha")] + [(n, _p) for n in ("w_router", "w_gu", "w_down")]


class VyomHipError(RuntimeError):
    pass


_lib: Optional[C.CDLL] = None


def load() -> C.CDLL:
    """Load the kernel library; raise loudly when it has not been built."""
    global _lib
    if _lib is not None:
        return _lib
    if not os.path.exists(LIB_PATH):
        raise VyomHipError(
            f"{LIB_PATH} is missing: build it with `python -c 'import __graft_entry__ as g; g.build()'` "
            "(hipcc --offload-arch=gfx950).  vyomai_amd has no CPU or PyTorch fallback."
        )
    lib = C.CDLL(LIB_PATH)
    for name, argtypes in PROTOTYPES.items():
        fn = getattr(lib, name)
        fn.argtypes = argtypes
        fn.restype = C.c_int
    lib.vy_last_error.restype = C.c_char_p
    lib.vy_last_error.argtypes = []
    lib.vy_abi_version.restype = C.c_int
    lib.vy_layernorm_bwd_ws_rows.restype = C.c_int64
    lib.vy_layernorm_bwd_ws_rows.argtypes = [_i64]
    lib.vy_decode_ws_bytes.restype = C.c_int64
    lib.vy_decode_ws_bytes.argtypes = [C.c_int32] * 7
    for name, argtypes in (("vy_latent_decode_ws_bytes", [_i, _i, _i]),
                           ("vy_decay_attn_ws_bytes", [_i64, _i64, _i, _i, _i, _i]), ("vy_hybrid_ws_bytes", [_p]),
                           ("vy_window_decode_ws_bytes", [_i, _i, _i, _i, _i, _i]), ("vy_moe_ws_bytes", [_p, _i64, _i]),
                           ("vy_gated_attn_ws_bytes", [_i64, _i64, _i, _i, _i, _i])):
        getattr(lib, name).restype = C.c_int64
        getattr(lib, name).argtypes = argtypes
    _lib = lib
    return lib


def call(name: str, *args) -> None:
    lib = load()
    rc = getattr(lib, name)(*args)
    if rc != 0:
        raise VyomHipError(f"{name} failed ({rc}): {lib.vy_last_error().decode()}")


def dtype_code(torch_dtype) -> int:
    import torch

    if torch_dtype == torch.bfloat16:
        return VY_BF16
    if torch_dtype == torch.float32:
        return VY_F32
    raise VyomHipError(f"vyomai_amd kernels support float32 and bfloat16, got {torch_dtype}")
