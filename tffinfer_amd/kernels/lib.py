"""Loads the kernel library and declares its C entry points for ctypes."""
from __future__ import annotations

import ctypes
from ctypes import c_char_p, c_float, c_int, c_int64, c_size_t, c_void_p

from .build import ensure_built

ABI_VERSION = 37


class KernelLibraryError(RuntimeError):
    """The compiled kernels are missing, stale or failed to load."""


class KernelError(RuntimeError):
    """An entry point refused its arguments or a launch failed."""


_P, _I, _F, _Z = c_void_p, c_int, c_float, c_size_t


class Recurrence(ctypes.Structure):
    """``TffRecurrence`` of csrc/tffinfer_kernels.h, field by field."""
    _fields_ = ([(n, _P) for n in ("q", "k", "v", "gate")] + [("ld", _Z)]
                + [(n, _P) for n in ("a1", "a2", "a_bias", "ig", "fg", "i_bias", "f_bias", "w", "state")] + [("state_row", _Z)]
                + [(n, _P) for n in ("cu_tokens", "state_slots", "out")] + [("out_row", _Z)]
                + [(n, _I) for n in ("kind", "R", "H", "D", "E", "rank", "w_per_head", "sigmoid_gate", "out_dtype")]
                + [(n, _F) for n in ("inv_tau", "cap", "den_eps", "eps", "q_scale", "out_scale")])


#: ``Recurrence.kind``: a decay per key channel; exponential gates per head with a running maximum
LR_DECAY, LR_EXP = 0, 1

_SIGNATURES = {
    "tff_embed": [_P, _P, _P, _I, _I, _I, _I, _P],
    "tff_add_rmsnorm": [_P, _P, _I, _Z, _P, _F, _P, _P, _I, _I, _I, _P],
    "tff_rmsnorm": [_P, _P, _F, _P, _I, _I, _I, _P],
    "tff_gemm": [_P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _P, _F, _F, _F, _P, _Z, _I, _P],
    "tff_gemm_workspace_bytes": [_I, _I, _I, _I, _I, _I],
    "tff_gemm_plan": [_I, _I, _I, _I, _I, _P, _P, _P],
    "tff_gemm_residual_prenorm": [_P, _P, _I, _I, _I, _I, _P, _P, _P, _P, _I, _P],
    "tff_gemm_residual_dyt": [_P, _P, _I, _I, _I, _I, _P, _F, _P, _P, _P, _P],
    "tff_gemm_row_scaled": [_P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _I, _I, _I, _F, _F, _F, _F, _P],
    "tff_pack_weight": [_P, _P, _I, _I, _P],
    "tff_embed_packed": [_P, _P, _P, _I, _I, _I, _P],
    "tff_qk_norm_rope_kv": [_P, _I, _I, _I, _I, _P, _P, _F, _P, _I, _I, _I, _P, _P, _P, _P,
                            _I, _I, _I, _I, _P],
    "tff_attention_generic": [_P, _I, _P, _P, _P, _P, _I, _P, _P, _I, _I, _I, _I, _I, _I, _I,
                              _F, _P, _F, _P, _I, _I, _I, _I, _P],
    "tff_attention_mfma_supported": [_I, _I],
    "tff_attention_mfma": [_P, _I, _P, _P, _P, _P, _P, _P, _I, _P, _P, _P, _I, _P, _I, _I, _I, _I, _I, _I,
                           _I, _I, _I, _I, _I, _I, _F, _P, _F, _P, _I, _I, _P],
    "tff_attention_decode_fused": [_P, _I, _P, _P, _P, _P, _P, _P, _I, _P, _P, _P, _P, _P, _F, _P, _I, _I,
                                   _I, _I, _I, _I, _I, _I, _I, _I, _F, _P],
    "tff_attention_decode_runs": [_P, _I, _P, _P, _P, _P, _P, _P, _I, _P, _P, _P, _P, _P, _F, _P, _I, _I,
                                  _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _F, _P],
    "tff_attention_mfma_runs": [_P, _I, _P, _P, _P, _P, _P, _P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I,
                                _I, _F, _P, _F, _P],
    "tff_attention_decode_fused_static": [_P, _I, _P, _P, _P, _P, _I, _P, _P, _P, _P, _P, _F, _P, _I, _I,
                                          _I, _I, _I, _I, _I, _I, _I, _I, _F, _P],
    "tff_attention_split_reduce": [_P, _P, _P, _I, _I, _I, _I, _P, _I, _P, _P],
    "tff_latent_kv_store": [_P, _I, _I, _I, _I, _I, _I, _P, _F, _P, _I, _P, _P, _P, _P, _I, _I, _I, _P, _I, _I, _P, _P, _I,
                            _I, _I, _P],
    "tff_head_linear": [_P, _I, _I, _P, _P, _I, _I, _I, _I, _I, _I, _P, _I, _I, _I, _I, _I, _P, _I, _P, _I, _P],
    "tff_add_dyt": [_P, _P, _I, _Z, _P, _I, _Z, _F, _P, _P, _P, _P, _I, _I, _I, _P],
    "tff_diff_qkv_store": [_P, _Z, _P, _P, _P, _P, _I, _I, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _P],
    "tff_diff_combine": [_P, _Z, _I, _P, _Z, _F, _F, _F, _P, _Z, _I, _I, _I, _I, _P],
    "tff_scale_add_rmsnorm": [_P, _P, _I, _Z, _F, _P, _F, _P, _I, _I, _I, _P],
    "tff_gelu": [_P, _P, c_int64, _I, _I, _P],
    "tff_route_topk": [_P, _I, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _F, _P, _P, _P, _I, _P],
    "tff_experts_gate_up": [_P, _I, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F, _F, _F, _P, _P, _I, _P],
    "tff_experts_tiles_supported": [_I, _I, _I],
    "tff_experts_by_tiles": [_P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _F, _F, _F, _P, _P, _P, _I, _P, _P, _I, _I, _P],
    "tff_group_rmsnorm_add": [_P, _P, _I, _Z, _P, _P, _I, _F, _P, _I, _I, _I, _P],
    "tff_depth_average": [_P, _Z, _I, _P, _P, _P, _Z, _I, _P],
    "tff_scale_rows": [_P, _F, _Z, _P],
    "tff_token_shift_mix": [_P, _P, _Z, _Z, _P, _I, _P, _P, _P, _P, _I, _I, _I, _P],
    "tff_wkv_recurrence": [_P, _P, _P, _P, _Z, _P, _P, _P, _Z, _P, _P, _P, _I, _I, _I, _P, _I, _Z, _I, _P],
    "tff_head_norm_gate": [_P, _P, _Z, _P, _F, _P, _I, _I, _I, _I, _P],
    "tff_tanh": [_P, _P, _Z, _I, _P],
    "tff_gdelta_prep": [_P, _Z, _P, _I, _P, _P, _P, _Z, _Z, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P],
    "tff_gdelta_recurrence": [_P, _P, _Z, _P, _Z, _Z, _I, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P],
    "tff_head_norm_silu_gate": [_P, _P, _Z, _P, _F, _F, _P, _Z, _I, _I, _I, _I, _P],
    "tff_sigmoid_gate_heads": [_P, _Z, _I, _P, _Z, _F, _P, _Z, _I, _I, _I, _I, _P],
    "tff_add_rmsnorm_pair": [_P, _P, _I, _Z, _P, _I, _Z, _P, _P, _P, _F, _P, _P, _P, _I, _I, _I, _P],
    "tff_softcap": [_P, _Z, _F, _P],
    "tff_route_by_table": [_P, _P, _I, _I, _I, _I, _P, _P, _P],
    "tff_qk_bias_norm_store": [_P, _Z, _P, _P, _F, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P],
    "tff_mixed_attention_supported": [_I, _I, _I],
    "tff_mixed_attention": [_P, _P, _P, _P, _I, _P, _P, _P, _I, _P, _F, _F, _I, _I, _I, _P, _I, _I, _I, _I, _I, _I, _I, _P, _I, _P],
    "tff_mixed_attention_workspace_bytes": [_I, _I, _I, _I],
    "tff_mixed_attention_q16_supported": [_I, _I, _I, _I],
    "tff_mixed_attention_q16": [_P, _P, _P, _P, _I, _P, _P, _P, _I, _P, _I, _P, _F, _F, _I, _I, _I, _P, _I, _I, _I, _I, _I, _I, _I, _P, _P],
    "tff_experts_down": [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _I, _I, _P, _I, _P],
    "tff_swiglu": [_P, _P, _P, _I, _I, _F, _F, _F, _I, _P],
    "tff_cast": [_P, _I, _P, _I, c_int64, _P],
    "tff_argmax_workspace_bytes": [_I, _I],
    "tff_argmax": [_P, _P, _I, _I, _P, _P],
    "tff_repetition_penalty": [_P, _I, _I, _P, _P, _P, _P],
    "tff_sample": [_P, _P, _I, _I, _P, _P, _P, _P, _P, _P, _P],
    "tff_add_layernorm": [_P, _P, _I, _Z, _P, _I, _Z, _P, _P, _P, _F, _P, _P, _P, _F, _P, _P, _P, _F, _P, _P, _I, _I, _P, _I, _P, _Z,
                          _Z, _P, _P, _Z, _I, _P],
    "tff_input_conv": [_P, _P, _I, _P, _Z, _Z, _P, _I, _I, _P, _P, _P, _I, _I, _P],
    "tff_lightning": [_P, _Z, _P, _P, _Z, _P, _P, _P, _I, _I, _I, _I, _P],
    "tff_lightning_chunk": [],
    "tff_lightning_chunks": [_P, _Z, _P, _P, _Z, _P, _P, _I, _P, _P, _P, _P, _I, _I, _I, _I, _P],
    "tff_row_norm_gate": [_P, _P, _Z, _P, _F, _P, _I, _I, _I, _P],
    "tff_grouped_qkv_store": [_P, _Z, _P, _I, _I, _I, _F, _I, _P, _P, _P, _F, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _P],
    "tff_pool_keys": [_P, _P, _P, _I, _P, _I, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P],
    "tff_gate_heads": [_P, _Z, _I, _P, _Z, _F, _P, _Z, _I, _I, _I, _I, _P],
    "tff_recurrence_few": [_P, _I, _P],
    "tff_recurrence_chunk": [],
    "tff_recurrence_workspace_bytes": [_I, _I, _I, _I, _I, _I],
    "tff_recurrence_chunks": [_P, _I, _P, _P, _I, _P, _Z, _P],
    "tff_bigram_embed": [_P, _I, _I, _P, _P, _P, _P, _P, _P, _P, _Z, c_int64, c_int64, c_int64, _P, _P, _I, _I, _I, _I, _P],
    "tff_probe_stream_read": [_P, _Z, _P, _I, _P],
    "tff_probe_mfma": [_P, _I, _I, _I, _P],
}

_lib = None


def load() -> ctypes.CDLL:
    """The library, built on first use if the tree holds none for these sources."""
    global _lib
    if _lib is not None:
        return _lib
    try:
        path = ensure_built()
        lib = ctypes.CDLL(path)
    except Exception as e:  # build errors, missing hipcc, dlopen errors
        raise KernelLibraryError(
            f"the HIP kernel library could not be built or loaded: {e}\n"
            "There is no fallback path; build it with `python -c 'import __graft_entry__ as g; g.build()'`."
        ) from e
    lib.tff_last_error.restype = c_char_p
    lib.tff_last_error.argtypes = []
    lib.tff_abi_version.restype = c_int
    if lib.tff_abi_version() != ABI_VERSION:
        raise KernelLibraryError(
            f"{path} has ABI {lib.tff_abi_version()}, the package expects {ABI_VERSION}; rebuild it")
    for name, args in _SIGNATURES.items():
        fn = getattr(lib, name)
        fn.argtypes = args
        fn.restype = c_size_t if name.endswith("_bytes") else c_int
    _lib = lib
    return lib


def check(rc: int) -> None:
    if rc != 0:
        raise KernelError(load().tff_last_error().decode())
