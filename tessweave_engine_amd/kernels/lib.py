"""ctypes binding of the HIP kernel library. There is no fallback: a missing GPU or library is an error."""
from __future__ import annotations

import ctypes
from ctypes import c_int, c_long, c_float, c_void_p, c_uint64

from . import build as _build

_lib = None

P, I, L, F = c_void_p, c_int, c_long, c_float

_SIGNATURES = {
    "tw_error_string": (ctypes.c_char_p, [I]),
    "tw_abi_version": (I, []),
    "tw_graph_begin": (I, [P]),
    "tw_graph_end": (I, [P, ctypes.POINTER(c_void_p)]),
    "tw_graph_launch": (I, [P, P]),
    "tw_graph_destroy": (I, [P]),
    "tw_probe_read": (I, [P, L, P, I, ctypes.POINTER(c_long), P]),
    "tw_upload_words": (I, [P, P, I, ctypes.POINTER(c_int), ctypes.POINTER(c_int), P]),
    "tw_embed_gather": (I, [I, P, P, P, I, I, I, P, I, P]),
    "tw_rmsnorm": (I, [I, P, P, P, P, I, I, F, P, I, L, P, P]),
    "tw_rope_table": (I, [P, P, P, P, P, I, I, F, P]),
    "tw_rope_kv_write": (I, [I, P, L, P, P, P, P, P, I, I, I, I, I, I, I, P, I, P, I, P]),
    "tw_silu_mul": (I, [I, P, P, I, I, P]),
    "tw_linear_workspace_bytes": (L, [I, I, I, I]),
    "tw_linear_partial_splits": (I, [I, I, I]),
    "tw_linear_partial_splits_rows": (I, [I, I, I, I, I, L]),
    "tw_linear_partials": (I, [I, P, L, P, L, I, P, L, I, I, I, P]),
    "tw_linear_glu": (I, [I, P, L, P, L, I, P, P, L, I, I, I, I, I, F, P]),
    "tw_linear": (I, [I, I, P, L, P, L, I, P, P, L, P, L, P, L, I, I, I, I, P]),
    "tw_linear_act": (I, [I, P, L, P, L, I, P, P, L, P, L, I, I, I, I, P]),
    "tw_attn_decode_splits": (I, [I, I, I, I]),
    "tw_attn_decode_workspace_floats": (L, [I, I, I, I]),
    "tw_attn_decode": (I, [I, P, L, P, P, P, I, P, P, I, I, P, L, P, L, I, I, I, I, I, I, F, F, I, I, P, P, I, P]),
    "tw_attn_prefill_split": (I, [I, I, I, I, I, I, ctypes.POINTER(c_int), ctypes.POINTER(c_int)]),
    "tw_attn_prefill_workspace_floats": (L, [I, I, I, I]),
    "tw_attn_prefill": (I, [I, P, L, P, P, P, I, P, P, I, I, I, P, L, P, L, I, I, I, I, I, I, I, I, I, I, F, F, I, P, P, P, I, P]),
    "tw_attn_kept_keys": (I, [I, P, L, P, P, P, I, P, P, I, I, I, I, P, L, P, P, I, I, I, I, I, I, F, P]),
    "tw_add_table_rows": (I, [I, P, P, P, I, I, I, P, P]),
    "tw_causal_conv": (I, [I, I, P, L, P, F, P, P, F, P, P, P, P, P, P, L, P, L, I, I, I, I, P, I, P]),
    "tw_gated_recurrence_workspace_floats": (L, [I, I, I]),
    "tw_gated_recurrence": (I, [I, P, L, P, L, P, L, P, P, P, P, P, L, I, I, I, I, I, F, F, P, L, P]),
    "tw_block_diagonal": (I, [I, P, L, P, P, P, L, I, I, I, I, P]),
    "tw_gelu_mul": (I, [I, P, P, I, I, F, P]),
    "tw_round_rows": (I, [I, P, P, L, P]),
    "tw_token_gate": (I, [I, P, P, L, P, P, I, I, I, P, I, I, P]),
    "tw_layer_end": (I, [P, P, P, F, F, P, L, I, P, I, I, P]),
    "tw_attn_mixed_splits": (I, [I, I]),
    "tw_attn_mixed_prefill_splits": (I, [I, I, I]),
    "tw_attn_mixed_workspace_floats": (L, [I, I, I, I, I]),
    "tw_attn_mixed": (I, [I, P, L, P, P, P, I, P, P, I, I, I, P, L, P, P, P, P, L, I, I, I, I, I, I, I, F, F, I, P]),
    "tw_kv_store": (I, [I, P, L, I, I, P, P, P, I, I, I, I, I, P]),
    "tw_residual_norm": (I, [I, P, P, L, P, I, L, P, P, P, I, I, F, F, P]),
    "tw_relu_squared": (I, [I, P, L, I, I, P, I, P]),
    "tw_embed_hashed": (I, [I, P, P, I, P, P, P, P, P, P, P, P, I, I, I, I, L, L, L, F, F, P, P, P]),
    "tw_latent_finish": (I, [I, P, L, I, I, I, P, P, P, P, L, P, L, I, I, I, I, P, P, P, I, I, I, I, I, I, I, F, P]),
    "tw_latent_decode_splits": (I, [I, I, I]),
    "tw_latent_decode_workspace_floats": (L, [I, I, I, I]),
    "tw_latent_decode": (I, [I, P, L, P, P, P, I, P, P, I, P, L, P, L, I, I, I, I, F, I, P, P]),
    "tw_latent_gather": (I, [I, P, P, I, P, P, P, P, I, I, I, I, I, I, P]),
    "tw_latent_expand_store": (I, [I, P, L, P, I, I, P, P, I, I, I, I, I, I, I, P]),
    "tw_head_linear": (I, [I, P, L, I, P, P, L, I, I, I, I, I, P]),
    "tw_retention_workspace_floats": (L, [I, I, I, I, I]),
    "tw_retention": (I, [I, P, L, I, I, I, P, P, I, P, P, P, P, P, L, I, I, I, I, I, I, F, P, L, P]),
    "tw_unit_gate": (I, [I, P, L, P, L, P, L, I, I, I, I, F, P]),
    "tw_swish_limited_mul": (I, [I, P, P, I, I, F, P]),
    "tw_rmsnorm_pair": (I, [I, P, P, P, P, P, I, I, F, P]),
    "tw_scale_values": (I, [P, L, F, P]),
    "tw_delta_rule": (I, [P, L, I, I, I, P, L, I, I, P, P, P, P, P, P, L, I, I, I, I, I, I, I, I, F, P]),
    "tw_head_norm_gate": (I, [I, P, L, P, L, P, P, L, I, I, I, F, I, I, P]),
    "tw_moe_route": (I, [I, P, L, P, P, I, I, I, I, I, P, P, I, I, F, P]),
    "tw_moe_capacity": (L, [L, I]),
    "tw_moe_experts": (I, [I, P, L, P, P, I, I, I, P, P, P, I, I, I, F, P, P, P, P, P, P, I, P, L, I, I, P, I, P]),
    "tw_add_normed": (I, [I, P, P, L, P, I, L, P, P, I, I, F, F, P]),
    "tw_activation": (I, [I, P, L, I, I, P, I, I, P]),
    "tw_sigmoid_gate": (I, [I, P, L, P, L, I, I, I, P]),
    "tw_softcap_values": (I, [P, L, F, P]),
    "tw_qk_finish": (I, [I, P, L, I, I, P, P, P, P, P, L, P, P, P, I, I, I, I, I, I, I, I, F, P]),
    "tw_mlstm": (I, [P, L, I, I, I, I, I, P, P, P, P, P, P, P, P, I, I, P, L, I, I, I, F, F, I, I, I, P]),
    "tw_embed_sinusoid": (I, [I, P, P, P, P, P, P, P, F, I, I, I, P, I, P]),
    "tw_head_finish": (I, [I, P, L, I, I, I, P, P, L, P, P, P, I, I, I, I, I, I, I, I, F, F, P]),
    "tw_add_normed_sum": (I, [P, I, ctypes.POINTER(c_void_p), ctypes.POINTER(c_int), ctypes.POINTER(c_void_p),
                              ctypes.POINTER(c_float), I, I, F, P]),
    "tw_add_values": (I, [P, P, L, P]),
    "tw_linear_state_workspace_floats": (L, [I, I, I, I, I]),
    "tw_linear_state": (I, [P, L, I, I, I, I, P, L, P, L, I, P, P, F, P, L, I, P, P, P, P, P, P, I, I, I, P, L, I, I, I, F, P, I, I, P, L, P]),
    "tw_decay_logs": (I, [P, L, P, P, F, P, L, I, I, I, P]),
    "tw_gate_group_norm": (I, [I, P, L, P, L, P, P, L, I, I, I, F, I, F, P]),
    "tw_rows_finish": (I, [I, P, L, I, L, P, I, I, I, I, I, P, P, P, P, P, I, I, P, L, P, P, P, P, I, I, I, I, I, I, I, I, F, F, P]),
    "tw_map_difference": (I, [I, P, L, P, P, L, I, I, I, I, I, F, F, F, P]),
    "tw_layer_norm": (I, [I, P, P, L, P, I, L, P, P, P, I, P, P, P, P, P, P, I, I, F, P]),
    "tw_sampling_uniform": (F, [c_uint64, c_uint64]),
    "tw_sample_workspace_bytes": (L, [I]),
    "tw_sample_rows": (I, [P, L, I, I, P, P, P, P, P, L, P]),
    "tw_sample_rows_static": (I, [P, L, I, I, P, P, P, P, P]),
}


class KernelError(RuntimeError):
    pass


def library():
    """The loaded kernel library; built on first use if it does not exist yet."""
    global _lib
    if _lib is None:
        path = _build.ensure_built()
        lib = ctypes.CDLL(str(path))
        for name, (restype, argtypes) in _SIGNATURES.items():
            fn = getattr(lib, name)
            fn.restype = restype
            fn.argtypes = argtypes
        if lib.tw_abi_version() != 1:
            raise KernelError(f"{path} has an unexpected ABI version")
        _lib = lib
    return _lib


def loaded_library_path():
    return None if _lib is None else _lib._name


def check(code, what):
    if code != 0:
        text = library().tw_error_string(int(code))
        raise KernelError(f"{what} failed: {text.decode() if text else code} (code {code})")
