"""Loading of the built kernel libraries through ctypes, one library at a time.

A library is compiled the first time one of its functions is asked for (see
`build.ensure`), so a program compiles only what it uses.  There is no other
implementation behind these functions: if a library cannot be built or loaded,
the call raises.
"""
from __future__ import annotations

import ctypes
import threading

from . import build

_p = ctypes.c_void_p
_i = ctypes.c_int
_ll = ctypes.c_longlong
_f = ctypes.c_float

# function name -> (library, argument types); every function returns a hipError_t as int
SIGNATURES = {
    "arle_embed_gather": ("elementwise", [_p, _i, _p, _p, _i, _i, _f, _p]),
    "arle_silu_mul": ("elementwise", [_p, _p, _ll, _p, _i, _i, _i, _i, _p]),
    "arle_rmsnorm": ("norm", [_p, _i, _ll, _p, _i, _p, _i, _p, _i, _i, _f, _p]),
    "arle_add_rmsnorm": ("norm", [_p, _p, _i, _ll, _i, _p, _i, _p, _i, _p, _i, _i, _f, _p]),
    "arle_sum_partials": ("elementwise", [_p, _i, _ll, _p, _i, _ll, _i, _p]),
    "arle_gemm_rows_rounds": ("gemm_rows", [_p, _ll, _p, _ll, _i, _p, _ll, _i, _i, _i, _i, _i, _p]),
    "arle_gemm_rows": ("gemm_rows", [_p, _ll, _p, _ll, _i, _p, _ll, _ll, _i, _i, _i, _i, _i, _i, _i, _i, _p]),
    "arle_gemm_rows_geometry": ("gemm_rows", [_i]),
    "arle_gemm_stream_geometry": ("gemm_rows", [_i]),
    "arle_gemm_stream_lds": ("gemm_rows", [_i, _i, _i]),
    "arle_gemm_stream": ("gemm_rows", [_p, _ll, _p, _ll, _i, _p, _ll, _ll, _i, _i, _i, _i, _i, _i, _i, _i, _p]),
    "arle_gemm_rows_lds": ("gemm_rows", [_i, _i, _i]),
    "arle_gemm_tiles": ("gemm_tiles", [_p, _ll, _p, _p, _ll, _i, _i, _i, _i, _i, _i, _i, _i, _i, _i, _ll, _p]),
    "arle_gemm_tiles_patch": ("gemm_tiles", [_i, _i]),
    "arle_gemm_rows_lds_max": ("gemm_rows", []),
    "arle_gemm_f32": ("gemm_f32", [_p, _ll, _p, _ll, _p, _ll, _i, _i, _i, _p]),
    "arle_qk_prep": ("rope_kv", [_p, _ll, _p, _ll, _p, _ll, _i, _p, _p, _i, _p, _p, _i, _p, _p, _p,
                                 _i, _p, _p, _i, _i, _i, _i, _i, _f, _p, _i, _ll, _ll, _p]),
    "arle_attn_paged_simt": ("attention_simt", [_p, _ll, _p, _ll, _p, _p, _i, _p, _i, _p, _p, _p, _i,
                                                _i, _i, _i, _i, _f, _i, _p]),
    "arle_attn_decode_prep": ("attention_mfma", [_p, _i, _i, _ll, _ll, _p, _p, _i, _p, _p, _i, _f, _p, _ll, _p, _p, _p, _i, _p,
                                                 _p, _p, _i, _i, _i, _i, _i, _f, _i, _i, _p, _p, _p]),
    "arle_attn_decode_inwg": ("attention_mfma", [_i]),
    "arle_attn_prefill_variant": ("attention_mfma", [_i]),
    "arle_attn_prefill_pair_up": ("attention_mfma", [_i]),
    "arle_attn_prefill_fixed_rounds": ("attention_mfma", [_i]),
    "arle_attn_prefill_groups": ("attention_mfma", [_i]),
    "arle_attn_side_branch": ("attention_mfma", [_i]),
    "arle_attn_paged_mfma": ("attention_mfma", [_p, _ll, _p, _ll, _p, _p, _p, _i, _p, _p, _p, _i, _i, _i, _i, _i, _i,
                                                _i, _i, _i, _f, _i, _i, _p, _p, _i, _p, _p, _ll, _p, _f, _p]),
    "arle_argmax_chunks": ("sampling", [_i, _i]),
    "arle_argmax_rows": ("sampling", [_p, _i, _i, _p, _p, _p]),
    "arle_sample_scratch_bytes": ("sampling", [_i, _i]),
    "arle_sample_rows": ("sampling", [_p, _i, _i, _p, _p, _p, _p, _p, _p, _p, _p, _i, _i, _p]),
    "arle_apply_penalties": ("sampling", [_p, _i, _i, _p, _p, _p, _p, _p, _p, _p]),
    "arle_token_logprobs": ("sampling", [_p, _i, _i, _p, _p, _p]),
    "arle_attn_decode_static": ("attention_mfma", [_p, _ll, _p, _ll, _p, _p, _p, _i, _p, _p, _p, _i, _i, _i, _i, _i,
                                                   _i, _f, _i, _i, _p]),
    "arle_add_layernorm": ("layernorm", [_p, _p, _i, _ll, _i, _p, _i, _p, _i, _ll, _i, _p, _i, _p, _p, _i, _p, _p, _i, _p, _i,
                                         _i, _f, _p, _p, _p]),
    "arle_causal_conv": ("short_conv", [_p, _ll, _i, _p, _i, _p, _i, _p, _i, _p, _i, _p, _p, _ll, _i, _i, _i, _i, _i, _p]),
    "arle_conv_state_update": ("short_conv", [_p, _ll, _i, _p, _i, _p, _i, _p, _p, _i, _i, _i, _p]),
    "arle_polynorm": ("polynorm", [_p, _ll, _i, _p, _i, _p, _i, _p, _i, _i, _i, _f, _p]),
    "arle_mlstm_scan": ("mlstm", [_p, _ll, _p, _ll, _p, _ll, _i, _p, _ll, _p, _p, _f, _p, _p, _p, _p, _p, _i, _p, _p, _p,
                                  _i, _i, _i, _p]),
    "arle_mlstm_output": ("mlstm", [_p, _p, _p, _p, _ll, _i, _p, _i, _p, _i, _i, _i, _i, _f, _p]),
    "arle_qkv_norm_store": ("attention_softcap", [_p, _ll, _p, _ll, _p, _ll, _i, _p, _p, _i, _f, _f, _i, _p, _p, _p, _i,
                                                  _p, _p, _i, _i, _i, _i, _i, _i, _p]),
    "arle_attn_softcap_simt": ("attention_softcap", [_p, _ll, _p, _ll, _p, _p, _i, _p, _i, _p, _p, _i, _i, _i, _i, _i, _i,
                                                     _f, _f, _p, _p, _i, _i, _i, _p, _i, _i, _f, _p]),
    "arle_attn_softcap_mfma": ("attention_softcap", [_p, _ll, _p, _ll, _p, _p, _p, _i, _p, _p, _p, _i, _i, _i, _i, _i, _i, _i,
                                                     _i, _f, _f, _p, _p, _i, _i, _i, _p, _i, _i, _f, _p]),
    "arle_attn_softcap_lds_limit": ("attention_softcap", []),
    "arle_wide_norm_store": ("attention_softcap", [_p, _ll, _p, _ll, _p, _ll, _p, _ll, _i, _p, _p, _i, _p, _i, _f, _p, _p,
                                                   _p, _i, _p, _p, _i, _i, _i, _i, _i, _i, _p, _p, _i, _i, _p]),
    "arle_tanh_cap": ("elementwise", [_p, _ll, _f, _p]),
    "arle_norm_add": ("post_norm", [_p, _p, _i, _ll, _ll, _p, _i, _i, _p, _i, _ll, _ll, _p, _i, _i, _p, _i, _i, _i, _p, _f, _p,
                                    _i, _i, _i, _f, _p]),
    "arle_group_norm": ("group_norm", [_p, _i, _ll, _p, *3 * [_p, _i, _ll, _ll, _p, _i, _i], _p, _i, _p, _ll, _i, _p, _i, _i, _i, _f,
                                       _i, _p]),
    "arle_retention_prep": ("retention", [_p, _ll, _p, _ll, _p, _p, _i, _p, _i, _i, _i, _p]),
    "arle_retention_scan": ("retention", [_p, _ll, _p, _ll, _p, _ll, _p, _p, _p, _p, _i, _p, _i, _i, _i, _p]),
    "arle_retention_output": ("retention", [_p, _p, _ll, _f, _p, _i, _i, _i, _i, _p]),
    "arle_retention_decode": ("retention", [_p, _i, _ll, _ll, _p, _p, _p, _i, _p, _p, _p, _p, _f, _p, _i, _i, _i, _i, _i, _p]),
    "arle_retention_chunks": ("retention", [_p, _ll, _p, _p, _i, _p, _p, _p, _p, _p, _i, _i, _p, _f, _p, _i, _i, _i, _i, _p]),
    "arle_decay_scan": ("decay_scan", [_p, _ll, _p, _ll, _p, _ll, _i, _p, _ll, _i, _p, _p, _p, _f, _p, _p, _p, _i, _p, _i, _i, _i,
                                       _i, _p]),
    "arle_decay_gates": ("decay_scan", [_p, _ll, _p, _i, _p, _f, _p, _i, _i, _i, _p, _i, _i, _i, _p]),
    "arle_gated_group_norm": ("decay_scan", [_p, _p, _ll, _i, _p, _f, _f, _p, _ll, _i, _i, _i, _p]),
    "arle_gated_linear_decode": ("gated_linear", [_p, _i, _ll, _ll, _p, _i, _i, _p, _f, _p, _p, _p, _p, _f, _p, _i, _i, _i, _i, _i,
                                                  _p]),
    "arle_gated_linear_chunks": ("gated_linear", [_p, _ll, _p, _p, _p, _p, _p, _i, _i, _p, _f, _p, _i, _i, _i, _i, _p]),
    "arle_state_space_decode": ("state_space", [_p, _i, _ll, _ll, _p, _i, _p, _i, _p, _i, _p, _p, _p, _p, _p, _p, _p, _p, _f, _f,
                                                _i, _p, _ll, _i, _i, _i, _i, _i, _p]),
    "arle_state_space_chunks": ("state_space", [_p, _ll, _p, _ll, _p, _p, _p, _p, _p, _i, _i, _p, _p, _p, _p, _i, _i, _i, _i, _p]),
    "arle_rotary_sums_store": ("rotary_store", [_p, _i, _ll, _ll, _p, _p, _p, _i, _f, _i, _p, _p, _i, _i, _p, _p, _p, _i, _p, _p,
                                                _i, _i, _i, _i, _i, _i, _p]),
    "arle_latent_prep": ("latent", [_p, _ll, _p, _ll, _p, _ll, _i, _p, _i, _f, _p, _p, _i, _p, _p, _p, _i, _p, _p, _i, _i,
                                    _i, _i, _i, _i, _i, _p]),
    "arle_latent_attn": ("latent_attention", [_p, _p, _p, _p, _p, _i, _p, _p, _p, _i, _i, _i, _i, _i, _f, _i, _p, _i, _i, _i, _p, _p,
                                              _p]),
    "arle_head_proj": ("latent", [_p, _ll, _i, _p, _p, _ll, _i, _i, _i, _i, _i, _i, _p]),
    "arle_head_proj_mfma": ("latent", [_p, _ll, _i, _p, _p, _ll, _i, _i, _i, _i, _i, _p, _p, _p, _i, _i, _i, _p]),
    "arle_latent_down": ("latent", [_p, _i, _i, _ll, _ll, _p, _i, _i, _p, _p, _i, _f, _p, _p, _i, _p, _p, _p, _i, _p, _p, _i, _i, _i,
                                    _i, _i, _p]),
    "arle_moe_route": ("moe", [_p, _ll, _i, _p, _i, _p, _i, _p, _i, _p, _p, _p, _p, _i, _i, _i, _i, _f, _i, _i, _i, _i, _p]),
    "arle_moe_identity": ("moe", [_p, _ll, _i, _p, _p, _i, _i, _i, _i, _p]),
    "arle_moe_expert": ("moe", [_p, _ll, _p, _p, _p, _p, _i, _i, _i, _i, _i, _i, _i, _p]),
    "arle_gate_mul": ("elementwise", [_p, _ll, _p, _ll, _p, _i, _i, _i, _i, _p]),
    "arle_token_gate": ("elementwise", [_p, _ll, _i, _p, _ll, _i, _i, _p, _p, _i, _i, _i, _p]),
    "arle_act_mul": ("elementwise", [_p, _p, _ll, _p, _i, _i, _i, _i, _i, _p]),
    "arle_hyper_step": ("hyper", [_p, _ll, _ll, _p, _p, _i, _ll, _i, _ll, _p, _p, _p, _p, _f, _p, _p, _i, _ll, _i, _i, _i,
                                  _i, _p]),
    "arle_pair_norm": ("hyper", [_p, _ll, _i, _ll, _p, _ll, _i, _ll, _i, _p, _p, _f, _f, _p, _i, _i, _i, _p]),
    "arle_rotary_qkv_store": ("rotary_store", [_p, _ll, _p, _ll, _p, _ll, _i, _p, _p, _i, _f, _i, _p, _p, _i, _i, _p, _p,
                                               _p, _i, _p, _p, _i, _i, _i, _i, _i, _i, _p]),
    "arle_gated_delta_scan": ("gated_delta", [_p, _ll, _p, _ll, _p, _ll, _i, _p, _ll, _p, _ll, _p, _p, _f, _p, _p, _p, _i, _i, _p,
                                              _i, _i, _i, _i, _i, _p]),
    "arle_gated_delta_output": ("gated_delta", [_p, _p, _ll, _i, _p, _i, _f, _p, _i, _i, _i, _i, _i, _p]),
    "arle_ceiling_read": ("ceilings", [_p, _ll, _i, _p, _p, _p]),
    "arle_ceiling_mfma": ("ceilings", [_i, _i, _i, _i, _p, _p]),
}

_libs: dict = {}
_funcs: dict = {}
_lock = threading.Lock()


class KernelError(RuntimeError):
    pass


def register_signature(name: str, library: str, argtypes: list) -> None:
    SIGNATURES[name] = (library, argtypes)


def library(name: str) -> ctypes.CDLL:
    with _lock:
        lib = _libs.get(name)
        if lib is None:
            path = build.ensure(name)
            try:
                lib = ctypes.CDLL(path)
            except OSError as exc:
                raise KernelError(f"cannot load kernel library {path}: {exc}") from exc
            _libs[name] = lib
        return lib


def loaded_libraries() -> dict:
    """name -> path of the libraries this process has loaded so far."""
    return {n: lib._name for n, lib in _libs.items()}


def function(name: str):
    fn = _funcs.get(name)
    if fn is None:
        lib_name, argtypes = SIGNATURES[name]
        fn = getattr(library(lib_name), name)
        fn.argtypes = argtypes
        fn.restype = ctypes.c_int
        _funcs[name] = fn
    return fn


def function_raw(name: str, restype, library_name: str = "attention_mfma", argtypes=()):
    """A function outside the `int f(...)` convention (one that returns text, say)."""
    fn = getattr(library(library_name), name)
    fn.argtypes = list(argtypes)
    fn.restype = restype
    return fn


def call(name: str, *args) -> None:
    status = function(name)(*args)
    if status != 0:
        raise KernelError(f"{name} failed with HIP error {status}")
