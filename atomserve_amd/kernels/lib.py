"""Loads the compiled kernel libraries through ctypes and declares their entry points.

The libraries use the HIP runtime that PyTorch has already loaded into the process,
so that device pointers and streams of torch tensors are valid in them; torch is
therefore imported before the first library.  There is no fallback: a kernel whose
library cannot be built or loaded raises.
"""

import ctypes
from ctypes import c_double, c_float, c_int, c_longlong, c_size_t, c_void_p

import torch  # noqa: F401  (loads libamdhip64 first)

from atomserve_amd.kernels import build

P, I, F = c_void_p, c_int, c_float

# name -> (library, argument types); every entry point returns an int status.
SIGNATURES = {
    "as_embed_gather": ("elementwise", [P, I, P, P, I, I, I, F, P]),
    "as_logits_finish": ("elementwise", [P, c_longlong, F, F, P]),
    "as_rmsnorm": ("elementwise", [P, P, P, P, I, F, P, I, I, I, I, P]),
    "as_rmsnorm_split": ("elementwise", [P, P, I, I, P, P, I, F, P, I, I, I, I, P]),
    "as_rope_table": ("elementwise", [P, P, P, I, I, P]),
    "as_rope_table_scaled": ("elementwise", [P, P, P, I, I, F, P]),
    "as_qk_norm_rope_store": ("elementwise", [P, I, P, P, I, P, P, P, P, P, I, I, I, I, I, F, I, I, P]),
    "as_silu_mul": ("elementwise", [P, P, I, I, I, P]),
    "as_rmsnorm_multi": ("elementwise", [P, P, P, P, P, P, I, F, P, P, I, I, I, I, P]),
    "as_head_norm_store": ("elementwise", [P, I, I, I, I, I, I, I, I, I, I, P, P, I, F, P, P, P, P, I, I, I, P, I, P]),
    "as_gated_add_norm": ("elementwise", [P, P, P, I, I, I, P, F, P, P, I, F, P, I, I, I, I, P, P, P]),
    "as_relu2": ("elementwise", [P, I, I, I, P, I, I, P]),
    "as_whole_norm_store": ("elementwise", [P, I, I, I, I, I, I, I, I, I, I, P, P, P, P, P, F, P, P, I, P, I, F, P, P, P, P, I, I, I, I, P]),
    "as_post_norm_add": ("sandwich", [P, P, P, I, P, P, P, P, F, P, F, P, F, I, I, P, P, I, I, I, P]),
    "as_layer_norm": ("sandwich", [P, P, P, F, P, P, I, I, I, I, P]),
    "as_token_product": ("sandwich", [P, P, P, P, P, I, I, I, P]),
    "as_token_gate": ("sandwich", [P, P, P, I, P, I, I, P]),
    "as_poly_norm": ("sandwich", [P, I, P, F, P, I, I, P]),
    "as_map_difference": ("sandwich", [P, I, I, I, I, F, F, F, P, I, I, I, I, P]),
    "as_streams_step": ("streams", [P, P, I, I, P, I, P, P, F, P, P, F, P, P, I, P]),
    "as_sigmoid_gate_heads": ("elementwise", [P, I, I, I, I, P, I, I, I, F, P, I, I, I, P]),
    "as_short_conv": ("recurrent", [P, I, I, I, I, P, P, P, I, I, I, P, P, P, P, P, P, P, I, I, I, P]),
    "as_delta_prepare": ("recurrent", [P, I, I, I, I, P, I, I, I, I, P, P, I, P, P, I, P]),
    "as_delta_scan": ("recurrent", [P, I, I, I, I, I, P, P, P, P, P, P, P, I, P, I, I, P]),
    "as_delta_finish": ("recurrent", [P, I, I, P, I, I, F, P, I, I, I, I, F, P, I, I, I, P]),
    "as_delta_scan_channels": ("recurrent", [P, I, I, I, I, I, P, P, P, P, P, P, P, I, P, I, I, P]),
    "as_delta_prepare_channels": ("recurrent", [P, I, I, I, I, P, I, I, I, P, I, I, P, P, P, P, I, P]),
    "as_memory_prepare": ("recurrent", [P, I, I, I, I, I, I, I, I, I, I, P, P, F, P, P, P, I, P]),
    "as_memory_scan": ("recurrent", [P, I, I, I, I, P, P, P, P, P, P, P, P, P, I, P, I, I, P]),
    "as_rglru_gates": ("recurrent", [P, I, I, P, P, P, P, P, I, F, P, P, I, P]),
    "as_rglru_scan": ("recurrent", [P, P, I, P, I, I, I, P, I, F, P, P, P, P, P, I, P, I, I, I, P]),
    "as_moe_route_table": ("moe", [P, P, I, I, I, I, P, P, P, I, I, P]),
    "as_moe_gemm": ("moe", [P, I, I, P, I, I, I, P, P, P, I, P, I, F, P]),
    "as_moe_combine": ("moe", [P, I, F, I, P, I, I, P, P, P, P, I, P]),
    "as_moe_route_scores": ("moe", [P, P, P, I, P, I, I, F, I, I, I, I, I, P, P, P]),
    "as_group_norm": ("layer_ops", [P, P, P, P, F, I, P, I, I, I, I, P]),
    "as_group_norm_shift": ("layer_ops", [P, P, P, F, I, P, P, P, P, P, P, P, I, I, I, I, P]),
    "as_depth_average": ("layer_ops", [P, P, I, P, P, I, c_longlong, P]),
    "as_clamped_gate": ("layer_ops", [P, P, I, I, I, F, F, P]),
    "as_decay_scan": ("linear_attention", [P, I, I, I, I, I, I, I, I, I, F, P, P, P, P, P, P, I, P, I, P]),
    "as_decay_chunks": ("linear_attention", [P, I, I, I, I, I, I, I, I, I, F, P, P, P, P, P, P, I, P, I, P]),
    "as_decay_step": ("linear_attention", [P, I, I, I, I, I, I, I, I, I, F, P, P, P, P, P, I, P, I, P]),
    "as_channel_scan": ("linear_attention", [P, I, I, I, I, I, I, I, I, F, P, P, P, P, P, P, I, P, I, P]),
    "as_channel_step": ("linear_attention", [P, I, I, I, I, I, I, I, I, F, P, P, P, P, P, I, P, I, P]),
    "as_channel_chunks": ("linear_attention", [P, I, I, I, I, I, I, I, I, F, P, P, P, P, P, P, I, P, I, P]),
    "as_channel_decays": ("linear_attention", [P, I, I, I, I, P, P, F, P, I, I, P]),
    "as_decay_finish": ("linear_attention", [P, I, I, F, P, P, I, I, I, I, P, I, P]),
    "as_state_space": ("state_space", [P, I, I, I, I, I, P, I, I, I, P, P, P, P, P, P, P, P, I, P, I, I, I, I, P, P, P]),
    "as_gated_group_norm": ("state_space", [P, P, I, I, I, P, F, I, I, P, I, P]),
    "as_rows_rms_norm": ("latent", [P, I, I, I, I, P, F, P, I, P]),
    "as_latent_kv_store": ("latent", [P, I, I, I, I, I, P, F, P, P, P, P, I, I, I, P]),
    "as_latent_q_absorb": ("latent", [P, I, I, P, P, I, I, I, I, I, P, P, I, I, P]),
    "as_latent_v_expand": ("latent", [P, P, P, I, I, I, I, I, P, I, I, P, I, P]),
    "as_wide_attend": ("latent", [P, P, P, I, P, P, P, I, P, I, I, I, I, F, I, I, I, F, I, P, I, I, P]),
    "as_attn_headmix_mfma": ("attention_mix", [P, P, P, P, I, I, I, P, P, P, I, P, P, I, I, I, I, I, F, I, I, I, P, P, P]),
    "as_attn_headmix": ("attention_mix", [P, P, P, I, P, I, I, P, P, P, I, P, P, I, I, I, I, I, F, I, I, P]),
    "as_attn_single_query": ("attention", [P, P, P, I, P, I, P, P, P, I, P, P, P, P, I, I, I, I, F, I, I, I, F, I, P, I, I, I, P]),
    "as_attn_decode_mfma": ("attention", [P, P, P, P, I, P, P, P, I, P, P, P, P, I, I, I, I, F, I, I, I, F, I, P, I, I, I, P]),
    "as_attn_decode_mfma_shared": ("attention", [P, P, P, P, I, P, P, P, I, P, P, P, P, I, I, I, I, F, I, I, I, F, I, P, I, I, I, I, P]),
    "as_attn_decode_fresh": ("attention", [P, P, P, I, P, P, F, I, P, P, P, I, P, P, I, P, P, P, P, I, I, I, I, F, I, I, I, P]),
    "as_attn_prefill_mfma": ("attention", [P, P, P, P, I, P, I, P, I, I, I, I, F, I, I, I, F, I, P, I, I, I, I, P, P, P, P]),
    "as_gemm_f32": ("gemm", [P, P, P, I, I, I, P]),
    "as_gemm_bf16_skinny": ("gemm", [P, P, P, P, I, I, I, I, I, P]),
    "as_gemm_bf16_gated": ("gemm", [P, P, P, P, I, I, I, P]),
    "as_gemm_bf16_gated_limited": ("gemm", [P, P, P, P, I, I, I, F, F, P]),
    "as_gemm_bf16_link": ("gemm", [P, P, P, P, P, P, P, I, I, I, P]),
    "as_gemm_bf16_scaled": ("gemm", [P, P, I, F, P, P, P, I, I, I, I, P]),
    "as_wave_order": ("gemm", [P, P, I, I, P]),
    "as_gemm_bf16_tile": ("gemm", [P, P, P, P, P, I, I, I, I, I, I, I, P]),
    "as_blas_plan": ("blas", [I, I, I, I, c_size_t]),
    "as_blas_candidate_index": ("blas", [I, I, I, I, c_size_t, I]),
    "as_blas_adopt": ("blas", [I, I, I, I, c_size_t, I]),
    "as_blas_prepare_adoption": ("blas", []),
    "as_blas_gemm": ("blas", [P, P, P, I, I, I, I, I, P, c_size_t, P]),
    "as_argmax": ("sampling", [P, P, I, I, P]),
    "as_sample": ("sampling", [P, I, I, P, P, P, P, P, P, P]),
    "as_sample_split": ("sampling", [P, I, I, P, P, P, P, P, P, P, P, P]),
    "as_apply_penalty": ("sampling", [P, P, P, P, I, I, P]),
    "as_topk": ("sampling", [P, I, I, I, P, P, P]),
}

STATUS = {-1: "unsupported dtype", -2: "unsupported shape or size", -3: "kernel launch failed",
          -4: "partial results exceed the library's static scratch array"}

_libs: dict = {}
_funcs: dict = {}


class KernelError(RuntimeError):
    pass


def _library(name: str):
    if name not in _libs:
        path = build.library_path(name)
        try:
            _libs[name] = ctypes.CDLL(path)
        except OSError as e:
            raise KernelError(f"cannot load {path}: {e}") from e
    return _libs[name]


def entry(name: str):
    """The ctypes function `name`, loading (and if needed compiling) its library."""
    fn = _funcs.get(name)
    if fn is None:
        lib_name, argtypes = SIGNATURES[name]
        try:
            fn = getattr(_library(lib_name), name)
        except AttributeError as e:
            raise KernelError(f"lib_{lib_name}.so has no entry point {name}") from e
        fn.argtypes = argtypes
        fn.restype = c_int
        _funcs[name] = fn
    return fn


def call(name: str, *args) -> None:
    status = entry(name)(*args)
    if status != 0:
        raise KernelError(f"{name}: {STATUS.get(status, status)}")


def loaded_libraries() -> list:
    return sorted(_libs)


__all__ = ["KernelError", "call", "entry", "loaded_libraries", "c_double"]
