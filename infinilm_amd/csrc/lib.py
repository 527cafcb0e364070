"""Loads the compiled kernel library and declares its C entry points.

The library shares the process's HIP runtime with PyTorch (PyTorch is imported first, so the
runtime it ships is the one the dynamic linker binds), which makes PyTorch's streams and device
pointers valid arguments.  There is no fallback: without the library, or without a GPU at call
time, the kernels raise.
"""
from __future__ import annotations

import ctypes
from ctypes import c_float, c_int, c_long, c_void_p
from typing import Optional

_lib: Optional[ctypes.CDLL] = None

_P = c_void_p
_I = c_int
_F = c_float
_L = c_long

_SIGNATURES = {
    "ilm_embed": [_P, _P, _P, _I, _I, _I, _F, _I, _P],
    "ilm_add_rmsnorm": [_P, _P, _P, _P, _I, _I, _F, _F, _I, _I, _I, _I, _L, _I, _F, _P],
    "ilm_gemm_ksplit": [_P, _I, _I, _L, _I, _P, _I, _P, _F, _I, _I, _I, _P, _I, _I, _P],
    "ilm_rope_kvwrite": [_P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _P],
    "ilm_swiglu": [_P, _P, _I, _I, _I, _I, _I, _P],
    "ilm_gather_rows": [_P, _P, _P, _I, _I, _I, _P],
    "ilm_scale_rows": [_P, _I, _I, _I, _F, _P],
    "ilm_gemm_gateup_swiglu": [_P, _I, _P, _I, _P, _I, _P, _I, _I, _I, _P, _I, _F, _I, _P],
    "ilm_gemm_tail": [_P, _I, _P, _I, _P, _P, _I, _P, _I, _P, _P, _I, _F, _I, _I, _I, _P],
    "ilm_gemm_rows64": [_P, _I, _L, _I, _P, _I, _I, _I, _I, _P, _I, _I, _P],
    "ilm_gemm_tall": [_P, _I, _L, _I, _I, _I, _P, _I, _I, _I, _I, _P, _I, _I, _P],
    "ilm_gemm_tall_swiglu": [_P, _I, _P, _I, _P, _I, _P, _I, _I, _I, _I, _I, _I, _P],
    "ilm_gemm_qkv_rope": [_P, _I, _P, _I, _P, _I, _P, _I, _I, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _P],
    "ilm_frag_pack_weight": [_P, _P, _P, _I, _I, _I, _I, _P],
    "ilm_frag_pack_rows": [_P, _P, _I, _I, _I, _P],
    "ilm_frag_unpack_rows": [_P, _P, _I, _I, _I, _P],
    "ilm_gemm_frag": [_P, _I, _L, _I, _P, _P, _P, _I, _I, _I, _I, _F, _I, _P],
    "ilm_gemm_frag_swiglu": [_P, _P, _P, _P, _I, _I, _I, _P, _I, _I, _F, _I, _P],
    "ilm_gemm_frag_rope": [_P, _I, _P, _P, _P, _I, _I, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _P],
    "ilm_gemm_frag_tail": [_P, _I, _P, _P, _P, _P, _P, _P, _I, _F, _I, _I, _I, _I, _P],
    "ilm_gemm_f32_skinny": [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F, _P],
    "ilm_gemm_f32_tile": [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F, _P],
    "ilm_attn_f32": [_P, _P, _I, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _F, _P],
    "ilm_gemm_basic": [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F, _I, _I, _P],
    "ilm_attn_basic": [_P, _P, _I, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _I, _F, _P],
    "ilm_gemm_skinny": [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F, _I, _I, _I, _P],
    "ilm_gemm_tall_act": [_P, _I, _P, _I, _P, _I, _P, _I, _I, _I, _I, _I, _I, _P],
    "ilm_attn_mfma": [_P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _I, _I, _F, _I, _P],
    "ilm_attn_mfma_static": [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _I, _I, _P],
    "ilm_attn_tile": [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _F, _I, _P],
    "ilm_argmax": [_P, _P, _I, _I, _I, _P],
    "ilm_sample": [_P, _P, _P, _P, _P, _P, _I, _I, _I, _P],
    "ilm_unary": [_P, _P, _I, _I, _I, _I, _I, _I, _I, _P],
    "ilm_lin_prep": [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _F, _I, _P],
    "ilm_decay_scan": [_P, _I, _P, _P, _I, _I, _P, _I, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P, _P, _P, _I, _P],
    "ilm_sigmoid_root": [_P, _P, _P, _I, _I, _I, _I, _F, _I, _I, _P],
    "ilm_add_layernorm": [_P, _P, _P, _P, _I, _I, _F, _I, _I, _I] + [_P, _I, _I, _L, _L, _F] * 4 + [_P],
    "ilm_add_rows": [_P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I] + [_P, _I, _I, _L, _L, _F] * 4 + [_P],
    "ilm_qkv_norm_rope_kvwrite": [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _I, _I, _I, _I, _F, _I, _P],
    "ilm_head_gate": [_P, _P, _I, _I, _I, _I, _I, _I, _P],
    "ilm_attn_headmix": [_P, _P, _P, _P, _P, _P, _P, _P, _I, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _I, _I, _P],
    "ilm_headmix_queries": [_P, _P, _P, _I, _I, _I, _I, _I, _P],
    "ilm_attn_headmix_mfma": [_P, _P, _P, _P, _P, _P, _P, _P, _I, _P, _I, _P, _I, _I, _I, _I, _I, _I, _F, _I, _P, _I, _I, _P, _I, _I, _P],
    "ilm_latent_prep": [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F, _I, _I, _I, _I, _I, _P],
    "ilm_embed_pos": [_P, _P, _P, _P, _P, _I, _I, _I, _I, _F, _I, _P],
    "ilm_stream_update": [_P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _F, _F, _F, _I, _I, _I, _I, _I, _L, _I, _I, _P],
    "ilm_embed_gate": [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _P],
    "ilm_softcap": [_P, _L, _F, _P],
    "ilm_moe_route": [_P, _P, _P, _I, _I, _I, _I, _I, _F, _P],
    "ilm_moe_route_groups": [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _F, _P],
    "ilm_moe_sort": [_P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _P],
    "ilm_moe_gemm": [_P, _I, _P, _I, _P, _I, _P, _P, _L, _I, _P, _P, _I, _I, _I, _I, _F, _F, _I, _I, _I, _I, _I, _P],
    "ilm_moe_combine": [_P, _P, _P, _I, _P, _P, _I, _I, _I, _I, _P, _P, _I, _I, _P],
    "ilm_maps_norm_rope_kvwrite": [_P, _P, _I, _I, _I, _I, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _I, _I, _I, _I, _P],
    "ilm_attn_maps_mfma": [_P, _P, _P, _P, _P, _P, _P, _P, _I, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _P, _P, _P, _P, _P, _F, _F, _F, _I, _P],
    "ilm_maps_combine": [_P, _P, _I, _I, _I, _I, _I, _P, _P, _P, _P, _F, _F, _F, _I, _I, _P],
    "ilm_attn_maps": [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _F, _I, _I, _P, _P, _P, _P, _P, _F, _F, _F,
                      _I, _I, _P],
    "ilm_selective_scan": [_P, _I, _P, _I, _P, _I, _P, _P, _P, _I, _P, _I, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P, _P, _I, _I, _P],
    "ilm_glu_clamp": [_P, _P, _I, _I, _I, _F, _F, _I, _P],
    "ilm_head_gemm": [_P, _P, _P, _I, _I, _I, _I, _L, _L, _L, _L, _L, _L, _L, _I, _I, _P],
    "ilm_head_gemm_mfma": [_P, _P, _P, _I, _I, _I, _I, _L, _L, _L, _L, _L, _L, _L, _P],
    "ilm_group_norm_gate": [_P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _F, _I, _I, _I, _I, _I, _I, _I, _L, _F, _I, _P],
    "ilm_causal_conv": [_P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _P],
    "ilm_ssm_steps": [_P, _P, _P, _P, _P, _I, _I, _I, _I, _P],
    "ilm_unit_qk_kvwrite": [_P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _F, _F, _I, _I, _P],
    "ilm_weighted_sum": [_P, _P, _P, _L, _F, _F, _I, _I, _I, _P],
    "ilm_hyper_update": [_P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _F, _F, _F, _I, _I, _I, _I, _L, _I, _P],
    "ilm_conv_delta_inputs": [_P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _F, _F, _I, _I, _P],
    "ilm_conv_norm_rope_kvwrite": [_P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _I, _F,
                                   _I, _I, _I, _P],
    "ilm_delta_step": [_P, _P, _P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P, _P, _I, _F, _I, _I, _I, _I, _P],
    "ilm_delta_chunks": [_P, _P, _I, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _I, _P, _P],
    "ilm_mlstm_step": [_P, _P, _P, _I, _I, _P, _P, _I, _I, _I, _I, _F, _F, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _P, _I, _F, _I, _I, _P],
    "ilm_mlstm_chunks": [_P, _P, _P, _I, _I, _P, _P, _I, _I, _I, _I, _F, _F, _P, _P, _P, _P, _P, _I, _I, _I, _I, _I, _I, _I, _P, _I, _F, _I, _I, _P, _P],
    "ilm_norm_add_norm": [_P, _P, _P, _P, _P, _I, _I, _F, _F, _F, _I, _I, _I, _I, _I, _L, _P],
}


def _check_single_hip_runtime() -> None:
    try:
        with open("/proc/self/maps") as fh:
            libs = {line.split()[-1] for line in fh if "libamdhip64" in line}
    except OSError:
        return
    real = {__import__("os").path.realpath(p) for p in libs}
    if len(real) > 1:
        raise RuntimeError("infinilm_amd: two HIP runtimes are loaded in this process (" + ", ".join(sorted(real))
                           + "); the kernel library and PyTorch must share one")


def load(verbose: bool = True) -> ctypes.CDLL:
    """The library, compiled first if no up-to-date build exists."""
    global _lib
    if _lib is not None:
        return _lib
    import torch  # noqa: F401  (binds PyTorch's HIP runtime before ours is resolved)
    from . import build as _build

    path = _build.ensure_built(verbose=verbose)
    lib = ctypes.CDLL(path, mode=ctypes.RTLD_GLOBAL)
    _check_single_hip_runtime()
    lib.ilm_last_error.restype = ctypes.c_char_p
    lib.ilm_last_error.argtypes = []
    for name, args in _SIGNATURES.items():
        fn = getattr(lib, name, None)
        if fn is None:
            raise RuntimeError(f"infinilm_amd: {path} lacks the entry point {name}; rebuild it "
                               "(python -c 'import __graft_entry__ as g; g.build()')")
        fn.argtypes = args
        fn.restype = c_int
    lib.ilm_attn_headmix_mfma_ok.restype = c_int
    lib.ilm_attn_headmix_mfma_ok.argtypes = [c_int, c_int, c_int, c_int]
    lib.ilm_attn_maps_mfma_ok.restype = c_int
    lib.ilm_attn_maps_mfma_ok.argtypes = [c_int, c_int, c_int, c_int, c_int, c_int]
    lib.ilm_delta_step_norm_ok.restype = c_int
    lib.ilm_delta_step_norm_ok.argtypes = [c_int, c_int]
    lib.ilm_mlstm_step_norm_ok.restype = c_int
    lib.ilm_mlstm_step_norm_ok.argtypes = [c_int, c_int]
    lib.ilm_mlstm_chunk_ws.restype = c_int
    lib.ilm_mlstm_chunk_ws.argtypes = [c_int, c_int, c_int]
    lib.ilm_delta_chunk_ws.restype = c_int
    lib.ilm_delta_chunk_ws.argtypes = [c_int, c_int]
    lib.ilm_attn_static_init.restype = c_int
    lib.ilm_attn_static_init.argtypes = []
    lib.ilm_attn_static_scratch_floats.restype = c_long
    lib.ilm_attn_static_scratch_floats.argtypes = []
    _lib = lib
    return lib


def last_error() -> str:
    return load().ilm_last_error().decode(errors="replace")
