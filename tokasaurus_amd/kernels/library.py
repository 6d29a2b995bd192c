"""Loads the gfx950 kernel library and declares its entry points for ctypes.

There is no fallback: when the library cannot be built or loaded, or no GPU is
present when a kernel is called, the caller gets an error.  torch must be
imported before the library so that both use the same HIP runtime.
"""

from __future__ import annotations

import ctypes
from ctypes import c_char_p, c_float, c_int, c_long, c_size_t, c_uint32, c_void_p

import torch  # noqa: F401  (loads the HIP runtime the library binds to)

from tokasaurus_amd.kernels import build as _build


class KernelError(RuntimeError):
    """A kernel refused its arguments, or its launch failed."""


_P = c_void_p
_SIGNATURES: dict[str, dict[str, list]] = {
    "core": {
        "tk_embed_gather": [c_int, _P, _P, _P, _P, c_int, c_int, c_int, _P],
        "tk_rmsnorm": [c_int, _P, _P, c_int, _P, c_int, c_int, c_float, _P],
        "tk_add_rmsnorm": [c_int, _P, _P, _P, c_int, _P, _P, c_int, c_int, c_float, _P],
        "tk_swiglu": [c_int, _P, _P, c_int, c_int, _P],
        "tk_gather_rows": [c_int, _P, c_int, _P, _P, c_int, c_int, _P],
        "tk_rope_table": [_P, _P, _P, c_int, c_int, _P],
        "tk_rope_append": [c_int, _P, c_int, _P, _P, _P, c_int, _P, _P, _P, _P] + [c_int] * 7 + [_P],
        "tk_fill_u32": [_P, c_uint32, c_size_t, _P],
        "tk_gemm_generic": [c_int, _P, c_int, _P, _P, c_int, _P, c_int, _P, c_int, c_int, c_int, c_int, _P],
        "tk_add_bias": [c_int, _P, _P, c_int, c_int, _P],
        "tk_head_rmsnorm": [c_int, _P, c_int, _P, c_int, c_int, c_int, c_int, c_int, c_float, _P],
        "tk_paged_attention_generic": [c_int, _P, c_int, _P, c_int, _P, _P, _P, c_int, _P, _P]
        + [c_int] * 8
        + [c_float, _P, _P, c_float, _P, c_int, _P, _P],
        "tk_paged_attention_generic_fits": [c_int, c_int, c_int, c_int],
        "tk_add": [c_int, _P, _P, _P, c_size_t, _P],
        "tk_embed_scaled": [c_int, _P, _P, _P, _P, c_int, c_int, c_int, c_float, _P, _P, c_int, _P],
        "tk_depth_average": [c_int, _P, c_size_t, c_int, _P, _P, _P, _P, _P, c_float, c_float, _P, c_int, c_int, _P, _P, c_float, _P],
        "tk_linear_attention": [c_int, _P, _P],
        "tk_linear_attention_state_words": [c_int] * 4,
        "tk_linear_attention_work_words": [c_int] * 5,
        "tk_linear_attention_chunk_words": [c_int] * 4,
        "tk_linear_attention_chunk_tokens": [],
        "tk_group_norm_gate": [c_int, _P, c_int, _P, c_int, c_int, _P, c_int, _P, c_float, c_float, _P, c_int, c_int, c_int, c_int, _P],
        "tk_sigmoid_gate": [c_int, _P, c_int, _P, c_int, c_float, _P, c_int, c_int, c_int, _P],
        "tk_short_conv": [c_int, _P, c_int, _P, c_int, _P, c_size_t, _P, _P, _P, _P] + [c_int] * 4 + [_P],
        "tk_gelu_glu": [c_int, _P, _P, c_int, c_int, _P],
        "tk_residual_norm": [c_int, _P, _P, _P, c_float, _P, _P, _P, _P, c_float, c_float, c_int, _P, _P, c_int, c_int, _P],
        "tk_state_space": [c_int, _P, c_int, c_int, c_int, _P, _P, c_int, _P, _P, _P, _P, c_size_t, c_size_t, _P, _P, _P, _P, _P, _P] + [c_int] * 7 + [_P],
        "tk_state_space_token_bytes": [c_int] * 6,
        "tk_gate_group_norm": [c_int, _P, _P, c_int, _P, c_float, _P, c_int, c_int, c_int, _P],
        "tk_rotate_heads": [c_int, _P, c_int, _P, _P] + [c_int] * 5 + [c_float, _P],
        "tk_softcap": [_P, c_size_t, c_float, _P],
        "tk_qk_prepare": [c_int, _P, c_int, _P, _P, _P, c_int, _P, _P, c_float, _P, _P, _P] + [c_int] * 13 + [_P, c_int, c_float, c_int, _P],
        "tk_unrotate_gate": [c_int, _P, c_int, _P, _P, c_int, _P, c_int, c_int, c_int, c_int, _P],
        "tk_min_gru": [c_int, _P, c_int, _P, _P, c_size_t, _P, _P, _P, c_int, c_int, c_int, _P],
        "tk_embed_bigram": [c_int, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P, c_int, c_int, c_int, c_float, c_int, c_int, c_int, _P],
        "tk_cast_rows": [c_int, _P, _P, c_size_t, _P],
        "tk_scale_values": [_P, c_size_t, c_float, _P],
        "tk_clamped_glu": [c_int, _P, _P, c_int, c_int, c_float, c_float, _P],
        "tk_gather_keys": [c_int, _P, _P, c_int, _P, _P, _P] + [c_int] * 5 + [_P],
        "tk_post_norm_residual": [c_int, _P, _P, _P, c_float, _P, _P, c_float, _P, _P, c_float, _P, c_int, c_int, _P],
        "tk_concat_cast": [c_int, _P, _P, _P, c_int, c_int, _P],
        "tk_expert_route": [c_int, _P, c_int, _P, _P, _P] + [c_int] * 6 + [_P, _P, _P, c_float, c_int, _P],
        "tk_expert_gate_up": [c_int, _P, c_int, _P, _P, _P, _P] + [c_int] * 5 + [c_float, c_float, _P],
        "tk_expert_lookup": [_P, _P, c_int, _P, _P, c_int, c_int, _P],
        "tk_expert_combine": [c_int, _P, c_int, _P, _P, _P, _P, _P, _P, _P] + [c_int] * 6 + [_P],
        "tk_head_linear": [c_int, _P, c_int, _P, _P, c_int, c_int] + [c_int] * 4 + [_P, _P, c_int, c_int, c_float, _P, c_int, _P],
        "tk_squared_relu": [c_int, _P, c_size_t, _P],
        "tk_attention_tile_f32": [c_int, _P, c_int, _P, c_int, _P, _P, _P, c_int, _P, _P, _P, _P] + [c_int] * 8
        + [c_float, _P, _P, c_int, c_int, c_int, c_int, _P, _P, c_int, _P, c_int, c_float, _P, c_int, _P, _P],
        "tk_attention_tile_turns_halves": [c_int],
        "tk_attention_tile_part_words": [c_int],
        "tk_attention_tile_f32_fits": [c_int] * 5,
        "tk_delta_prepare": [c_int, _P, c_int, c_int, _P, c_int, _P, c_int, _P, _P, _P, c_size_t, c_size_t, _P, _P, _P, _P]
        + [c_int] * 7 + [_P],
        "tk_delta_rule": [_P, c_int, _P, c_size_t, _P, _P, _P] + [c_int] * 6 + [_P],
        "tk_gated_head_norm": [c_int, _P, _P, c_int, _P, c_float, _P, c_int, c_int, c_int, _P],
        "tk_sample": [_P, c_int, c_int, c_int, _P, _P, _P, _P, _P, _P, _P, _P, _P, _P],
        "tk_sample_static": [_P, c_int, c_int, c_int, _P, _P, _P, _P, _P, _P, _P],
        "tk_sample_chunks": [c_int],
        "tk_topk_logprobs": [_P, c_int, c_int, c_int, _P, c_int, _P, _P, _P, _P, _P, _P, _P],
        "tk_stage_step": [_P, _P, _P, c_int, c_int, _P],
        "tk_publish_step": [_P, _P, c_int, c_int, _P, _P, c_int, _P, _P, c_int, _P],
    },
    "mfma": {
        "tk_paged_attention_mfma": [_P, c_int, _P, c_int, _P, _P, _P, c_int, _P, _P, _P, _P, _P]
        + [c_int] * 7
        + [c_float, c_int, c_int, c_int, c_int, _P, _P, _P, c_int, _P],
        "tk_gemm_skinny_bf16": [_P, c_int, _P, _P, c_int, _P, c_int, _P] + [c_int] * 9 + [_P],
        "tk_gemm_skinny_parts": [c_int, c_int, c_int],
        "tk_grouped_gemm_bf16": [_P, c_int, _P, _P, _P, c_int, c_int, c_int, c_int, _P, c_size_t, _P, c_int, c_int, c_int, c_int,
                                 c_int, c_int, _P, _P, c_int, c_float, c_float, _P],
        "tk_expert_sort": [_P, c_int, _P],
        "tk_expert_sum": [_P, c_int, _P, _P, _P, _P, _P, _P, c_int, c_int, c_int, c_int, c_int, _P],
    },
    "library": {
        "tk_gemm_library_bf16": [_P, c_int, _P, c_int, _P, c_int, c_int, c_int, c_int, c_int, _P, c_size_t, _P],
    },
}
_GROUP_OF = {name: group for group, sigs in _SIGNATURES.items() for name in sigs}

_libs: dict[str, ctypes.CDLL] = {}


def load(group: str = "core") -> ctypes.CDLL:
    """The loaded library of a group; builds it first when it is not there."""
    if group in _libs:
        return _libs[group]
    path = _build.ensure_built(group)
    try:
        lib = ctypes.CDLL(str(path))
    except OSError as e:
        raise KernelError(f"cannot load the kernel library {path}: {e}") from None
    lib.tk_last_error.restype = c_char_p
    lib.tk_last_error.argtypes = []
    for name, argtypes in _SIGNATURES[group].items():
        try:
            fn = getattr(lib, name)
        except AttributeError:
            raise KernelError(
                f"kernel library {path} lacks entry point {name}; rebuild it with `python -m tokasaurus_amd.kernels.build`"
            ) from None
        fn.argtypes = argtypes
        fn.restype = c_int
    _libs[group] = lib
    return lib


_entry: dict[str, tuple] = {}  # name -> (the library, the entry point), looked up once


def call(name: str, *args) -> None:
    """Call an entry point and raise KernelError with its message on refusal."""
    found = _entry.get(name)
    if found is None:
        lib = load(_GROUP_OF[name])
        found = _entry[name] = (lib, getattr(lib, name))
    if found[1](*args) != 0:
        raise KernelError(found[0].tk_last_error().decode(errors="replace"))
