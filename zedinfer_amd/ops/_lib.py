"""Loading the HIP kernel library and declaring its entry points.

There is no fallback: when the library cannot be loaded, every op raises.
"""
from __future__ import annotations

import ctypes
import struct
import threading
from ctypes import c_char_p, c_float, c_int, c_int64, c_void_p
from typing import Optional

_lock = threading.Lock()
_lib: Optional[ctypes.CDLL] = None
_lib_path: Optional[str] = None

P, I, L, F = c_void_p, c_int, c_int64, c_float

_PROTOTYPES = {
    "zi_abi_version": [],
    "zi_embedding": [P, I, P, I, P, I, I, I, P],
    "zi_embedding_scaled": [P, I, P, I, P, I, I, I, F, P],
    "zi_gather_rows": [P, P, I, P, I, I, I, P],
    "zi_add": [P, I, P, I, P, I, L, P],
    "zi_swiglu": [P, I, P, P, I, I, I, L, L, I, I, L, P],
    "zi_swiglu_t": [P, P, I, I, I, L, P],
    "zi_rmsnorm": [P, I, P, I, P, I, I, I, L, L, F, I, P],
    "zi_add_rmsnorm": [P, I, P, P, I, I, L, P, I, I, I, F, I, P],
    "zi_rope_kv_store": [P, P, P, I, I, L, L, L, P, P, P, P, L, I, I, I, I, I, I, P],
    "zi_rope": [P, P, I, I, L, L, P, P, I, I, I, P],
    "zi_attention_generic": [P, P, I, I, L, L, P, P, P, P, P, P, I, I, I, I, I, I, I, F, P],
    "zi_attention_decode": [P, P, I, I, L, L, P, P, P, P, P, P, I, I, I, I, I, I, I, F, I, P, L, P],
    "zi_attention_decode_supported": [I, I, I, I, I],
    "zi_attention_decode_fused": [P, I, I, L, P, I, L, L, P, I, P, I, P, L, I, P, P, P, P, P, P, I, I, I, I, I, I, I, F,
                                  I, P, L, P],
    "zi_attention_decode_fused_supported": [I, I, I, I, I, I, I, L, L],
    "zi_attention_decode_project": [P, P, L, I, P, I, I, P, I, L, I, I, I, P],
    "zi_attention_decode_project_supported": [I, I, I, I, L],
    "zi_attention_decode_project_heads": [I],
    "zi_rope_table": [P, P, P, I, I, P],
    "zi_decode_layer": [P, I, I, I, P, P, I, F, F, I, P, L, P, I, P, L, P, L, P, L, I, P, I, P, L, P, P, P, P, I, I, I, I,
                        I, I, I, F, I, P, L, P, P, I, P],
    "zi_decode_layer_supported": [I, I, I, I, I, I, I, I, I, I, I],
    "zi_decode_layer_sync_words": [],
    "zi_decode_layer_stamps": [],
    "zi_attention_decode_chunks": [I],
    "zi_attention_prefill": [P, P, I, I, L, L, P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, F, I, I, P, L, I, I, I, P],
    "zi_attention_prefill_chunk_keys_for": [I, I],
    "zi_attention_prefill_cuts": [I, I, I, P],
    "zi_attention_prefill_tile_min": [],
    "zi_compute_units": [],
    "zi_gemm_skinny_pays": [I, I, I],
    "zi_gemm_skinny_act_pays": [I, I, I],
    "zi_attention_prefill_chunks": [I],
    "zi_attention_prefill_variant": [I],
    "zi_attention_prefill_supported": [I, I, I, I, I],
    "zi_attention_prefill_tile": [I, I],
    "zi_attention_prefill_chunk_keys": [],
    "zi_gemm_generic": [P, I, P, I, P, I, P, I, I, I, I, L, L, L, P],
    "zi_gemm_skinny": [P, I, I, P, P, P, I, I, I, L, L, L, P, L, P],
    "zi_gemm_skinny_act": [P, I, I, P, P, P, I, I, I, L, L, L, P, L, F, P],
    "zi_clamped_glu_il8": [P, L, P, L, I, I, F, F, P],
    "zi_gemm_skinny_splits": [I, I, I],
    "zi_gemm_lt": [P, I, P, P, P, I, L, L, L, L, L, L, P, L, P],
    "zi_gemm_lt_tune": [P, I, P, P, P, I, L, L, L, L, L, L, P, L, I, I, P, P, P, P],
    "zi_gemm_lt_choose": [I, I, I, L, L, L, L, L, L, L, I],
    "zi_reduce_splits": [P, I, P, P, I, I, L, I, P],
    "zi_rope_kv_store_split": [P, I, L, P, I, L, L, P, I, I, P, P, P, P, L, I, I, I, I, I, I, P],
    "zi_gemm_skinny_supported": [I, I, I, L, L],
    "zi_argmax": [P, P, P, I, I, I, L, P, L, P],
    "zi_sample": [P, P, L, P, I, I, P, P, P, P, P, P, P, I, P],
    "zi_gated_act": [P, I, L, P, P, I, L, L, I, I, I, P],
    "zi_rope_pairs": [P, I, L, P, I, I, I, I, P],
    "zi_latent_store": [P, I, L, I, P, I, F, P, P, P, P, L, I, I, P],
    "zi_latent_query": [P, P, I, L, P, I, P, I, I, I, I, I, P],
    "zi_latent_attention": [P, P, P, P, I, I, P, P, P, P, I, I, I, I, I, I, I, F, P],
    "zi_latent_attention_cores": [P, I, P, L, P, I, P, P, P, P, P, P, I, I, I, I, I, I, I, I, I, F, I, I, I, P],
    "zi_latent_attention_cores_supported": [I, I, I],
    "zi_latent_attention_cores_tiles": [I, I, I, I],
    "zi_headwise_linear": [P, I, L, I, P, I, L, I, P, I, I, I, I, P],
    "zi_headwise_linear_supported": [I, I, L, I],
    "zi_latent_query_rot": [P, I, P, I, L, P, I, I, I, I, I, P],
    "zi_latent_value": [P, I, L, P, P, I, I, I, I, I, P],
    "zi_delta_prepare": [P, P, P, P, L, I, P, P, P, I, P, L, L, P, P, P, I, I, I, I, I, P],
    "zi_delta_conv_state": [P, L, L, P, L, P, P, P, I, I, I, P],
    "zi_delta_rule": [P, P, P, P, P, L, P, P, P, I, I, I, I, I, P],
    "zi_gated_rmsnorm": [P, I, P, P, I, P, L, I, I, I, F, P],
    "zi_moe_route": [P, P, P, P, I, I, I, F, P],
    "zi_moe_group": [P, P, P, P, I, I, I, P],
    "zi_moe_linear": [P, I, L, P, I, L, P, I, P, P, I, I, I, I, I, I, P],
    "zi_moe_combine": [P, P, P, P, I, I, I, P],
    "zi_attention_generic_sink": [P, P, I, I, L, L, P, P, P, P, P, P, I, I, I, I, I, I, I, F, P, P],
    "zi_attention_decode_sink": [P, P, I, I, L, L, P, P, P, P, P, P, I, I, I, I, I, I, I, F, I, P, L, P, P],
    "zi_attention_prefill_sink": [P, P, I, I, L, L, P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, F, I, I, P, L, I, I, I,
                                  P, P],
    "zi_attention_decode_project_sink": [P, P, L, I, P, I, I, P, I, L, I, I, I, P, P],
    "zi_attention_decode_project_gated": [P, P, L, I, P, I, I, P, I, L, I, I, I, P, P, L, I, L, P],
    "zi_attention_decode_merge_gated": [P, L, P, L, I, P, I, I, I, I, I, P, P, L, I, L, P],
    "zi_layer_norm": [P, I, L, P, P, I, I, L, L, P, P, I, I, I, F, P],
    "zi_conv_qkv": [P, I, L, P, P, P, I, L, I, L, P, P, P, L, I, P, P, F, P, I, I, P, P, P, P, L, I, I, I, I, I, I, I, P, P, F, P],
    "zi_conv_tail": [P, L, P, I, L, I, L, P, P, P, P, P, I, I, I, P],
    "zi_relu_squared": [P, I, L, P, I, L, I, L, I, I, P],
    "zi_clamped_glu": [P, I, L, P, P, I, L, L, I, L, I, I, F, F, P, P, P],
    "zi_softcap": [P, L, F, P],
    "zi_convert": [P, I, P, I, L, P],
    "zi_moe_route_top": [P, P, P, P, I, I, I, P],
    "zi_embedding_sum": [P, P, I, P, I, P, P, P, P, P, P, P, L, P, I, I, I, I, L, L, P],
    "zi_token_shift": [P, I, L, P, I, L, P, I, P, L, P, P, P, P, P, I, I, P],
    "zi_stream_reenter": [P, P, I, I, L, P, P, I, I, I, P],
    "zi_lowrank_decay": [P, L, P, L, P, P, I, I, I, I, F, P],
    "zi_linear_attention": [P, L, P, P, P, L, P, L, P, P, L, P, P, P, P, I, I, I, I, I, F, P],
    "zi_gate_heads": [P, I, L, P, I, L, I, P, L, I, L, I, I, I, I, F, P],
    "zi_gated_rmsnorm_act": [P, I, L, P, P, I, P, L, I, I, I, F, I, F, P],
    "zi_normed_kv_store": [P, I, L, P, P, P, L, I, I, I, P, L, I, I, I, I, I, I, I, F, I, P],
    "zi_attention_generic_biased": [P, P, I, I, L, L, P, P, P, P, P, P, I, I, I, I, I, I, I, F, P, F, P, I, I, P, P, P],
    "zi_attention_prefill_biased": [P, P, I, I, L, L, P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, F, I, I, P, L, I, I, I,
                                    P, F, P, I, I, P, P, P],
    "zi_attention_decode_biased": [P, P, I, I, L, L, P, P, P, P, P, P, I, I, I, I, I, I, I, F, I, P, L, P, F, P, I, I, P, P,
                                   P],
    "zi_moe_route_table": [P, P, P, P, I, I, I, I, P],
    "zi_rope_table_scaled": [P, P, P, I, I, F, P],
    "zi_linear_attention_grouped": [P, L, P, P, P, L, P, L, P, P, L, P, P, P, P, I, I, I, I, I, F, I, I, I, P],
    "zi_ssm_prepare": [P, L, P, L, I, P, P, P, P, P, L, P, P, P, I, I, I, I, P],
    "zi_ssm_finish": [P, I, L, P, L, P, L, P, L, P, P, I, I, I, I, F, P],
    "zi_norm_rope_store": [P, I, L, P, P, P, L, I, L, P, P, F, P, I, P, P, L, I, I, I, I, I, P],
    "zi_pool_blocks": [P, P, L, P, P, I, P, P, P, P, I, I, I, I, I, I, I, I, P],
    "zi_pooled_attention": [P, L, P, L, I, P, P, P, P, P, P, P, I, I, I, P, I, I, I, I, I, I, I, I, I, I, F, P, P, I, P],
    "zi_pooled_attention_cores": [P, L, P, L, P, P, P, P, P, P, P, I, I, P, I, I, I, P, I, I, I, I, I, I, I, I, I, F, P, I,
                                  I, I, P, L, P, I, P],
    "zi_pooled_attention_cores_supported": [I, I, I, I, I],
    "zi_normed_add_norm": [P, I, P, P, I, L, I, L, P, P, I, I, I, F, F, I, P],
    "zi_moe_route_sigmoid": [P, P, P, L, I, I, I, P],
    "zi_moe_weighted_glu": [P, I, L, P, L, P, P, I, I, P],
    "zi_moe_sum_shared": [P, P, P, P, I, L, P, L, I, I, I, P],
    "zi_stream_scale": [P, P, P, I, I, L, I, I, F, P],
    "zi_input_conv": [P, I, L, P, I, L, P, P, I, F, P, P, L, P, P, P, P, P, I, I, I, P],
    "zi_norm_input_conv": [P, I, P, P, I, I, L, P, I, F, F, P, P, L, P, P, P, I, I, I, P],
    "zi_norm_input_conv_supported": [I, I, I],
    "zi_lowrank_gates": [P, P, P, I, I, P, P, I, P, P, P, I, I, I, L, I, P],
    "zi_delta_channel": [P, P, P, P, L, P, P, L, P, P, P, I, I, I, I, I, I, P, I, P, P, F, P],
    "zi_delta_channel_finishes": [I, L],
    "zi_channel_inputs": [P, P, P, L, P, P, L, I, L, P, P, L, P, P, P, P, I, I, I, I, I, I, I, I, I, P],
    "zi_attention_prefill_maps": [P, P, I, I, L, L, P, P, P, P, P, P, P, P, I, I, I, I, I, I, I, F, I, I, P, L, I, I, I, I, P],
    "zi_attention_prefill_maps_supported": [I, I, I, I, I, I],
    "zi_stream_mix": [P, I, P, L, P, L, P, I, I, L, P, P, P, P, P, I, I, I, I, F, I, P],
    "zi_stream_mix_max_streams": [],
    "zi_head_norm_store": [P, I, L, P, P, P, I, L, I, L, P, P, F, P, I, P, L, I, I, I, I, I, I, I, I, I, P],
    "zi_difference_heads": [P, I, L, P, L, I, I, I, I, F, F, F, P, I, L, I, L, P],
    "zi_difference_merge": [P, L, P, L, I, P, I, I, I, I, I, F, F, F, P, I, L, I, L, P],
    "zi_activate": [P, I, L, P, I, L, I, L, I, I, I, P],
    "zi_latent_inputs": [P, I, L, P, I, L, I, L, I, P, P, I, F, I, I, P, P, P, P, L, I, I, P],
    "zi_latent_query_sums": [P, I, P, I, L, L, P, P, I, I, I, I, I, P],
    "zi_headwise_linear_gated": [P, I, L, I, P, I, L, I, P, I, I, I, I, P, I, L, I, L, P],
    "zi_tape_record": [P, c_char_p, P, I],
    "zi_tape_record_many": [P, c_char_p, P, P, I],
    "zi_tape_run": [P, P],
    "zi_tape_length": [P],
}


class KernelLibraryError(RuntimeError):
    pass


def library_path() -> Optional[str]:
    return _lib_path


def load() -> ctypes.CDLL:
    """The loaded library; builds it first when nothing built matches the sources."""
    global _lib, _lib_path
    if _lib is not None:
        return _lib
    with _lock:
        if _lib is not None:
            return _lib
        import torch  # noqa: F401  (loads the HIP runtime the library links against)
        from ..csrc.build import ensure_library
        try:
            path = ensure_library()
            lib = ctypes.CDLL(path)
        except (OSError, RuntimeError) as e:
            raise KernelLibraryError(f"cannot load the HIP kernel library: {e}") from e
        lib.zi_last_error.restype = c_char_p
        lib.zi_last_error.argtypes = []
        for name, args in _PROTOTYPES.items():
            try:
                fn = getattr(lib, name)
            except AttributeError as e:
                raise KernelLibraryError(f"{path} lacks entry point {name}; rebuild it") from e
            fn.argtypes = args
            fn.restype = c_int
        lib.zi_gemm_skinny_workspace.argtypes = [I, I, I]
        lib.zi_gemm_skinny_workspace.restype = c_int64
        lib.zi_attention_decode_workspace.argtypes = [I, I, I]
        lib.zi_attention_decode_workspace.restype = c_int64
        lib.zi_attention_prefill_workspace.argtypes = [I, I, I, I]
        lib.zi_attention_prefill_workspace.restype = c_int64
        lib.zi_decode_layer_workspace.argtypes = [I, I, I, I, I, I, I, I]
        lib.zi_decode_layer_workspace.restype = c_int64
        lib.zi_argmax_workspace.argtypes = [I, I]
        lib.zi_argmax_workspace.restype = c_int64
        lib.zi_tape_new.argtypes = []
        lib.zi_tape_new.restype = c_void_p
        lib.zi_tape_free.argtypes = [P]
        lib.zi_tape_free.restype = None
        _lib, _lib_path = lib, path
        return lib


# The calls made while a tape records (``ops.tape.Recording``): a list of (name, arguments), or None.
_recorded: Optional[list] = None


def call(name: str, *args) -> None:
    lib = load()
    rc = getattr(lib, name)(*args)
    if rc != 0:
        raise KernelLibraryError(lib.zi_last_error().decode("utf-8", "replace"))
    if _recorded is not None:
        _recorded.append((name, args))


def argument_words(name: str, args) -> list:
    """The arguments of a call as the 64-bit words a tape holds: integers and pointers by value, floats as
    the bits of a double."""
    kinds = _PROTOTYPES[name]
    if len(kinds) != len(args):
        raise KernelLibraryError(f"{name} takes {len(kinds)} arguments, {len(args)} were given")
    words = []
    for kind, a in zip(kinds, args):
        if kind is F:
            words.append(struct.unpack("<q", struct.pack("<d", float(a.value if isinstance(a, c_float) else a)))[0])
        elif kind is P:
            v = a.value if isinstance(a, c_void_p) else a
            if v is not None and not isinstance(v, int):
                raise KernelLibraryError(f"{name}: an argument of a kind a tape cannot hold ({type(a).__name__})")
            words.append(int(v or 0))
        else:
            words.append(int(a.value if hasattr(a, "value") else a))
    return words
