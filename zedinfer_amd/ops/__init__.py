"""The operators: thin, checked Python entries over the HIP kernels.

Each function checks devices, storage types, shapes and strides on the host,
then launches on torch's current stream.  The op-level names follow the
reference's Python module (reference: python/bindings/zedinfer_ops.cpp:257-291:
add, argmax, embedding, linear, rms_norm, rope, swiglu).
"""
from .functional import (add, add_rms_norm, argmax, attention, attention_decode, attention_decode_chunks,
                         attention_decode_fused,
                         attention_decode_fused_supported, attention_decode_project,
                         attention_decode_project_splits, attention_decode_project_supported,
                         attention_decode_merge_gated, attention_decode_supported, attention_decode_workspace, attention_prefill, attention_prefill_maps_supported,
                         attention_prefill_supported, attention_prefill_tile, attention_prefill_tile_min, attention_prefill_variant,
                         attention_prefill_workspace, compute_units, decode_layer, decode_layer_stamps, decode_layer_supported, decode_layer_sync_words,
                         decode_layer_workspace, device_synchronize, embedding, gather_rows, kv_store,
                         has_cuda, has_gpu, linear, linear_choose, linear_splits, linear_sums,
                         linear_sums_supported, linear_clamped_glu, linear_swiglu, linear_swiglu_supported,
                         linear_transposed, linear_tune, reduce_sums, rms_norm, rope, rope_inv_freq,
                         rope_kv_store, rope_kv_store_sums, rope_table, sample, swiglu, swiglu_t,
                         DECODE_LAYER_SPIN_LIMIT, FEW_ROWS, SUMS_MAX_ROWS)
from .mixing import (delta_conv_state, delta_prepare, delta_rule, delta_state_floats, gated_act, gated_rms_norm,
                     latent_attention, latent_attention_cores, latent_attention_cores_plan,
                     latent_attention_cores_supported, latent_attention_cores_workspace, latent_inputs, latent_query, latent_query_cores, latent_store, latent_value, latent_value_gates,
                     moe_combine, moe_group, moe_linear,
                     moe_max_tiles, moe_route, moe_tile_rows, rope_pairs)
from .sublayers import (clamped_glu, clamped_glu_il8, conv_qkv, conv_state_floats, conv_tail, convert, layer_norm, moe_route_top,
                        relu_squared, softcap)
from .recurrent import (attention_biased, embedding_sum, gate_heads, gated_rms_norm_act, linear_attention,
                        linear_attention_state_floats, lowrank_decay, moe_route_table, normed_kv_store, stream_reenter,
                        token_shift)
from .convolved import (channel_inputs, channel_state_floats, delta_channel, delta_channel_finishes, input_conv, lowrank_gates, norm_input_conv,
                        norm_input_conv_supported, stream_scale)
from . import hybrid
from .hybrid import (linear_attention_grouped, moe_route_sigmoid, moe_sum_shared, moe_weighted_glu, norm_rope_store,
                     normed_add_norm, pool_blocks, pooled_attention, pooled_attention_cores, pooled_attention_cores_cut, pooled_attention_cores_supported,
                     pooled_attention_cores_workspace,
                     rope_table_scaled, ssm_finish, ssm_prepare,
                     ssm_state_floats)
from .streams import (ACTIVATIONS, activate, difference_heads, difference_merge, head_norm_store, linear_activated, linear_activated_supported,
                      stream_mix, stream_mix_max_streams)
from ._lib import KernelLibraryError, library_path, load

__all__ = [
    "DECODE_LAYER_SPIN_LIMIT",
    "add", "add_rms_norm", "argmax", "attention", "attention_decode", "attention_decode_chunks", "attention_decode_fused",
    "attention_decode_fused_supported", "attention_decode_project", "attention_decode_project_splits",
    "attention_decode_project_supported", "attention_decode_supported", "attention_decode_workspace",
    "attention_prefill", "attention_prefill_supported", "attention_prefill_tile", "attention_prefill_tile_min", "attention_prefill_variant",
    "attention_prefill_workspace", "compute_units", "decode_layer", "decode_layer_stamps", "decode_layer_supported", "decode_layer_sync_words",
    "decode_layer_workspace", "device_synchronize", "embedding", "gather_rows", "has_cuda", "kv_store", "has_gpu",
    "linear", "linear_choose", "linear_splits", "linear_sums", "linear_sums_supported", "linear_swiglu",
    "linear_swiglu_supported", "linear_transposed", "linear_tune", "reduce_sums", "rms_norm", "rope",
    "rope_inv_freq", "rope_kv_store", "rope_kv_store_sums", "rope_table", "sample", "swiglu", "swiglu_t",
    "delta_conv_state", "delta_prepare", "delta_rule", "delta_state_floats", "gated_act", "gated_rms_norm",
    "latent_attention", "latent_attention_cores", "latent_attention_cores_plan", "latent_attention_cores_supported",
    "latent_attention_cores_workspace", "latent_query", "latent_store", "latent_value", "moe_combine", "moe_group", "moe_linear",
    "moe_max_tiles", "moe_route", "moe_tile_rows", "rope_pairs",
    "clamped_glu", "conv_qkv", "conv_state_floats", "conv_tail", "convert", "layer_norm", "moe_route_top", "relu_squared",
    "softcap",
    "attention_biased", "embedding_sum", "gate_heads", "gated_rms_norm_act", "linear_attention",
    "linear_attention_state_floats", "lowrank_decay", "moe_route_table", "normed_kv_store", "stream_reenter", "token_shift",
    "linear_attention_grouped", "moe_route_sigmoid", "moe_sum_shared", "moe_weighted_glu", "norm_rope_store",
    "normed_add_norm", "pool_blocks", "pooled_attention", "pooled_attention_cores", "pooled_attention_cores_cut", "pooled_attention_cores_supported", "pooled_attention_cores_workspace", "rope_table_scaled", "ssm_finish", "ssm_prepare", "ssm_state_floats",
    "channel_inputs", "channel_state_floats", "delta_channel", "delta_channel_finishes", "input_conv", "lowrank_gates", "norm_input_conv", "norm_input_conv_supported",
    "stream_scale", "attention_decode_merge_gated", "linear_clamped_glu", "clamped_glu_il8",
    "ACTIVATIONS", "activate", "attention_prefill_maps_supported", "difference_heads", "difference_merge", "head_norm_store", "latent_inputs", "linear_activated", "linear_activated_supported",
    "latent_query_cores", "latent_value_gates", "stream_mix", "stream_mix_max_streams",
    "KernelLibraryError", "library_path", "load", "FEW_ROWS", "SUMS_MAX_ROWS",
]
