"""ctypes binding of libmvhip.so (include/mvhip.h) for torch tensors.

This is the only place the Python host touches the C-ABI.  Every wrapper
launches on torch's *current* stream, so the calls are captured by
``torch.cuda.graph`` (= hipGraph) like any torch op.  There is no fallback:
if the shared library is missing, importing this module raises.
"""
from __future__ import annotations

import ctypes
import os
from ctypes import c_char_p, c_float, c_int, c_int64, c_size_t, c_uint64, c_void_p
from typing import NamedTuple

import torch

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "lib", "libmvhip.so")

MV_BF16, MV_F16, MV_F32 = 0, 1, 2
_DTYPES = {torch.bfloat16: MV_BF16, torch.float16: MV_F16, torch.float32: MV_F32}

# name -> (restype, argtypes); mirrors include/mvhip.h one-to-one
_SIGNATURES = {
    "mv_version": (c_int, []),
    "mv_strerror": (c_char_p, [c_int]),
    "mv_store_kvcache": (c_int, [c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_void_p,
                                 c_int, c_int, c_int, c_int64, c_int, c_void_p]),
    "mv_rmsnorm": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_int, c_float,
                           c_int, c_void_p]),
    "mv_add_rmsnorm": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_int64,
                               c_int, c_int, c_float, c_int, c_void_p]),
    "mv_add_rmsnorm_partial": (c_int, [c_void_p, c_int, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_int,
                                       c_float, c_int, c_void_p]),
    "mv_rope_qk_store": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_void_p,
                                 c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_float, c_void_p,
                                 c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int, c_int,
                                 c_int, c_int, c_void_p]),
    "mv_rope_qk_store_ex": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_int64, c_int64, c_void_p,
                                 c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_float, c_void_p,
                                 c_void_p, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int, c_int,
                                 c_int, c_int, c_void_p, c_void_p]),
    "mv_paged_decode_workspace_bytes": (c_size_t, [c_int, c_int, c_int, c_int, c_int, c_int, c_int]),
    "mv_paged_decode_workspace_bytes_ex": (c_size_t, [c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_void_p]),
    "mv_paged_decode": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_void_p,
                                c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_int64, c_float,
                                c_void_p, c_size_t, c_int, c_int, c_void_p]),
    "mv_paged_decode_ex": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_void_p,
                                c_void_p, c_int, c_int, c_int, c_int, c_int, c_int, c_int64, c_float,
                                c_void_p, c_size_t, c_int, c_int, c_void_p, c_void_p]),
    "mv_rope_paged_decode": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p,
                                     c_void_p, c_int64, c_void_p, c_void_p, c_float, c_void_p, c_void_p, c_void_p,
                                     c_void_p, c_int64, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int,
                                     c_int64, c_float, c_void_p, c_size_t, c_int, c_int, c_void_p]),
    "mv_rope_paged_decode_ex": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p,
                                     c_void_p, c_int64, c_void_p, c_void_p, c_float, c_void_p, c_void_p, c_void_p,
                                     c_void_p, c_int64, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int,
                                     c_int64, c_float, c_void_p, c_size_t, c_int, c_int, c_void_p, c_void_p]),
    "mv_prefill_varlen": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_void_p,
                                  c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_void_p,
                                  c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_float, c_int,
                                  c_int, c_void_p]),
    "mv_prefill_varlen_ex": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int64, c_void_p,
                                  c_void_p, c_void_p, c_int64, c_int64, c_void_p, c_void_p, c_void_p,
                                  c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_float, c_int,
                                  c_int, c_void_p, c_void_p]),
    "mv_sample_workspace_bytes": (c_size_t, [c_int, c_int]),
    "mv_sample": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p, c_uint64,
                          c_uint64, c_void_p, c_void_p, c_void_p, c_int, c_int, c_void_p, c_size_t,
                          c_int, c_void_p]),
    "mv_decode_advance": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_void_p]),
    "mv_silu_and_mul": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int, c_int, c_int, c_void_p]),
    "mv_gelu_and_mul": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int, c_int, c_int, c_void_p]),
    "mv_residual_update": (c_int, [c_void_p, c_int, c_int, c_int, c_int, c_void_p]),
    "mv_gated_lookup": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_int, c_void_p, c_void_p, c_int64, c_int,
                                c_int, c_int, c_int, c_void_p]),
    "mv_gated_lookup_linear": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int64, c_int, c_void_p, c_void_p, c_void_p,
                                       c_int64, c_int, c_int, c_int, c_int, c_int, c_void_p]),
    "mv_act_and_mul": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int, c_int, c_void_p, c_int, c_void_p]),
    "mv_latent_prep": (c_int, [c_void_p, c_int, c_int, c_void_p]),
    "mv_head_linear": (c_int, [c_void_p, c_int, c_int, c_void_p]),
    "mv_latent_gather": (c_int, [c_void_p, c_int64, c_int, c_int, c_void_p, c_int64, c_int, c_void_p, c_void_p, c_int, c_int,
                                 c_void_p, c_int, c_void_p]),
    "mv_latent_decode_workspace_bytes": (c_size_t, [c_int] * 8),
    "mv_latent_decode": (c_int, [c_void_p, c_void_p, c_void_p, c_int64, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int,
                                 c_int, c_int64, c_int, c_float, c_void_p, c_size_t, c_int, c_int, c_void_p]),
    "mv_latent_prefill": (c_int, [c_void_p, c_int, c_int, c_void_p]),
    "mv_causal_conv": (c_int, [c_void_p, c_int, c_void_p]),
    "mv_ssm_prefill": (c_int, [c_void_p, c_int, c_int, c_void_p]),
    "mv_ssm_step": (c_int, [c_void_p, c_int, c_void_p]),
    "mv_gated_group_norm": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_int, c_int, c_int,
                                    c_int, c_float, c_int, c_void_p]),
    "mv_delta_prefill_workspace_bytes": (c_size_t, [c_int] * 6),
    "mv_delta_prefill": (c_int, [c_void_p, c_int, c_int, c_void_p]),
    "mv_delta_step": (c_int, [c_void_p, c_int, c_void_p]),
    "mv_head_norm_gate": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_int, c_int, c_int,
                                  c_float, c_int, c_float, c_int, c_void_p]),
    "mv_moe_route": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_int, c_int, c_int,
                             c_float, c_int, c_int, c_void_p]),
    "mv_moe_group": (c_int, [c_void_p, c_int, c_int, c_int, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p]),
    "mv_gelu_erf": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_int, c_int, c_int, c_void_p]),
    "mv_stream_update": (c_int, [c_void_p, c_int, c_int, c_int, c_int, c_void_p]),
    "mv_gru_prefill_workspace_bytes": (c_size_t, [c_int] * 4),
    "mv_gru_prefill": (c_int, [c_void_p, c_int, c_void_p]),
    "mv_gru_step": (c_int, [c_void_p, c_int, c_void_p]),
    "mv_moe_linear": (c_int, [c_void_p, c_int, c_void_p]),
    "mv_gated_act_small_m": (c_int, [c_void_p, c_int64, c_void_p, c_int, c_void_p, c_int64, c_int, c_int, c_int, c_void_p,
                                     c_int, c_int, c_void_p]),
    "mv_gated_act_mid_m": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_int, c_int, c_void_p, c_int, c_int,
                                   c_void_p]),
    "mv_linear_small_m": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int,
                                  c_int, c_int, c_int, c_void_p]),
    "mv_gate_up_silu_small_m": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_int, c_int,
                                        c_int, c_int, c_void_p]),
    "mv_linear_small_m_packed": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int,
                                         c_int, c_int, c_int, c_void_p]),
    "mv_gate_up_silu_small_m_packed": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_int, c_int,
                                               c_int, c_int, c_void_p]),
    "mv_norm_linear_small_m_packed": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64, c_void_p,
                                              c_float, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int, c_int,
                                              c_int, c_int, c_void_p]),
    "mv_norm_gate_up_silu_small_m_packed": (c_int, [c_void_p, c_int64, c_void_p, c_int64, c_void_p, c_int64,
                                                    c_void_p, c_float, c_void_p, c_void_p, c_int64, c_int, c_int,
                                                    c_int, c_int, c_int, c_void_p]),
    "mv_packed_weight_elems": (c_size_t, [c_int, c_int]),
    "mv_pack_weight": (c_int, [c_void_p, c_void_p, c_int, c_int, c_int, c_void_p]),
    "mv_linear_mid_m": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_void_p, c_int64, c_int, c_int,
                                c_int, c_int, c_int, c_void_p]),
    "mv_gate_up_silu_mid_m": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int64, c_int, c_int, c_int,
                                      c_int, c_int, c_void_p]),
    "mv_linear_mid_m_partial": (c_int, [c_void_p, c_int64, c_void_p, c_void_p, c_int, c_int, c_int, c_int,
                                        c_int, c_int, c_void_p]),
    "mv_ar_region_bytes": (c_size_t, [c_size_t]),
    "mv_ar_max_world": (c_int, []),
    "mv_ar_alloc": (c_int, [c_size_t, c_void_p]),
    "mv_ar_free": (c_int, [c_void_p]),
    "mv_ar_ipc_handle_bytes": (c_int, []),
    "mv_ar_ipc_export": (c_int, [c_void_p, c_void_p]),
    "mv_ar_ipc_open": (c_int, [c_void_p, c_void_p]),
    "mv_ar_ipc_close": (c_int, [c_void_p]),
    "mv_ar_status": (c_int, [c_void_p, c_size_t, c_void_p]),
    "mv_ar_status_async": (c_int, [c_void_p, c_size_t, c_void_p, c_void_p]),
    "mv_ar_set_wait_limit_ms": (c_int, [c_void_p, c_size_t, ctypes.c_uint32]),
    "mv_ar_all_reduce": (c_int, [c_void_p, c_void_p, c_int64, c_void_p, c_int, c_int, c_size_t, c_int, c_void_p]),
    "mv_ar_all_reduce_add_rmsnorm": (c_int, [c_void_p, c_void_p, c_void_p, c_float, c_void_p, c_int, c_int, c_void_p,
                                             c_int, c_int, c_size_t, c_int, c_void_p]),
    "mv_greedy_pack": (c_int, [c_void_p, c_int64, c_void_p, c_int, c_int, c_int64, c_int, c_int, c_void_p, c_int,
                               c_void_p]),
    "mv_greedy_merge": (c_int, [c_void_p, c_int, c_int, c_int, c_void_p, c_int, c_void_p]),
    "mv_mass_pack": (c_int, [c_void_p, c_void_p, c_int, c_int, c_int64, c_int, c_int, c_void_p, c_int, c_void_p]),
    "mv_mass_merge": (c_int, [c_void_p, c_void_p, c_uint64, c_uint64, c_void_p, c_int, c_int, c_int, c_void_p, c_int,
                              c_void_p]),
    "mv_topc_width": (c_int, []),
    "mv_topc_pack": (c_int, [c_void_p, c_int64, c_int, c_int, c_int, c_int64, c_int, c_int, c_void_p, c_int, c_void_p]),
    "mv_topc_unpack": (c_int, [c_void_p, c_int, c_int, c_int, c_void_p, c_void_p, c_int, c_void_p]),
    "mv_shard_key_hist": (c_int, [c_void_p, c_int64, c_int, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_void_p]),
    "mv_nucleus_pick": (c_int, [c_void_p, c_int, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_void_p,
                                c_int, c_int, c_void_p]),
    "mv_mask_below": (c_int, [c_void_p, c_int64, c_int, c_int, c_void_p, c_void_p, c_int64, c_int, c_void_p]),
    "mv_topc_pick": (c_int, [c_void_p, c_void_p, c_void_p, c_void_p, c_void_p, c_int, c_int, c_int, c_void_p]),
    "mv_decode_layers_persistent_workspace_bytes": (c_size_t, [c_int, c_int, c_int, c_int, c_int, c_int, c_int, c_int]),
    "mv_decode_layers_persistent": (c_int, [c_void_p, c_int, c_void_p, c_void_p, c_size_t, c_void_p, c_int, c_int, c_void_p]),
    "mv_persist_struct_bytes": (c_size_t, [c_int]),
}
EXPORTED_SYMBOLS = tuple(_SIGNATURES)


class MvHipError(RuntimeError):
    pass


class MvAttnOpts(ctypes.Structure):
    """Options of the ``_ex`` attention entry points (include/mvhip.h)."""
    _fields_ = [("rot_pairs", c_int), ("interleaved", c_int), ("chunk", c_int), ("norm_dim", c_int), ("out_stride", c_int64),
                ("window", c_int), ("keep_first", c_int), ("softcap", c_float), ("out_scale", c_float), ("sink", c_void_p),
                ("gate", c_void_p), ("gate_stride", c_int64), ("unit_norm", c_int), ("reserved", c_int)]


class AttnMask(NamedTuple):
    """What a query sees and how its scores become weights (include/mvhip.h: MvAttnOpts): a window of positions with the first
    ``keep_first`` tokens kept, capped scores, a factor of the output, one more term per head in the softmax denominator, a gate
    (rows [N, heads * D], one per query: the output is multiplied by its sigmoid)."""
    window: int = 0
    keep_first: int = 0
    softcap: float = 0.0
    out_scale: float = 1.0
    sink: torch.Tensor | None = None
    gate: torch.Tensor | None = None


NO_MASK = AttnMask()


class MvResidualArgs(ctypes.Structure):
    _fields_ = [("x", c_void_p), ("y", c_void_p), ("y_norm_w", c_void_p), ("embed", c_void_p), ("ids", c_void_p),
                ("vec", c_void_p), ("norm_w", c_void_p), ("out", c_void_p), ("y_stride", c_int64), ("out_stride", c_int64),
                ("vocab", c_int64), ("embed_scale", c_float), ("norm_offset", c_float), ("eps", c_float),
                ("y_splits", c_int), ("embed_mode", c_int), ("y_mult", c_float), ("y_scale", c_void_p),
                ("y_norm_b", c_void_p), ("norm_b", c_void_p), ("pairs", c_void_p), ("positions", c_void_p),
                ("state_slots", c_void_p), ("cu_q", c_void_p), ("prev_tokens", c_void_p), ("moe_out", c_void_p),
                ("moe_rows", c_void_p), ("moe_w", c_void_p), ("buckets", c_int64), ("mul_prev", c_int64), ("mul_cur", c_int64),
                ("slots", c_int64), ("layer_norm", c_int), ("n_seqs", c_int), ("moe_top", c_int), ("reserved", c_int)]


class GateAct(ctypes.Structure):
    """Activation of a gated projection with its constants (include/mvhip.h: MvGateAct)."""
    _fields_ = [("kind", c_int), ("limit", c_float), ("alpha", c_float)]


RELU_GLU = GateAct(3, 0.0, 0.0)     # max(gate, 0) * up
MV_LINEAR_GELU_ERF = 1 << 18        # plain projections: 0.5 y (1 + erf(y / sqrt(2))) in the epilogue


def clamped_glu(limit: float, alpha: float = 1.702) -> GateAct:
    """g = min(gate, limit), u = clamp(up, -limit, limit): g * sigmoid(alpha * g) * (u + 1)."""
    return GateAct(2, float(limit), float(alpha))


def _struct(name: str, **fields):
    return type(name, (ctypes.Structure,), {"_fields_": [(f, t) for k, t in fields.items() for f in k.split("__")]})


# include/mvhip.h, field for field
MvLatentPrepArgs = _struct(
    "MvLatentPrepArgs", z=c_void_p, z_stride=c_int64, q_norm_w__kv_norm_w__q_out=c_void_p, q_out_stride=c_int64,
    rows_out__plane__slot_mapping=c_void_p, num_slots=c_int64, positions__cos__sin=c_void_p, max_pos=c_int64,
    q_off__q_rank__q_cols__kv_off__kv_rank__kv_cols__rot_off__rot_dim__rot_cols=c_int, eps=c_float)
MvHeadLinearArgs = _struct(
    "MvHeadLinearArgs", x__w__out=c_void_p, x_tok__x_head__out_tok__out_head=c_int64, positions__cos__sin=c_void_p,
    max_pos=c_int64, heads__n__k__rot_dim__rot_cols=c_int)
MvLatentPrefillArgs = _struct(
    "MvLatentPrefillArgs", q__k__v__rot__out=c_void_p, q_stride__k_stride__v_stride__rot_stride__out_stride=c_int64,
    cu_q__cu_k__positions__cos__sin=c_void_p, max_pos=c_int64,
    n_seqs__max_q__max_k__heads__plain_cols__rot_dim__rot_cols__dq__dv__window=c_int, scale=c_float)
MvSsmArgs = _struct(
    "MvSsmArgs", x=c_void_p, x_stride=c_int64, dt=c_void_p, dt_stride=c_int64,
    conv_w__conv_b__dt_bias__a_log__d__conv_state__ssm_state__state_slots__cu_q__cu_k__context_lens__out=c_void_p,
    out_stride__slots=c_int64, n_seqs__max_q__channels__taps__heads__groups__p__n__b_off__c_off=c_int)


MvDeltaArgs = _struct(
    "MvDeltaArgs", x__beta__a__gate__conv_w__dt_bias__a_log__norm_w__conv_state__state__state_slots__cu_q__cu_k__context_lens__out__workspace=c_void_p,
    x_stride__beta_stride__a_stride__gate_stride__out_stride__slots__ws_bytes=c_int64,
    n_seqs__max_q__total_q__channels__taps__heads__groups__p__p_true__n__k_off__q_off__channel_decay__gate_kind=c_int,
    eps__unit_eps__q_scale__out_scale=c_float)
MvMoeLinearArgs = _struct(
    "MvMoeLinearArgs", x__w__out__tokens__tiles__act__in_scale=c_void_p, x_stride__out_stride=c_int64, max_tiles__tile_m__n__k=c_int)


MvStreamArgs = _struct(
    "MvStreamArgs", x__x_out__y__mix__out_w__embed__ids__in_w__norm_w__shift__out__moe_out__moe_rows__moe_w__prev__positions__state_slots__cu_q=c_void_p,
    y_stride__out_stride__vocab__slots=c_int64, streams__y_splits__moe_top__n_seqs=c_int, eps=c_float, reserved=c_int)
MvGruArgs = _struct(
    "MvGruArgs", z__u__g__state__state_slots__cu_q__cu_k__context_lens__out__workspace=c_void_p,
    stride__out_stride__slots__ws_bytes=c_int64, n_seqs__max_q__total_q__n=c_int)


def _attn_opts(interleaved_pairs=None, chunk: int = 0, out=None, mask: AttnMask | None = None, norm_dim: int = 0, like=None,
               unit_norm: bool = False):
    """``interleaved_pairs``: None = rotary halves, n = interleaved layout with n rotated pairs; ``chunk``: chunk size of
    the causal mask (0 = whole context); ``out``: output tensor [rows, H, D] whose rows may be strided; ``norm_dim``: columns that
    the head norms are means over (0 = all); ``like``: q, whose dtype and heads the mask's sink must have, whose rows and columns its
    gate must have; ``unit_norm``: q and k divided by their rms behind the rotation."""
    il, m = interleaved_pairs is not None, mask or NO_MASK
    _need_cuda(m.sink)
    if m.sink is not None and like is not None and (m.sink.dtype != like.dtype or m.sink.numel() != like.shape[1]
                                                    or not m.sink.is_contiguous()):
        raise MvHipError(f"sink: a number of {like.dtype} per head required")
    if m.gate is not None and like is not None and (m.gate.dtype != like.dtype or m.gate.stride(1) != 1 or m.gate.shape[0] < like.shape[0]
                                                    or m.gate.shape[1] < like.shape[1] * like.shape[2]):
        raise MvHipError(f"gate: a row of {like.shape[1] * like.shape[2]} {like.dtype} per query required")
    o = MvAttnOpts(int(interleaved_pairs) if il else 0, int(il), int(chunk), int(norm_dim), out.stride(0) if out is not None else 0,
                   int(m.window), int(m.keep_first), float(m.softcap), float(m.out_scale), _ptr(m.sink), _ptr(m.gate),
                   m.gate.stride(0) if m.gate is not None else 0, int(unit_norm))
    return ctypes.byref(o)


def _out_rows(out, rows: int, h: int, d: int):
    if out.shape != (rows, h, d) or out.stride(2) != 1 or out.stride(1) != d:
        raise MvHipError(f"output must be [{rows}, {h}, {d}] and dense in its last two dims")
    return out


# ---------------------------------------------------------------- tuning switches
# The C-ABI reads no environment: the overrides below are read HERE, once, and passed as explicit arguments.
MV_DECODE_VECTOR, MV_DECODE_MFMA, MV_DECODE_KLDS_OFF, MV_DECODE_KLDS_ON, MV_DECODE_PER_HEAD = 1, 2, 4, 8, 16
MV_PREFILL_SIMPLE = 1
MV_E_SHAPE = -2   # include/mvhip.h


def _decode_flags_from_env() -> int:
    """MV_DECODE_MFMA_MIN_G=1 / 99: matrix-core decode kernel always / never; MV_DECODE_MFMA_KLDS=0 / 1: K straight
    to registers / through LDS; MV_DECODE_PER_HEAD=1: vector kernel with one kv head per workgroup;
    MV_DECODE_TARGET_WGS=n: workgroups the context split aims for (multiple of 16).
    (Bench and debugging aids; unset = the kernels choose from the shape.)"""
    f = 0
    g = os.environ.get("MV_DECODE_MFMA_MIN_G")
    if g is not None:
        f |= MV_DECODE_MFMA if int(g) <= 1 else (MV_DECODE_VECTOR if int(g) >= 17 else 0)
    k = os.environ.get("MV_DECODE_MFMA_KLDS")
    if k is not None:
        f |= MV_DECODE_KLDS_ON if int(k) else MV_DECODE_KLDS_OFF
    if os.environ.get("MV_DECODE_PER_HEAD") == "1":
        f |= MV_DECODE_PER_HEAD
    t = os.environ.get("MV_DECODE_TARGET_WGS")
    if t is not None:
        f |= (max(1, min(255, int(t) // 16))) << 8
    return f


DECODE_FLAGS = _decode_flags_from_env()
PREFILL_FLAGS = MV_PREFILL_SIMPLE if os.environ.get("MV_PREFILL_FORCE_SIMPLE") == "1" else 0


def _load():
    if not os.path.exists(LIB_PATH):
        raise MvHipError(
            f"{LIB_PATH} is missing: the HIP extension is not built. Run "
            "`python -c 'import __graft_entry__ as g; g.build()'` (or `make -C mini-vllm_amd/csrc`). "
            "There is no CPU fallback for the GPU hot path."
        )
    lib = ctypes.CDLL(LIB_PATH)
    for name, (res, args) in _SIGNATURES.items():
        fn = getattr(lib, name)  # AttributeError => ABI mismatch, fail loudly
        fn.restype = res
        fn.argtypes = args
    return lib


_lib = _load()


def lib():
    return _lib


def version() -> int:
    return int(_lib.mv_version())


def _check(code: int, what: str) -> None:
    if code != 0:
        msg = _lib.mv_strerror(code)
        raise MvHipError(f"{what} failed: [{code}] {msg.decode() if msg else '?'}")


def _dt(t: torch.Tensor) -> int:
    try:
        return _DTYPES[t.dtype]
    except KeyError:
        raise MvHipError(f"unsupported dtype {t.dtype}") from None


def _ptr(t):
    return None if t is None else t.data_ptr()


def _stream() -> int:
    return torch.cuda.current_stream().cuda_stream


def _need_cuda(*ts):
    for t in ts:
        if t is not None and not t.is_cuda:
            raise MvHipError("libmvhip kernels need device tensors (got a CPU tensor); "
                             "the product path has no CPU fallback")


def _i32(t):
    if t is None:
        return None
    return t if t.dtype == torch.int32 else t.to(torch.int32)


# ---------------------------------------------------------------- workspace
_workspace: dict[int, torch.Tensor] = {}
_workspace_retired: list[torch.Tensor] = []   # outgrown buffers stay alive: captured graphs hold their pointers


def workspace(nbytes: int, device) -> torch.Tensor:
    """Grow-only per-device scratch buffer (allocate before graph capture).  A buffer that is outgrown is never
    freed: a hipGraph captured earlier still reads and writes it (split-KV partials), and handing its memory
    back to the caching allocator would let another tensor land under a replaying graph."""
    idx = torch.device(device).index or 0
    buf = _workspace.get(idx)
    if buf is None or buf.numel() < nbytes:
        if buf is not None:
            _workspace_retired.append(buf)
        # generous first allocation: captured graphs hold this pointer, so it should not have to move later
        buf = torch.empty(max(int(nbytes), 32 << 20), dtype=torch.uint8, device=device)
        _workspace[idx] = buf
    return buf


# ---------------------------------------------------------------- K1
def store_kvcache(key, value, k_cache, v_cache, slot_mapping) -> None:
    """key/value [N,Hkv,D] (last two dims dense), caches [nb,bs,Hkv,D] contiguous."""
    _need_cuda(key, value, k_cache, v_cache, slot_mapping)
    n, hkv, d = key.shape
    if slot_mapping.numel() != n:
        raise ValueError(f"slot_mapping size {slot_mapping.numel()} != batch_size {n}")
    if key.stride(-1) != 1 or key.stride(1) != d or value.stride(-1) != 1 or value.stride(1) != d:
        raise MvHipError("key/value must be dense in their last two dims")
    if key.dtype != k_cache.dtype:
        key, value = key.to(k_cache.dtype), value.to(v_cache.dtype)
    if not (k_cache.is_contiguous() and v_cache.is_contiguous()):
        raise MvHipError("KV cache must be contiguous")
    num_slots = k_cache.numel() // (hkv * d)
    _check(_lib.mv_store_kvcache(key.data_ptr(), value.data_ptr(), key.stride(0), value.stride(0),
                                 k_cache.data_ptr(), v_cache.data_ptr(), _i32(slot_mapping).data_ptr(),
                                 n, hkv, d, num_slots, _dt(k_cache), _stream()), "mv_store_kvcache")


# ---------------------------------------------------------------- K6
def _rows2d(x):
    cols = x.shape[-1]
    if x.stride(-1) != 1:
        x = x.contiguous()
    x2 = x.reshape(-1, cols)  # view when possible
    return x2, cols


def rmsnorm(x, weight, eps: float):
    _need_cuda(x, weight)
    x2, cols = _rows2d(x)
    out = torch.empty((x2.shape[0], cols), dtype=x.dtype, device=x.device)
    w = weight if weight.dtype == x.dtype else weight.to(x.dtype)
    _check(_lib.mv_rmsnorm(x2.data_ptr(), x2.stride(0), w.data_ptr(), out.data_ptr(), out.stride(0),
                           x2.shape[0], cols, float(eps), _dt(x), _stream()), "mv_rmsnorm")
    return out.view(x.shape)


def add_rmsnorm(x, residual, weight, eps: float, inplace: bool = True):
    """Returns (normed, new_residual).  With inplace=True ``residual`` is overwritten
    by the rounded sum (the reference allocates a new tensor, layernorm.py:95-105)."""
    _need_cuda(x, residual, weight)
    x2, cols = _rows2d(x)
    res = residual if inplace else residual.clone()
    if not res.is_contiguous():
        res = res.contiguous()
    r2 = res.view(-1, cols)
    out = torch.empty((x2.shape[0], cols), dtype=x.dtype, device=x.device)
    w = weight if weight.dtype == x.dtype else weight.to(x.dtype)
    _check(_lib.mv_add_rmsnorm(x2.data_ptr(), x2.stride(0), r2.data_ptr(), r2.stride(0), w.data_ptr(),
                               out.data_ptr(), out.stride(0), x2.shape[0], cols, float(eps), _dt(x),
                               _stream()), "mv_add_rmsnorm")
    return out.view(x.shape), res.view(residual.shape)


def add_rmsnorm_partial(partial, residual, weight, eps: float):
    """``add_rmsnorm`` whose x is the sum of fp32 K-split partials [S, rows, cols] (linear_mid_m_partial);
    residual is updated in place.  Returns (normed, residual)."""
    _need_cuda(partial, residual, weight)
    s, rows, cols = partial.shape
    if partial.dtype != torch.float32 or not partial.is_contiguous() or not residual.is_contiguous():
        raise MvHipError("partial sums must be contiguous fp32, the residual contiguous")
    r2 = residual.view(-1, cols)
    out = torch.empty((rows, cols), dtype=residual.dtype, device=residual.device)
    w = weight if weight.dtype == residual.dtype else weight.to(residual.dtype)
    _check(_lib.mv_add_rmsnorm_partial(partial.data_ptr(), s, r2.data_ptr(), r2.stride(0), w.data_ptr(),
                                       out.data_ptr(), out.stride(0), rows, cols, float(eps), _dt(residual),
                                       _stream()), "mv_add_rmsnorm_partial")
    return out.view(residual.shape), residual


# ---------------------------------------------------------------- K7
def _rot_tables_ok(cos, sin, d: int, interleaved_pairs) -> bool:
    """cos / sin are dense fp32 [max_pos, rotated pairs] tables (none if nothing is rotated)."""
    if interleaved_pairs == 0:
        return True
    want = d // 2 if interleaved_pairs is None else int(interleaved_pairs)
    return (cos.shape == sin.shape and cos.dim() == 2 and cos.shape[1] == want and cos.is_contiguous() and sin.is_contiguous()
            and cos.dtype == torch.float32 and sin.dtype == torch.float32)


def rope_qk_store(q, k, v, positions, cos, sin, q_norm_w=None, k_norm_w=None, eps: float = 1e-6,
                  k_cache=None, v_cache=None, slot_mapping=None, want_k_out: bool = True, interleaved_pairs=None,
                  norm_dim: int = 0, unit_norm: bool = False):
    """q [T,H,D], k/v [T,Hkv,D] (views of the qkv GEMM output are fine).
    ``interleaved_pairs``: n = the interleaved layout on the first 2n dims (cos / sin [max_pos, n]); None = halves.  ``unit_norm``:
    q and k are divided by their rms behind the rotation (no weights).
    Returns (q_rot [T,H,D], k_rot [T,Hkv,D] or None)."""
    _need_cuda(q, k, positions, cos, sin)
    t, h, d = q.shape
    hkv = k.shape[1]
    for name, x in (("q", q), ("k", k), ("v", v)):
        if x is not None and (x.stride(-1) != 1 or x.stride(1) != d):
            raise MvHipError(f"{name} must be dense in its last two dims")
    q_out = torch.empty((t, h, d), dtype=q.dtype, device=q.device)
    k_out = torch.empty((t, hkv, d), dtype=q.dtype, device=q.device) if want_k_out else None
    has_cache = k_cache is not None and k_cache.numel() > 0 and slot_mapping is not None \
        and slot_mapping.numel() > 0
    num_slots = 0
    if has_cache:
        if k_cache.dtype != q.dtype:
            raise MvHipError("q/k/v dtype must equal the KV-cache dtype")
        num_slots = k_cache.numel() // (hkv * d)
        if slot_mapping.numel() != t:
            raise ValueError(f"slot_mapping size {slot_mapping.numel()} != batch_size {t}")
    pos = positions if positions.dtype == torch.int64 else positions.to(torch.int64)
    qn = q_norm_w if q_norm_w is None or q_norm_w.dtype == q.dtype else q_norm_w.to(q.dtype)
    kn = k_norm_w if k_norm_w is None or k_norm_w.dtype == q.dtype else k_norm_w.to(q.dtype)
    if not _rot_tables_ok(cos, sin, d, interleaved_pairs):
        raise MvHipError(f"cos / sin: dense fp32 [max_pos, rotated pairs] tables required, got {tuple(cos.shape)}")
    _check(_lib.mv_rope_qk_store_ex(
        q.data_ptr(), k.data_ptr(), _ptr(v), q.stride(0), k.stride(0), v.stride(0) if v is not None else 0,
        pos.data_ptr(), _ptr(cos), _ptr(sin), 0 if cos is None else cos.shape[0], _ptr(qn), _ptr(kn), float(eps),
        q_out.data_ptr(), _ptr(k_out),
        k_cache.data_ptr() if has_cache else None, v_cache.data_ptr() if has_cache else None,
        _i32(slot_mapping).data_ptr() if has_cache else None, num_slots, t, h, hkv, d, _dt(q),
        _attn_opts(interleaved_pairs, norm_dim=norm_dim, unit_norm=unit_norm), _stream()), "mv_rope_qk_store")
    return q_out, k_out


# ---------------------------------------------------------------- K3
def paged_decode_workspace_bytes(batch, n_heads, n_kv_heads, head_dim, block_size, max_blocks,
                                 flags: int | None = None, chunk: int = 0, mask: AttnMask | None = None) -> int:
    return int(_lib.mv_paged_decode_workspace_bytes_ex(batch, n_heads, n_kv_heads, head_dim, block_size,
                                                       max_blocks, DECODE_FLAGS if flags is None else flags,
                                                       _attn_opts(None, chunk, mask=mask)))


def paged_decode(q, k_cache, v_cache, block_tables, context_lens, scale: float, out=None, flags: int | None = None,
                 chunk: int = 0, mask: AttnMask | None = None):
    """q [B,H,D]; caches [nb,bs,Hkv,D]; block_tables int [B,nblk] (row-strided view ok);
    context_lens int [B].  ``chunk``: > 0 = only the keys of the last token's chunk of positions.  Returns [B,H,D] in
    q's dtype (``out``: a row-strided view is fine)."""
    _need_cuda(q, k_cache, v_cache, block_tables, context_lens)
    b, h, d = q.shape
    if q.stride(-1) != 1 or q.stride(1) != d:
        q = q.contiguous()
    if out is None:
        out = torch.empty((b, h, d), dtype=q.dtype, device=q.device)
    _out_rows(out, b, h, d)
    nb, bs, hkv = k_cache.shape[0], k_cache.shape[1], k_cache.shape[2]
    bt = _i32(block_tables)
    if bt.dim() != 2 or (bt.shape[1] > 0 and bt.stride(1) != 1):
        bt = bt.contiguous()
    cl = _i32(context_lens)
    max_blocks = bt.shape[1]
    flags = DECODE_FLAGS if flags is None else flags
    ws_bytes = paged_decode_workspace_bytes(b, h, hkv, d, bs, max_blocks, flags, chunk, mask)
    ws = workspace(ws_bytes, q.device)
    _check(_lib.mv_paged_decode_ex(q.data_ptr(), q.stride(0), k_cache.data_ptr(), v_cache.data_ptr(),
                                bt.data_ptr(), bt.stride(0) if max_blocks else 0, cl.data_ptr(),
                                out.data_ptr(), b, h, hkv, d, bs, max_blocks, nb, float(scale),
                                ws.data_ptr(), ws.numel(), _dt(q), flags, _attn_opts(None, chunk, out, mask, like=q),
                                   _stream()), "mv_paged_decode")
    return out


# ---------------------------------------------------------------- K2
def rope_paged_decode(q, k, v, positions, cos, sin, q_norm_w, k_norm_w, eps: float, slot_mapping,
                      k_cache, v_cache, block_tables, context_lens, scale: float, flags: int | None = None,
                      interleaved_pairs=None, chunk: int = 0, out=None, mask: AttnMask | None = None, norm_dim: int = 0,
                      unit_norm: bool = False):
    """Decode step of one layer in ONE launch: q [B,H,D], k/v [B,Hkv,D] RAW rows of the qkv projection (views are
    fine) -> per-head RMSNorm (weights or None) + RoPE on q and k, the new K/V rows stored at ``slot_mapping``, paged
    attention over ``block_tables`` / ``context_lens`` (which count the new token).  Returns [B,H,D], or None when
    the fused kernel does not take the layout (the caller then runs rope_qk_store + paged_decode)."""
    _need_cuda(q, k, v, k_cache, v_cache, block_tables, context_lens, slot_mapping)
    b, h, d = q.shape
    hkv = k.shape[1]
    nb, bs = k_cache.shape[0], k_cache.shape[1]
    if q.dtype not in (torch.bfloat16, torch.float16) or k_cache.dtype != q.dtype or slot_mapping.numel() != b:
        return None
    for x in (q, k, v):
        if x.stride(-1) != 1 or x.stride(1) != d:
            return None
    bt, cl = _i32(block_tables), _i32(context_lens)
    if bt.dim() != 2 or bt.stride(1) != 1 or bt.shape[1] == 0:
        return None
    flags = DECODE_FLAGS if flags is None else flags
    ws_bytes = paged_decode_workspace_bytes(b, h, hkv, d, bs, bt.shape[1], flags, chunk, mask)
    ws = workspace(ws_bytes, q.device)
    if out is None:
        out = torch.empty((b, h, d), dtype=q.dtype, device=q.device)
    _out_rows(out, b, h, d)
    if not _rot_tables_ok(cos, sin, d, interleaved_pairs):
        return None
    pos = positions if positions.dtype == torch.int64 else positions.to(torch.int64)
    qn = q_norm_w if q_norm_w is None or q_norm_w.dtype == q.dtype else q_norm_w.to(q.dtype)
    kn = k_norm_w if k_norm_w is None or k_norm_w.dtype == q.dtype else k_norm_w.to(q.dtype)
    rc = _lib.mv_rope_paged_decode_ex(
        q.data_ptr(), q.stride(0), k.data_ptr(), k.stride(0), v.data_ptr(), v.stride(0), pos.data_ptr(),
        _ptr(cos), _ptr(sin), 0 if cos is None else cos.shape[0], _ptr(qn), _ptr(kn), float(eps), _i32(slot_mapping).data_ptr(),
        k_cache.data_ptr(), v_cache.data_ptr(), bt.data_ptr(), bt.stride(0), cl.data_ptr(), out.data_ptr(), b, h, hkv,
        d, bs, bt.shape[1], nb, float(scale), ws.data_ptr(), ws.numel(), _dt(q), flags,
        _attn_opts(interleaved_pairs, chunk, out, mask, norm_dim, q, unit_norm), _stream())
    if rc == MV_E_SHAPE:
        return None
    _check(rc, "mv_rope_paged_decode")
    return out


def prefill_varlen(q, k, v, cu_seqlens_q, cu_seqlens_k, max_seqlen_q, max_seqlen_k, scale: float,
                   k_cache=None, v_cache=None, block_tables=None, out=None, flags: int | None = None,
                   chunk: int = 0, mask: AttnMask | None = None):
    """Packed causal prefill.  Contiguous K/V (k,v [Tk,Hkv,D]) unless ``block_tables`` is
    given, in which case keys come from the paged caches (prefix-cache hit).  ``chunk``: > 0 = a query sees only the
    keys of its own chunk of positions."""
    _need_cuda(q, cu_seqlens_q, cu_seqlens_k)
    t, h, d = q.shape
    if q.stride(-1) != 1 or q.stride(1) != d:
        q = q.contiguous()
    if out is None:
        out = torch.empty((t, h, d), dtype=q.dtype, device=q.device)
    _out_rows(out, t, h, d)
    n_seqs = cu_seqlens_q.numel() - 1
    paged = block_tables is not None
    if paged:
        nb, bs, hkv = k_cache.shape[0], k_cache.shape[1], k_cache.shape[2]
        bt = _i32(block_tables)
        if bt.stride(1) != 1:
            bt = bt.contiguous()
        args_kv = (None, None, 0, 0, k_cache.data_ptr(), v_cache.data_ptr(), bt.data_ptr(), bt.stride(0), nb)
    else:
        hkv = k.shape[1]
        bs = 0
        for name, x in (("k", k), ("v", v)):
            if x.stride(-1) != 1 or x.stride(1) != d:
                raise MvHipError(f"{name} must be dense in its last two dims")
        args_kv = (k.data_ptr(), v.data_ptr(), k.stride(0), v.stride(0), None, None, None, 0, 0)
    _check(_lib.mv_prefill_varlen_ex(q.data_ptr(), q.stride(0), *args_kv, out.data_ptr(),
                                  _i32(cu_seqlens_q).data_ptr(), _i32(cu_seqlens_k).data_ptr(), n_seqs,
                                  int(max_seqlen_q), int(max_seqlen_k), h, hkv, d, bs, float(scale),
                                  _dt(q), PREFILL_FLAGS if flags is None else flags,
                                     _attn_opts(None, chunk, out, mask, like=q), _stream()), "mv_prefill_varlen")
    return out


# ---------------------------------------------------------------- K8
def sample(logits, temperatures, top_ks, top_ps, min_ps, seed: int = 0, offset: int = 0,
           offset_dev=None, return_mask: bool = False, return_stats: bool = False):
    """logits [B,V]; per-row params [B].  Returns int64 tokens [B] (and the uint8 keep mask; and, with
    ``return_stats``, fp32 [B, 2] = {row maximum, kept mass}: the input of ``mass_pack``)."""
    _need_cuda(logits, temperatures, top_ks, top_ps, min_ps)
    b, v = logits.shape
    if logits.stride(-1) != 1:
        logits = logits.contiguous()
    out = torch.empty((b,), dtype=torch.int64, device=logits.device)
    mask = torch.empty((b, v), dtype=torch.uint8, device=logits.device) if return_mask else None
    stats = torch.empty((b, 2), dtype=torch.float32, device=logits.device) if return_stats else None

    def f32(x):
        return None if x is None else (x if x.dtype == torch.float32 else x.float())
    tk = None if top_ks is None else (top_ks if top_ks.dtype == torch.int64 else top_ks.to(torch.int64))
    temperatures, top_ps, min_ps = f32(temperatures), f32(top_ps), f32(min_ps)
    _check(_lib.mv_sample(logits.data_ptr(), logits.stride(0), _ptr(temperatures), _ptr(tk), _ptr(top_ps),
                          _ptr(min_ps), int(seed) & (2**64 - 1), int(offset) & (2**64 - 1),
                          _ptr(offset_dev), out.data_ptr(), _ptr(mask), b, v, _ptr(stats), 8 * b if return_stats else 0,
                          _dt(logits), _stream()), "mv_sample")
    if return_stats:
        return (out, mask, stats) if return_mask else (out, stats)
    return (out, mask) if return_mask else out


# ---------------------------------------------------------------- K9
GATE_ACTS = {"silu": 0, "gelu_tanh": 1 << 16}    # include/mvhip.h: MV_GATE_GELU


def _gated_out(out, rows: int, n: int, x):
    if out is None:
        return torch.empty((rows, n), dtype=x.dtype, device=x.device)
    if tuple(out.shape) != (rows, n) or out.dtype != x.dtype or out.stride(1) != 1:
        raise MvHipError(f"act(gate) * up: out must be [{rows}, {n}] rows of {x.dtype}")
    return out


def silu_and_mul(x, out=None):
    _need_cuda(x)
    if x.size(-1) % 2 != 0:
        raise ValueError(f"Input last dimension must be even for SiluAndMul, got {x.size(-1)}")
    x2, cols2 = _rows2d(x)
    cols = cols2 // 2
    given, out = out, _gated_out(out, x2.shape[0], cols, x)
    _check(_lib.mv_silu_and_mul(x2.data_ptr(), x2.stride(0), out.data_ptr(), out.stride(0), x2.shape[0],
                                cols, _dt(x), _stream()), "mv_silu_and_mul")
    return out if given is not None else out.view(*x.shape[:-1], cols)


def gelu_and_mul(x, out=None):
    """x [rows, 2 * cols] (row-strided view ok) -> gelu_tanh(x[:, :cols]) * x[:, cols:]; ``out`` may be row-strided."""
    _need_cuda(x)
    if x.dim() != 2 or x.stride(1) != 1 or x.shape[1] % 2:
        raise ValueError(f"gelu_and_mul wants [rows, 2 * cols] rows, got {tuple(x.shape)}")
    rows, cols = x.shape[0], x.shape[1] // 2
    out = _gated_out(out, rows, cols, x)
    _check(_lib.mv_gelu_and_mul(x.data_ptr(), x.stride(0), out.data_ptr(), out.stride(0), rows, cols, _dt(x), _stream()),
           "mv_gelu_and_mul")
    return out


def act_and_mul(x, act, out=None):
    """x [rows, 2 * cols] (row-strided view ok) -> act(x[:, :cols], x[:, cols:]); ``act``: "silu", "gelu_tanh" or a GateAct."""
    if not isinstance(act, GateAct):
        return (silu_and_mul if act == "silu" else gelu_and_mul)(x, out=out)
    _need_cuda(x)
    if x.dim() != 2 or x.stride(1) != 1 or x.shape[1] % 2:
        raise ValueError(f"act_and_mul wants [rows, 2 * cols] rows, got {tuple(x.shape)}")
    rows, cols = x.shape[0], x.shape[1] // 2
    out = _gated_out(out, rows, cols, x)
    _check(_lib.mv_act_and_mul(x.data_ptr(), x.stride(0), out.data_ptr(), out.stride(0), rows, cols, ctypes.byref(act), _dt(x),
                               _stream()), "mv_act_and_mul")
    return out


def gelu_erf(x, out=None):
    """0.5 x (1 + erf(x / sqrt(2))) of rows [rows, cols] (row-strided view ok; ``out`` may be x)."""
    _need_cuda(x, out)
    if x.dim() != 2 or x.stride(1) != 1:
        raise ValueError(f"gelu_erf wants [rows, cols] rows, got {tuple(x.shape)}")
    out = _gated_out(out, x.shape[0], x.shape[1], x)
    _check(_lib.mv_gelu_erf(x.data_ptr(), x.stride(0), out.data_ptr(), out.stride(0), x.shape[0], x.shape[1], _dt(x), _stream()),
           "mv_gelu_erf")
    return out


# ---------------------------------------------------------------- K13
def residual_update(x, y=None, y_norm_w=None, embed=None, ids=None, embed_scale: float = 1.0, start: bool = False,
                    vec=None, norm_w=None, norm_offset: float = 0.0, eps: float = 0.0, cols_true: int | None = None,
                    out=None, want_out: bool = True, dtype=None, y_scale=None, y_mult: float = 1.0, y_norm_b=None, norm_b=None,
                    layer_norm: bool = False, pairs=None, experts=None):
    """One edge of the fp32 residual stream ``x`` [rows, cols] (updated in place; include/mvhip.h: mv_residual_update).
    ``y``: [rows, cols] of the activation dtype, or fp32 K-split partial sums [splits, rows, cols]; ``y_norm_w``: its RMS
    norm; ``y_scale`` (a vector) and ``y_mult`` multiply it.  ``embed`` / ``ids``: the scaled embedding is added (``start``: the row starts from it).  ``vec``: added to every
    row.  ``layer_norm``: both norms are layer norms, with biases ``y_norm_b`` / ``norm_b``.  ``pairs`` (a ``PairTable``): a row
    per (previous token, token) is added where the embedding is.  ``experts`` (rows [pairs, cols], place per pair, weight per pair):
    y also gets the weighted rows of a token's choices, place < 0 standing for x itself.  Returns rms(x) * (norm_offset + norm_w), or x cast to ``dtype`` when norm_w is None; None if not want_out."""
    _need_cuda(x, y, y_norm_w, embed, ids, vec, norm_w, y_scale, y_norm_b, norm_b)
    rows, cols = x.shape
    if x.dtype != torch.float32 or not x.is_contiguous():
        raise MvHipError("the residual stream must be a dense fp32 [rows, cols] tensor")
    dt = dtype or next(t.dtype for t in (norm_w, vec, embed, y_norm_w, y) if t is not None)
    splits = 0
    if y is not None:
        if y.dim() == 3:
            splits = y.shape[0]
            if y.dtype != torch.float32 or tuple(y.shape[1:]) != (rows, cols) or not y.is_contiguous():
                raise MvHipError("partial sums must be dense fp32 [splits, rows, cols]")
        elif tuple(y.shape) != (rows, cols) or y.dtype != dt or y.stride(1) != 1:
            raise MvHipError(f"y must be [{rows}, {cols}] of {dt}")
    for name, w in (("y_norm_w", y_norm_w), ("y_scale", y_scale), ("vec", vec), ("norm_w", norm_w), ("y_norm_b", y_norm_b),
                    ("norm_b", norm_b)):
        if w is not None and (w.dtype != dt or w.numel() != cols or not w.is_contiguous()):
            raise MvHipError(f"{name} must be [{cols}] of {dt}")
    if embed is not None and (embed.dtype != dt or embed.shape[1] != cols or not embed.is_contiguous()
                              or ids is None or ids.dtype != torch.int64 or ids.numel() != rows or not ids.is_contiguous()):
        raise MvHipError("embedding table [vocab, cols] of the activation dtype and int64 ids [rows] required")
    if start and embed is None:
        raise MvHipError("a row can only start from an embedding")
    if want_out and out is None:
        out = torch.empty((rows, cols), dtype=dt, device=x.device)
    if out is not None and (tuple(out.shape) != (rows, cols) or out.dtype != dt or out.stride(1) != 1):
        raise MvHipError(f"out must be [{rows}, {cols}] of {dt}")
    a = MvResidualArgs(x.data_ptr(), _ptr(y), _ptr(y_norm_w), _ptr(embed), _ptr(ids) if embed is not None else None,
                       _ptr(vec), _ptr(norm_w), _ptr(out), y.stride(0) if y is not None and splits == 0 else 0,
                       out.stride(0) if out is not None else 0, embed.shape[0] if embed is not None else 0,
                       float(embed_scale), float(norm_offset), float(eps), splits,
                       0 if embed is None else (1 if start else 2), float(y_mult), _ptr(y_scale), _ptr(y_norm_b), _ptr(norm_b))
    a.layer_norm = int(layer_norm)
    if pairs is not None:
        _pair_args(a, pairs, rows, cols, dt)
    if experts is not None:
        rows_out, place, weight = experts
        if (rows_out.dtype != dt or rows_out.shape[1] != cols or not rows_out.is_contiguous() or place.dtype != torch.int32
                or weight.dtype != torch.float32 or place.numel() != weight.numel() or place.numel() % rows
                or not place.is_contiguous() or not weight.is_contiguous()):
            raise MvHipError(f"expert outputs: dense rows of {cols} {dt}, an int32 place and an fp32 weight per choice required")
        a.moe_out, a.moe_rows, a.moe_w, a.moe_top = rows_out.data_ptr(), place.data_ptr(), weight.data_ptr(), place.numel() // rows
    _check(_lib.mv_residual_update(ctypes.byref(a), rows, cols, cols if cols_true is None else int(cols_true), _DTYPES[dt],
                                   _stream()), "mv_residual_update")
    return out


class PairTable(NamedTuple):
    """A table row per (previous token, token): (previous * mul_prev + token * mul_cur) mod (rows - 1), the last row for a
    sequence's first token.  ``prev_tokens`` int32 [2, slots] keeps the token before a step's first at ``state_slots``."""
    table: torch.Tensor
    mul_prev: int
    mul_cur: int
    positions: torch.Tensor
    prev_tokens: torch.Tensor
    state_slots: torch.Tensor
    cu_q: torch.Tensor | None = None     # None: one row per sequence


def _pair_args(a, t: PairTable, rows: int, cols: int, dt) -> None:
    n = rows if t.cu_q is None else t.cu_q.numel() - 1
    slots = t.prev_tokens.shape[1] if t.prev_tokens.numel() else 0
    _need_cuda(*t[:1], *t[3:])
    if (t.table.dtype != dt or t.table.dim() != 2 or t.table.shape[1] != cols or t.table.shape[0] < 2 or not t.table.is_contiguous()
            or t.positions.dtype != torch.int64 or t.positions.numel() != rows or not t.positions.is_contiguous()
            or t.state_slots.dtype != torch.int32 or t.state_slots.numel() != n or not t.state_slots.is_contiguous()
            or (slots and (t.prev_tokens.dtype != torch.int32 or t.prev_tokens.shape[0] != 2 or not t.prev_tokens.is_contiguous()))
            or (t.cu_q is not None and t.cu_q.dtype != torch.int32)):
        raise MvHipError(f"pair table [buckets + 1, {cols}] of {dt}, int64 positions, int32 state slots and kept tokens required")
    a.pairs, a.buckets, a.mul_prev, a.mul_cur = t.table.data_ptr(), t.table.shape[0] - 1, int(t.mul_prev), int(t.mul_cur)
    a.positions, a.state_slots, a.slots, a.n_seqs = t.positions.data_ptr(), t.state_slots.data_ptr(), slots, n
    a.prev_tokens, a.cu_q = t.prev_tokens.data_ptr() if slots else None, _ptr(t.cu_q)


def gated_lookup(s, table, offset: int, dim: int, ids, out=None):
    """gelu_tanh(s[:, j]) * table[ids, offset + j] for j < dim, zeros for the padding columns behind."""
    _need_cuda(s, table, ids)
    rows, cols = s.shape
    if s.stride(1) != 1 or table.dtype != s.dtype or not table.is_contiguous() or ids.dtype != torch.int64 \
            or ids.numel() != rows or not ids.is_contiguous():
        raise MvHipError("gated_lookup: rows of s, a dense table of the same dtype and int64 ids [rows] required")
    if out is None:
        out = torch.empty((rows, cols), dtype=s.dtype, device=s.device)
    _check(_lib.mv_gated_lookup(s.data_ptr(), s.stride(0), table.data_ptr(), table.stride(0), table.shape[0], int(offset),
                                ids.data_ptr(), out.data_ptr(), out.stride(0), rows, int(dim), cols, _dt(s), _stream()),
           "mv_gated_lookup")
    return out


GATED_LOOKUP_LINEAR_MAX_K = 512


def gated_lookup_linear(s, table, offset: int, dim: int, ids, w_packed, n: int):
    """gated_lookup(s, ...) @ W^T in one launch, W [n, K] packed by ``pack_weight`` (K = columns of ``s`` <= 512)."""
    _need_cuda(s, table, ids, w_packed)
    rows, k = s.shape
    if s.stride(1) != 1 or table.dtype != s.dtype or not table.is_contiguous() or ids.dtype != torch.int64 \
            or ids.numel() != rows or not ids.is_contiguous():
        raise MvHipError("gated_lookup_linear: rows of s, a dense table of the same dtype and int64 ids [rows] required")
    if not _packed_ok(w_packed, n, k, s.dtype):
        raise MvHipError(f"packed weight does not match [{n}, {k}]")
    out = torch.empty((rows, -(-n // 8) * 8), dtype=s.dtype, device=s.device)[:, :n]
    _check(_lib.mv_gated_lookup_linear(s.data_ptr(), s.stride(0), table.data_ptr(), table.stride(0), table.shape[0], int(offset),
                                       ids.data_ptr(), w_packed.data_ptr(), out.data_ptr(), out.stride(0), rows, int(dim), k,
                                       int(n), _dt(s), _stream()), "mv_gated_lookup_linear")
    return out


# ---------------------------------------------------------------- K10
LINEAR_SMALL_M_MAX = 64


def linear_small_m_ok(x, weight) -> bool:
    """True when mv_linear_small_m takes this shape (else the caller uses the library GEMM)."""
    k = x.shape[-1]
    return (x.is_cuda and x.dtype in (torch.bfloat16, torch.float16) and weight.dtype == x.dtype
            and weight.dim() == 2 and weight.shape[1] == k and k >= 256 and k % 32 == 0
            and 0 < x.numel() // k <= LINEAR_SMALL_M_MAX and weight.shape[0] % 4 == 0
            and weight.is_contiguous() and x.stride(-1) == 1 and x.data_ptr() % 16 == 0
            and (x.dim() != 2 or x.stride(0) % 8 == 0))


def small_m_shape(rpw: int = 0, waves: int = 0, xlds: int = 0, wlds: int = 0) -> int:
    """Launch-shape override of the small-M kernels (tools/bench_linear.py --sweep): xlds / wlds 1 = on, -1 = off."""
    return (rpw & 15) | ((waves & 31) << 4) | (({0: 0, 1: 1, -1: 2}[xlds]) << 9) | (({0: 0, 1: 1, -1: 2}[wlds]) << 11)


def _packed_ok(packed, n_rows: int, k: int, dtype) -> bool:
    return (packed is not None and packed.dtype == dtype and packed.is_contiguous()
            and packed.numel() == -(-n_rows // 16) * 16 * k)


def linear_narrow(x, packed, n: int, bias=None, shape: int = 0):
    """x [..., K] (any number of rows), packed = pack_weight(W [n, K]), n small -> [..., n]: rows in groups of 16."""
    _need_cuda(x, packed)
    x2, k = _rows2d(x)
    if not _packed_ok(packed, n, k, x.dtype) or (bias is not None and (bias.dtype != x.dtype or bias.shape[0] != n)):
        raise ValueError(f"packed weight / bias do not match [{n}, {k}] of {x.dtype}")
    out = torch.empty((x2.shape[0], n), dtype=x.dtype, device=x.device)
    _check(_lib.mv_linear_small_m_packed(x2.data_ptr(), x2.stride(0), packed.data_ptr(), _ptr(bias), out.data_ptr(),
                                         out.stride(0), x2.shape[0], n, k, _dt(x), 1 << 17 | int(shape), _stream()),   # MV_LINEAR_ROW_GROUPS
           "mv_linear_small_m_packed")
    return out.view(*x.shape[:-1], n)


def linear_small_m(x, weight, bias=None, shape: int = 0, packed=None):
    """x [..., K] (<= 64 rows), weight [N, K], bias [N] | None -> [..., N]; fp32 accumulation.  ``packed``: the
    fragment-ordered copy of ``weight`` (pack_weight) — same result, streamed in whole lines."""
    _need_cuda(x, weight)
    x2, k = _rows2d(x)
    n = weight.shape[0]
    if weight.shape[1] != k or not weight.is_contiguous():
        raise ValueError(f"weight {tuple(weight.shape)} does not match x [..., {k}]")
    if bias is not None and (bias.dtype != x.dtype or bias.shape[0] != n):
        raise ValueError("bias dtype/shape mismatch")
    out = torch.empty((x2.shape[0], n), dtype=x.dtype, device=x.device)
    if _packed_ok(packed, n, k, x.dtype):
        _check(_lib.mv_linear_small_m_packed(x2.data_ptr(), x2.stride(0), packed.data_ptr(), _ptr(bias),
                                             out.data_ptr(), out.stride(0), x2.shape[0], n, k, _dt(x), int(shape),
                                             _stream()), "mv_linear_small_m_packed")
    else:
        _check(_lib.mv_linear_small_m(x2.data_ptr(), x2.stride(0), weight.data_ptr(), _ptr(bias), out.data_ptr(),
                                      out.stride(0), x2.shape[0], n, k, _dt(x), int(shape), _stream()),
               "mv_linear_small_m")
    return out.view(*x.shape[:-1], n)


def gate_up_silu_small_m(x, weight, shape: int = 0, packed=None, act: str = "silu", out=None):
    """x [..., K] (<= 64 rows), weight [2I, K] = [gate rows ; up rows] -> act(x Wg^T) * (x Wu^T), [..., I].  ``out`` ([rows, I],
    rows may be strided): where it goes."""
    _need_cuda(x, weight)
    x2, k = _rows2d(x)
    if weight.shape[0] % 2 or weight.shape[1] != k or not weight.is_contiguous():
        raise ValueError(f"weight {tuple(weight.shape)} is not a merged [2I, {k}] gate_up matrix")
    n = weight.shape[0] // 2
    given, out = out, _gated_out(out, x2.shape[0], n, x)
    if isinstance(act, GateAct):
        use = n % 16 == 0 and _packed_ok(packed, 2 * n, k, x.dtype)
        _check(_lib.mv_gated_act_small_m(x2.data_ptr(), x2.stride(0), (packed if use else weight).data_ptr(), int(use),
                                         out.data_ptr(), out.stride(0), x2.shape[0], n, k, ctypes.byref(act), _dt(x), int(shape),
                                         _stream()), "mv_gated_act_small_m")
        return out if given is not None else out.view(*x.shape[:-1], n)
    shape = int(shape) | GATE_ACTS[act]
    if n % 16 == 0 and _packed_ok(packed, 2 * n, k, x.dtype):
        _check(_lib.mv_gate_up_silu_small_m_packed(x2.data_ptr(), x2.stride(0), packed.data_ptr(), out.data_ptr(),
                                                   out.stride(0), x2.shape[0], n, k, _dt(x), int(shape), _stream()),
               "mv_gate_up_silu_small_m_packed")
    else:
        _check(_lib.mv_gate_up_silu_small_m(x2.data_ptr(), x2.stride(0), weight.data_ptr(), out.data_ptr(),
                                            out.stride(0), x2.shape[0], n, k, _dt(x), int(shape), _stream()),
               "mv_gate_up_silu_small_m")
    return out if given is not None else out.view(*x.shape[:-1], n)


# rows x vectors-per-norm-thread up to which the layer norm rides in the prologue of the small-M projection behind it.  The
# kernel takes up to 8 (csrc/linear_small_m.hip: kNormRows, in passes of 4 / PT rows, round 4), but beyond one pass the
# prologue costs more than the norm launch it saves — Qwen3-1.7B, ctx 1024: B = 5 1.52 -> 1.61 ms per step, B = 8 1.66 ->
# 1.81 — so the default stays at one pass (4); MV_NORM_FOLD_MAX_ROWS=8 selects the longer fold
NORM_FUSED_MAX_ROWS = min(8, int(os.environ.get("MV_NORM_FOLD_MAX_ROWS", "4")))


def norm_linear_small_m_ok(x, n_rows_w: int, packed) -> bool:
    """True when the norm-in-the-prologue form of the small-M projection takes ``x`` [rows, K] (rows x vectors per
    norm thread <= 4, the packed weight present)."""
    if not (x.is_cuda and x.dim() == 2 and x.dtype in (torch.bfloat16, torch.float16) and x.stride(1) == 1):
        return False
    rows, k = x.shape
    if not 0 < rows <= NORM_FUSED_MAX_ROWS or k % 64 or k > 8192 or x.data_ptr() % 16 or x.stride(0) % 8:
        return False
    nvec = k // 8
    threads = min(256, -(-nvec // 64) * 64)
    per_thread = -(-nvec // threads)
    pt = 1 if per_thread <= 1 else (2 if per_thread == 2 else 4)
    return rows * pt <= NORM_FUSED_MAX_ROWS and _packed_ok(packed, n_rows_w, k, x.dtype)


def norm_linear_small_m(x, residual, norm_weight, eps: float, weight_packed, n: int, bias=None, gated: bool = False):
    """(RMSNorm -> projection) of a <= 4-row decode step in ONE launch.  x [rows, K]; residual [rows, K] | None.
    Returns (out [rows, n], new_residual) — new_residual is ``x`` itself when residual is None (reference:
    layernorm.py:81-105, the caller keeps x as the residual), else a fresh tensor holding x + residual.
    gated: weight_packed is the packed merged [2n, K] gate_up matrix, out = silu(gate) * up.
    Returns None when the kernel declines the shape (the caller then runs norm and projection separately)."""
    _need_cuda(x, norm_weight, weight_packed)
    rows, k = x.shape
    out = torch.empty((rows, n), dtype=x.dtype, device=x.device)
    nw = norm_weight if norm_weight.dtype == x.dtype else norm_weight.to(x.dtype)
    if residual is not None:
        r2 = residual if residual.is_contiguous() else residual.contiguous()
        r2 = r2.view(rows, k)
        res_out = torch.empty_like(r2)
        rp, rs, rop, ros = r2.data_ptr(), r2.stride(0), res_out.data_ptr(), res_out.stride(0)
    else:
        res_out, rp, rs, rop, ros = x, None, 0, None, 0
    if gated:
        rc = _lib.mv_norm_gate_up_silu_small_m_packed(x.data_ptr(), x.stride(0), rp, rs, rop, ros, nw.data_ptr(),
                                                      float(eps), weight_packed.data_ptr(), out.data_ptr(),
                                                      out.stride(0), rows, n, k, _dt(x), 0, _stream())
    else:
        rc = _lib.mv_norm_linear_small_m_packed(x.data_ptr(), x.stride(0), rp, rs, rop, ros, nw.data_ptr(),
                                                float(eps), weight_packed.data_ptr(), _ptr(bias), out.data_ptr(),
                                                out.stride(0), rows, n, k, _dt(x), 0, _stream())
    if rc == MV_E_SHAPE:
        return None
    _check(rc, "mv_norm_linear_small_m_packed")
    return out, res_out


# ---------------------------------------------------------------- K11
def pack_weight(weight):
    """[N, K] row-major -> the fragment-ordered copy mv_linear_mid_m streams ([ceil(N/16), K/32, 64, 8])."""
    _need_cuda(weight)
    n, k = weight.shape
    if not weight.is_contiguous():
        weight = weight.contiguous()
    out = torch.empty((int(_lib.mv_packed_weight_elems(n, k)),), dtype=weight.dtype, device=weight.device)
    _check(_lib.mv_pack_weight(weight.data_ptr(), out.data_ptr(), n, k, _dt(weight), _stream()), "mv_pack_weight")
    return out.view((n + 15) // 16, k // 32, 64, 8)


def linear_mid_m_ok(x, n: int) -> bool:
    """True when mv_linear_mid_m takes this shape (else the caller uses the library GEMM)."""
    k = x.shape[-1]
    return (x.is_cuda and x.dtype in (torch.bfloat16, torch.float16) and k % 64 == 0 and k >= 64
            and x.numel() // k > 0 and n % 4 == 0 and x.stride(-1) == 1 and x.data_ptr() % 16 == 0
            and (x.dim() != 2 or x.stride(0) % 8 == 0))


def linear_mid_m(x, w_packed, n: int, bias=None, cfg: int = 0, out=None):
    """x [..., K], w_packed = pack_weight(W [n, K]), bias [n] | None -> [..., n]; fp32 accumulation."""
    _need_cuda(x, w_packed)
    x2, k = _rows2d(x)
    if w_packed.numel() != ((n + 15) // 16) * 16 * k or w_packed.dtype != x.dtype:
        raise ValueError(f"packed weight of {w_packed.numel()} elements does not match [{n}, {k}]")
    if bias is not None and (bias.dtype != x.dtype or bias.shape[0] != n):
        raise ValueError("bias dtype/shape mismatch")
    if out is None:
        out = torch.empty((x2.shape[0], n), dtype=x.dtype, device=x.device)
    _check(_lib.mv_linear_mid_m(x2.data_ptr(), x2.stride(0), w_packed.data_ptr(), _ptr(bias), out.data_ptr(),
                                out.stride(0), x2.shape[0], n, k, _dt(x), int(cfg), _stream()), "mv_linear_mid_m")
    return out.view(*x.shape[:-1], n)


def gate_up_silu_mid_m(x, w_packed, n_inter: int, cfg: int = 0, act: str = "silu", out=None):
    """x [..., K], w_packed = pack_weight([gate rows ; up rows] of shape [2I, K]) -> act(x Wg^T) * (x Wu^T)."""
    _need_cuda(x, w_packed)
    x2, k = _rows2d(x)
    if w_packed.numel() != 2 * n_inter * k or n_inter % 16:
        raise ValueError(f"packed weight of {w_packed.numel()} elements is not a merged [2*{n_inter}, {k}] matrix")
    given, out = out, _gated_out(out, x2.shape[0], n_inter, x)
    if isinstance(act, GateAct):
        _check(_lib.mv_gated_act_mid_m(x2.data_ptr(), x2.stride(0), w_packed.data_ptr(), out.data_ptr(), out.stride(0),
                                       x2.shape[0], n_inter, k, ctypes.byref(act), _dt(x), int(cfg), _stream()),
               "mv_gated_act_mid_m")
        return out if given is not None else out.view(*x.shape[:-1], n_inter)
    _check(_lib.mv_gate_up_silu_mid_m(x2.data_ptr(), x2.stride(0), w_packed.data_ptr(), out.data_ptr(),
                                      out.stride(0), x2.shape[0], n_inter, k, _dt(x), int(cfg) | GATE_ACTS[act], _stream()),
           "mv_gate_up_silu_mid_m")
    return out if given is not None else out.view(*x.shape[:-1], n_inter)


def linear_mid_m_partial(x, w_packed, n: int, splits: int, cfg: int = 0):
    """fp32 partial sums [splits, M, n] of x @ W^T over `splits` K slices."""
    _need_cuda(x, w_packed)
    x2, k = _rows2d(x)
    out = torch.empty((splits, x2.shape[0], n), dtype=torch.float32, device=x.device)
    _check(_lib.mv_linear_mid_m_partial(x2.data_ptr(), x2.stride(0), w_packed.data_ptr(), out.data_ptr(),
                                        x2.shape[0], n, k, int(splits), _dt(x), int(cfg), _stream()),
           "mv_linear_mid_m_partial")
    return out


# ---------------------------------------------------------------- K12: persistent small-batch decode
class MvPersistArgs(ctypes.Structure):
    """include/mvhip.h: MvPersistArgs (host struct, read at call time)."""
    _fields_ = [("m", c_int), ("hidden", c_int), ("n_heads", c_int), ("n_kv_heads", c_int), ("head_dim", c_int),
                ("inter", c_int), ("eps", c_float), ("scale", c_float), ("x_in", c_void_p), ("res_in", c_void_p),
                ("x_in_stride", c_int64), ("res_in_stride", c_int64), ("positions", c_void_p),
                ("slot_mapping", c_void_p), ("block_tables", c_void_p), ("context_lens", c_void_p),
                ("table_stride", c_int64), ("num_blocks", c_int64), ("max_pos", c_int64), ("block_size", c_int),
                ("max_blocks", c_int), ("cos", c_void_p), ("sin", c_void_p), ("out_h_offset", c_int64),
                ("out_res_offset", c_int64)]


PERSIST_LAYER_FIELDS = ("ln1_w", "wqkv", "bqkv", "q_norm_w", "k_norm_w", "wo", "ln2_w", "wgu", "wdown", "k_cache", "v_cache")
PERSIST_MAX_ROWS = 16


def persist_layer_table(rows, device) -> torch.Tensor:
    """Device array of MvPersistLayer: ``rows`` = per layer a dict field -> tensor | None (PERSIST_LAYER_FIELDS)."""
    flat = [[0 if r[f] is None else r[f].data_ptr() for f in PERSIST_LAYER_FIELDS] for r in rows]
    return torch.tensor(flat, dtype=torch.int64).to(device)


def decode_layers_persistent_workspace(m, hidden, n_heads, n_kv_heads, head_dim, inter, block_size, max_blocks, device):
    n = int(_lib.mv_decode_layers_persistent_workspace_bytes(m, hidden, n_heads, n_kv_heads, head_dim, inter, block_size,
                                                             max_blocks))
    return torch.zeros(n, dtype=torch.uint8, device=device)


def decode_layers_persistent(table, n_layers, x, positions, slot_mapping, block_tables, context_lens, cos, sin, k_cache0,
                             n_heads, n_kv_heads, head_dim, inter, eps, scale, workspace, status, flags: int = 0):
    """Every decoder layer of a decode step of <= 16 rows in ONE launch (csrc/decode_persistent.hip).  ``x`` [M, hidden] =
    the embedding output.  -> (h, residual): views of ``workspace`` holding the last layer's down_proj output and the
    residual (the caller applies the final norm), or None when the kernel does not take the shape (MV_E_SHAPE)."""
    _need_cuda(x, positions, slot_mapping, block_tables, context_lens, cos, sin, workspace, status)
    m, hidden = x.shape
    bt = _i32(block_tables)
    if bt.dim() != 2 or bt.stride(1) != 1 or x.stride(1) != 1 or positions.dtype != torch.int64:
        return None
    a = MvPersistArgs()
    a.m, a.hidden, a.n_heads, a.n_kv_heads, a.head_dim, a.inter = m, hidden, n_heads, n_kv_heads, head_dim, inter
    a.eps, a.scale = float(eps), float(scale)
    a.x_in, a.res_in, a.x_in_stride, a.res_in_stride = x.data_ptr(), None, x.stride(0), 0
    a.positions, a.slot_mapping = positions.data_ptr(), _i32(slot_mapping).data_ptr()
    a.block_tables, a.context_lens = bt.data_ptr(), _i32(context_lens).data_ptr()
    a.table_stride, a.num_blocks, a.max_pos = bt.stride(0), k_cache0.shape[0], cos.shape[0]
    a.block_size, a.max_blocks = k_cache0.shape[1], bt.shape[1]
    a.cos, a.sin = cos.data_ptr(), sin.data_ptr()
    rc = _lib.mv_decode_layers_persistent(table.data_ptr(), n_layers, ctypes.byref(a), workspace.data_ptr(),
                                          workspace.numel(), status.data_ptr(), _dt(x), int(flags), _stream())
    if rc == MV_E_SHAPE:
        return None
    _check(rc, "mv_decode_layers_persistent")
    esz = x.element_size()
    h = workspace[a.out_h_offset:a.out_h_offset + m * hidden * esz].view(x.dtype).view(m, hidden)
    r = workspace[a.out_res_offset:a.out_res_offset + m * hidden * esz].view(x.dtype).view(m, hidden)
    return h, r


# ---------------------------------------------------------------- f2
def greedy_pack(logits_local, local_tokens, rank: int, world: int, rows_padded: int):
    """-> buf [world, rows_padded, 4] in the logits' dtype (see mv_greedy_pack)."""
    _need_cuda(logits_local, local_tokens)
    rows, vpr = logits_local.shape
    buf = torch.empty((world, rows_padded, 4), dtype=logits_local.dtype, device=logits_local.device)
    _check(_lib.mv_greedy_pack(logits_local.data_ptr(), logits_local.stride(0), local_tokens.data_ptr(), rank, world,
                               vpr, rows, rows_padded, buf.data_ptr(), _dt(logits_local), _stream()),
           "mv_greedy_pack")
    return buf


def greedy_merge(buf, rows: int):
    world, rows_padded, _ = buf.shape
    out = torch.empty((rows,), dtype=torch.int64, device=buf.device)
    _check(_lib.mv_greedy_merge(buf.data_ptr(), world, rows, rows_padded, out.data_ptr(), _dt(buf), _stream()),
           "mv_greedy_merge")
    return out


TOPC = 64   # == mv_topc_width(): candidates a rank contributes per row


def topc_pack(logits_local, rank: int, world: int, rows_padded: int):
    """-> buf [world, rows_padded, 64, 4] in the logits' dtype (see mv_topc_pack)."""
    _need_cuda(logits_local)
    rows, vpr = logits_local.shape
    buf = torch.empty((world, rows_padded, TOPC, 4), dtype=logits_local.dtype, device=logits_local.device)
    _check(_lib.mv_topc_pack(logits_local.data_ptr(), logits_local.stride(0), vpr, rank, world, vpr, rows, rows_padded,
                             buf.data_ptr(), _dt(logits_local), _stream()), "mv_topc_pack")
    return buf


def topc_unpack(buf, rows: int):
    """-> (cand_logits [rows, world*64] in buf's dtype, cand_idx int32 [rows, world*64] global token ids)."""
    world, rows_padded = buf.shape[0], buf.shape[1]
    cl = torch.empty((rows, world * TOPC), dtype=buf.dtype, device=buf.device)
    ci = torch.empty((rows, world * TOPC), dtype=torch.int32, device=buf.device)
    _check(_lib.mv_topc_unpack(buf.data_ptr(), world, rows, rows_padded, cl.data_ptr(), ci.data_ptr(), _dt(buf), _stream()),
           "mv_topc_unpack")
    return cl, ci


def mass_pack(stats, local_tokens, rank: int, world: int, vocab_per_rank: int, rows_padded: int, dtype):
    """-> buf [world, rows_padded, 8] in the logits' 16-bit dtype (see mv_mass_pack)."""
    _need_cuda(stats, local_tokens)
    rows = local_tokens.shape[0]
    assert stats.dtype == torch.float32 and stats.shape == (rows, 2) and stats.is_contiguous()
    assert local_tokens.dtype == torch.int64 and dtype in (torch.bfloat16, torch.float16)
    buf = torch.empty((world, rows_padded, 8), dtype=dtype, device=stats.device)
    _check(_lib.mv_mass_pack(stats.data_ptr(), local_tokens.data_ptr(), rank, world, vocab_per_rank, rows, rows_padded,
                             buf.data_ptr(), _DTYPES[dtype], _stream()), "mv_mass_pack")
    return buf


def mass_merge(buf, rows: int, temperatures, seed: int = 0, offset: int = 0, offset_dev=None):
    """Summed ``mass_pack`` buffers -> int64 tokens [rows] (see mv_mass_merge; seed / offset as given to ``sample``)."""
    _need_cuda(buf, temperatures)
    world, rows_padded, _ = buf.shape
    assert temperatures is None or (temperatures.dtype == torch.float32 and temperatures.is_contiguous())
    out = torch.empty((rows,), dtype=torch.int64, device=buf.device)
    _check(_lib.mv_mass_merge(buf.data_ptr(), _ptr(temperatures), int(seed) & (2**64 - 1), int(offset) & (2**64 - 1),
                              _ptr(offset_dev), world, rows, rows_padded, out.data_ptr(), _dt(buf), _stream()),
           "mv_mass_merge")
    return out


def shard_key_hist(logits_local, row_max, temperatures, prefix=None):
    """-> int64 [rows, 256]: this shard's fixed-point mass per key bin below the row's global maximum (mv_shard_key_hist)."""
    _need_cuda(logits_local, row_max, temperatures, prefix)
    rows, vl = logits_local.shape
    assert logits_local.stride(1) == 1 and row_max.dtype == torch.float32 and row_max.is_contiguous()
    assert temperatures is None or (temperatures.dtype == torch.float32 and temperatures.is_contiguous())
    assert prefix is None or (prefix.dtype == torch.int32 and prefix.is_contiguous())
    hist = torch.empty((rows, 256), dtype=torch.int64, device=logits_local.device)
    _check(_lib.mv_shard_key_hist(logits_local.data_ptr(), logits_local.stride(0), vl, rows, row_max.data_ptr(),
                                  _ptr(temperatures), _ptr(prefix), hist.data_ptr(), _dt(logits_local), _stream()),
           "mv_shard_key_hist")
    return hist


def nucleus_pick(hist, level: int, top_ps, min_ps, temperatures, row_max, dtype, state=None, prefix=None):
    """Level 0 -> (state int64 [rows, 2], prefix int32 [rows]); level 1 (with those) -> floor fp32 [rows]
    (mv_nucleus_pick; ``hist`` = the all-reduced ``shard_key_hist`` of that level)."""
    _need_cuda(hist, top_ps, min_ps, temperatures, row_max)
    rows = hist.shape[0]
    assert hist.dtype == torch.int64 and hist.shape == (rows, 256) and hist.is_contiguous()
    for x in (top_ps, min_ps, temperatures, row_max):
        assert x is None or (x.dtype == torch.float32 and x.is_contiguous())
    dev = hist.device
    if level == 0:
        state = torch.empty((rows, 2), dtype=torch.int64, device=dev)
        prefix = torch.empty((rows,), dtype=torch.int32, device=dev)
    floor = torch.empty((rows,), dtype=torch.float32, device=dev) if level == 1 else None
    _check(_lib.mv_nucleus_pick(hist.data_ptr(), level, _ptr(top_ps), _ptr(min_ps), _ptr(temperatures), _ptr(row_max),
                                state.data_ptr(), prefix.data_ptr(), _ptr(floor), rows, _DTYPES[dtype], _stream()),
           "mv_nucleus_pick")
    return (state, prefix) if level == 0 else floor


def mask_below(logits, floor):
    """-> copy of ``logits`` [rows, V] with everything below the row's ``floor`` (fp32 [rows]) at -inf (mv_mask_below)."""
    _need_cuda(logits, floor)
    rows, vl = logits.shape
    assert logits.stride(1) == 1 and floor.dtype == torch.float32 and floor.is_contiguous()
    out = torch.empty((rows, vl), dtype=logits.dtype, device=logits.device)
    _check(_lib.mv_mask_below(logits.data_ptr(), logits.stride(0), vl, rows, floor.data_ptr(), out.data_ptr(),
                              out.stride(0), _dt(logits), _stream()), "mv_mask_below")
    return out


def topc_pick(cand_logits, cand_idx, pos, temperatures=None):
    """Candidate positions -> int64 token ids; temperature-0 rows take the lowest global index among the row maxima
    (see mv_topc_pick)."""
    _need_cuda(cand_logits, cand_idx, pos)
    rows, width = cand_logits.shape
    assert cand_idx.dtype == torch.int32 and pos.dtype == torch.int64 and cand_idx.shape == cand_logits.shape
    assert cand_logits.is_contiguous() and cand_idx.is_contiguous()
    if temperatures is not None:
        assert temperatures.dtype == torch.float32 and temperatures.shape[0] >= rows and temperatures.is_contiguous()
    out = torch.empty((rows,), dtype=torch.int64, device=cand_logits.device)
    _check(_lib.mv_topc_pick(cand_logits.data_ptr(), cand_idx.data_ptr(), pos.data_ptr(), _ptr(temperatures),
                             out.data_ptr(), rows, width, _dt(cand_logits), _stream()), "mv_topc_pick")
    return out


# ---------------------------------------------------------------- a2 (device side)
def decode_advance(input_ids, tokens, positions, slot_mapping, context_lens, rng_offset) -> None:
    """In place: ids <- tokens, positions/context/slots += 1 (padding rows untouched), rng += 1."""
    _need_cuda(input_ids, tokens, positions, slot_mapping, context_lens, rng_offset)
    assert input_ids.dtype == tokens.dtype == positions.dtype == torch.int64
    assert slot_mapping.dtype == context_lens.dtype == torch.int32
    _check(_lib.mv_decode_advance(input_ids.data_ptr(), tokens.data_ptr(), positions.data_ptr(),
                                  slot_mapping.data_ptr(), context_lens.data_ptr(), _ptr(rng_offset),
                                  input_ids.shape[0], _stream()), "mv_decode_advance")


# ---------------------------------------------------------------- K14
MV_LATENT_SIMPLE = 1


def _rows_ok(what: str, t, cols: int, dtype=None) -> None:
    if t.dim() != 2 or t.stride(1) != 1 or t.shape[1] < cols or (dtype is not None and t.dtype != dtype):
        raise MvHipError(f"{what}: rows of at least {cols} elements of {dtype} required, got {tuple(t.shape)} {t.dtype}")


def _tables_ok(positions, cos, sin, n_tok: int, pairs: int) -> None:
    if positions.dtype != torch.int64 or positions.numel() != n_tok or not positions.is_contiguous():
        raise MvHipError(f"int64 positions of {n_tok} tokens required")
    for t in (cos, sin):
        if t.dtype != torch.float32 or t.dim() != 2 or t.shape[1] != pairs or not t.is_contiguous():
            raise MvHipError(f"cos / sin must be dense fp32 [max_pos, {pairs}]")


def latent_prep(z, q_norm_w, q_off: int, q_rank: int, eps: float, kv=None, positions=None, cos=None, sin=None, plane=None,
                slot_mapping=None, want_rows: bool = False):
    """Merged down projection ``z`` -> (normed query latent [T, q_cols], cached rows [T, kv_cols + rot_cols] or None).  ``kv``:
    None (the layer has no latent of its own), or (norm weight, kv_off, kv_rank, rot_off, rot_dim, rot_cols); the rows also go to
    ``plane`` [..., kv_cols + rot_cols] at ``slot_mapping``."""
    _need_cuda(z, q_norm_w, plane, slot_mapping)
    t, q_cols = z.shape[0], q_norm_w.numel()
    _rows_ok("z", z, q_off + q_cols)
    out = torch.empty((t, q_cols), dtype=z.dtype, device=z.device)
    a = MvLatentPrepArgs(z=z.data_ptr(), z_stride=z.stride(0), q_norm_w=q_norm_w.data_ptr(), q_out=out.data_ptr(),
                         q_out_stride=q_cols, q_off=q_off, q_rank=q_rank, q_cols=q_cols, eps=eps)
    rows = None
    if kv is not None:
        w, kv_off, kv_rank, rot_off, rot_dim, rot_cols = kv
        _rows_ok("z", z, max(kv_off + w.numel(), rot_off + rot_cols))
        _tables_ok(positions, cos, sin, t, rot_dim // 2)
        cols = w.numel() + rot_cols
        if want_rows:
            rows = torch.empty((t, cols), dtype=z.dtype, device=z.device)
        a.kv_norm_w, a.kv_off, a.kv_rank, a.kv_cols = w.data_ptr(), kv_off, kv_rank, w.numel()
        a.rot_off, a.rot_dim, a.rot_cols = rot_off, rot_dim, rot_cols
        a.positions, a.cos, a.sin, a.max_pos = positions.data_ptr(), cos.data_ptr(), sin.data_ptr(), cos.shape[0]
        a.rows_out = _ptr(rows)
        if plane is not None and slot_mapping is not None and plane.numel():
            if plane.dtype != z.dtype or plane.shape[-1] != cols or not plane.is_contiguous() or slot_mapping.numel() != t:
                raise MvHipError(f"latent plane: dense rows of {cols} {z.dtype} and a slot per token required")
            slots = _i32(slot_mapping)
            a.plane, a.slot_mapping, a.num_slots = plane.data_ptr(), slots.data_ptr(), plane.numel() // cols
    _check(_lib.mv_latent_prep(ctypes.byref(a), t, _dt(z), _stream()), "mv_latent_prep")
    return out, rows


def head_linear(x, w, out, rot=None):
    """out[t, h, :n] = w[h] x[t, h, :k] for x [T, H, >= k], w [H, n, k], out [T, H, >= n]; ``rot`` (rot_dim, rot_cols, positions,
    cos, sin): also out[t, h, n : n + rot_cols] = the rotated x[t, h, k : k + rot_dim]."""
    _need_cuda(x, w, out)
    t, h, n, k = x.shape[0], *w.shape
    rot_cols = rot[1] if rot else 0
    if (not w.is_contiguous() or w.dtype != x.dtype or out.dtype != x.dtype or x.shape[1] != h or tuple(out.shape[:2]) != (t, h)
            or x.shape[2] < k + rot_cols or out.shape[2] < n + rot_cols or x.stride(2) != 1 or out.stride(2) != 1):
        raise MvHipError(f"head_linear: {tuple(x.shape)} x {tuple(w.shape)} -> {tuple(out.shape)} does not fit")
    a = MvHeadLinearArgs(x=x.data_ptr(), w=w.data_ptr(), out=out.data_ptr(), x_tok=x.stride(0), x_head=x.stride(1),
                         out_tok=out.stride(0), out_head=out.stride(1), heads=h, n=n, k=k)
    if rot:
        rot_dim, _, positions, cos, sin = rot
        _tables_ok(positions, cos, sin, t, rot_dim // 2)
        a.positions, a.cos, a.sin, a.max_pos = positions.data_ptr(), cos.data_ptr(), sin.data_ptr(), cos.shape[0]
        a.rot_dim, a.rot_cols = rot_dim, rot_cols
    _check(_lib.mv_head_linear(ctypes.byref(a), t, _dt(x), _stream()), "mv_head_linear")
    return out


def latent_gather(plane, block_tables, cu, start, total: int, max_len: int):
    """Rows of ``plane`` [blocks, block_size, cols]: positions start[s] .. of sequence s at cu[s] .. cu[s + 1] of [total, cols]."""
    _need_cuda(plane, block_tables, cu, start)
    cols = plane.shape[2]
    out = torch.empty((total, cols), dtype=plane.dtype, device=plane.device)
    bt = _i32(block_tables)
    if bt.stride(1) != 1 or bt.shape[0] != start.numel() or cu.numel() != start.numel() + 1:
        raise MvHipError("block tables [sequences, blocks], one start per sequence and cumulative lengths required")
    _check(_lib.mv_latent_gather(plane.data_ptr(), plane.shape[0], plane.shape[1], cols, bt.data_ptr(), bt.stride(0), bt.shape[1],
                                 cu.data_ptr(), start.data_ptr(), bt.shape[0], int(max_len), out.data_ptr(), _dt(plane),
                                 _stream()), "mv_latent_gather")
    return out


def latent_decode_workspace_bytes(batch, heads, kv_cols, rot_cols, block_size, max_blocks, window, dtype) -> int:
    return int(_lib.mv_latent_decode_workspace_bytes(int(batch), int(heads), int(kv_cols), int(rot_cols), int(block_size),
                                                     int(max_blocks), int(window), _DTYPES[dtype]))


def latent_decode(q, plane, block_tables, context_lens, kv_cols: int, scale: float, window: int = 0, flags: int = 0):
    """q [B, H, kv_cols + rot_cols] (latent coordinates | rotated part) against the cached rows -> latents [B, H, kv_cols]."""
    _need_cuda(q, plane, block_tables, context_lens)
    b, h, cols = q.shape
    if not q.is_contiguous() or plane.dtype != q.dtype or plane.shape[-1] != cols or not plane.is_contiguous():
        raise MvHipError(f"latent_decode: dense q [B, H, {cols}] and a plane of such rows required")
    bt, cl = _i32(block_tables), _i32(context_lens)
    if bt.shape[1] and bt.stride(1) != 1 or bt.shape[0] != b or cl.numel() != b:
        raise MvHipError("latent_decode: one block table and one length per row required")
    out = torch.empty((b, h, kv_cols), dtype=q.dtype, device=q.device)
    nb, bs, rot_cols = plane.shape[0], plane.shape[1], cols - kv_cols
    ws = workspace(latent_decode_workspace_bytes(b, h, kv_cols, rot_cols, bs, bt.shape[1], window, q.dtype), q.device)
    _check(_lib.mv_latent_decode(q.data_ptr(), plane.data_ptr(), bt.data_ptr(), bt.stride(0) if bt.shape[1] else 0, cl.data_ptr(),
                                 out.data_ptr(), b, h, kv_cols, rot_cols, bs, bt.shape[1], nb, int(window), float(scale),
                                 ws.data_ptr(), ws.numel(), _dt(q), int(flags), _stream()), "mv_latent_decode")
    return out


def latent_prefill(q, k, v, rot, cu_q, cu_k, max_q: int, max_k: int, positions, cos, sin, rot_dim: int, scale: float,
                   window: int = 0, out=None, flags: int = 0):
    """q [T, H, dq] ([plain | rotated part, not yet rotated]), k [G, H, plain], v [G, H, dv], rot [G, rot_cols] -> [T, H, dv]."""
    _need_cuda(q, k, v, rot, cu_q, cu_k, positions)
    t, h, dq = q.shape
    dp, dv = k.shape[2], v.shape[2]
    for x, d in ((q, dq), (k, dp), (v, dv)):
        if x.shape[1] != h or x.stride(2) != 1 or x.stride(1) != d or x.dtype != q.dtype:
            raise MvHipError("latent_prefill: heads must lie side by side in the rows of q, k and v")
    _rows_ok("rot", rot, 1, q.dtype)
    _tables_ok(positions, cos, sin, t, rot_dim // 2)
    if out is None:
        out = torch.empty((t, h, dv), dtype=q.dtype, device=q.device)
    _out_rows(out, t, h, dv)
    a = MvLatentPrefillArgs(q=q.data_ptr(), k=k.data_ptr(), v=v.data_ptr(), rot=rot.data_ptr(), out=out.data_ptr(),
                            q_stride=q.stride(0), k_stride=k.stride(0), v_stride=v.stride(0), rot_stride=rot.stride(0),
                            out_stride=out.stride(0), cu_q=cu_q.data_ptr(), cu_k=cu_k.data_ptr(), positions=positions.data_ptr(),
                            cos=cos.data_ptr(), sin=sin.data_ptr(), max_pos=cos.shape[0], n_seqs=cu_q.numel() - 1,
                            max_q=int(max_q), max_k=int(max_k), heads=h, plain_cols=dp, rot_dim=rot_dim, rot_cols=rot.shape[1],
                            dq=dq, dv=dv, window=int(window), scale=float(scale))
    _check(_lib.mv_latent_prefill(ctypes.byref(a), _dt(q), int(flags), _stream()), "mv_latent_prefill")
    return out


# ---------------------------------------------------------------- K15
MV_SSM_SCAN = 1


def _ssm_args(shape, x, state_slots, out, conv_w=None, conv_b=None, conv_state=None, ssm_state=None, dt=None, dt_bias=None,
              a_log=None, d=None):
    """``shape``: (heads, groups, p, n, b_off, c_off)."""
    _need_cuda(x, state_slots, conv_state, ssm_state, dt)
    heads, groups, p, n, b_off, c_off = shape
    a = MvSsmArgs(x=x.data_ptr(), x_stride=x.stride(0), state_slots=state_slots.data_ptr(), out=out.data_ptr(),
                  out_stride=out.stride(0), n_seqs=state_slots.numel(), channels=c_off + groups * n, taps=1, heads=heads,
                  groups=groups, p=p, n=n, b_off=b_off, c_off=c_off)
    _rows_ok("x", x, a.channels)
    if state_slots.dtype != torch.int32 or not state_slots.is_contiguous():
        raise MvHipError("int32 state slots required")
    if conv_w is not None:
        if conv_w.dtype != x.dtype or conv_w.shape[1] != a.channels or (
                conv_b is not None and (conv_b.dtype != x.dtype or conv_b.numel() != a.channels)):
            raise MvHipError(f"convolution weight [taps, {a.channels}] (and bias) of {x.dtype} required")
        a.conv_w, a.conv_b, a.taps = conv_w.data_ptr(), _ptr(conv_b), conv_w.shape[0]
    slots = 0
    if conv_state is not None and conv_state.numel():
        slots = conv_state.shape[1]
        if conv_state.dtype != x.dtype or tuple(conv_state.shape) != (2, slots, a.taps - 1, a.channels) or not conv_state.is_contiguous():
            raise MvHipError(f"convolution state must be dense [2, slots, {a.taps - 1}, {a.channels}] of {x.dtype}")
        a.conv_state = conv_state.data_ptr()
    if ssm_state is not None and ssm_state.numel():
        slots = ssm_state.shape[1]
        if ssm_state.dtype != torch.float32 or tuple(ssm_state.shape) != (2, slots, heads, n, p) or not ssm_state.is_contiguous():
            raise MvHipError(f"recurrent state must be dense fp32 [2, slots, {heads}, {n}, {p}]")
        a.ssm_state = ssm_state.data_ptr()
    a.slots = slots
    if dt is not None:
        if dt.dtype != x.dtype or dt.shape[0] != x.shape[0] or dt.stride(1) != 1:
            raise MvHipError("raw step sizes: rows of x's dtype, one per token")
        for w in (dt_bias, a_log, d):
            if w.dtype != x.dtype or w.numel() < heads:
                raise MvHipError(f"per-head parameters of {x.dtype} required")
        a.dt, a.dt_stride = dt.data_ptr(), dt.stride(0)
        a.dt_bias, a.a_log, a.d = dt_bias.data_ptr(), a_log.data_ptr(), d.data_ptr()
    return a


def causal_conv(x, conv_w, conv_b, shape, conv_state, state_slots, cu_q, cu_k, max_q: int):
    """silu(causal convolution) of the projected channels [T, channels] of a batch of sequences; keeps the last inputs."""
    out = torch.empty((x.shape[0], conv_w.shape[1]), dtype=x.dtype, device=x.device)
    a = _ssm_args(shape, x, state_slots, out, conv_w, conv_b, conv_state)
    a.cu_q, a.cu_k, a.max_q = cu_q.data_ptr(), cu_k.data_ptr(), int(max_q)
    _check(_lib.mv_causal_conv(ctypes.byref(a), _dt(x), _stream()), "mv_causal_conv")
    return out


def ssm_prefill(x, dt, dt_bias, a_log, d, shape, ssm_state, state_slots, cu_q, cu_k, max_q: int, out=None, flags: int = 0):
    """The recurrence over convolved channels [T, channels] and raw step sizes [T, heads] -> y [T, heads * p]."""
    if out is None:
        out = torch.empty((x.shape[0], shape[0] * shape[2]), dtype=x.dtype, device=x.device)
    a = _ssm_args(shape, x, state_slots, out, ssm_state=ssm_state, dt=dt, dt_bias=dt_bias, a_log=a_log, d=d)
    a.cu_q, a.cu_k, a.max_q = cu_q.data_ptr(), cu_k.data_ptr(), int(max_q)
    _check(_lib.mv_ssm_prefill(ctypes.byref(a), _dt(x), int(flags), _stream()), "mv_ssm_prefill")
    return out


def ssm_step(x, dt, conv_w, conv_b, dt_bias, a_log, d, shape, conv_state, ssm_state, state_slots, context_lens, out=None):
    """One token per sequence: convolution and recurrence of the projected channels [B, channels] -> y [B, heads * p]."""
    if out is None:
        out = torch.empty((x.shape[0], shape[0] * shape[2]), dtype=x.dtype, device=x.device)
    a = _ssm_args(shape, x, state_slots, out, conv_w, conv_b, conv_state, ssm_state, dt, dt_bias, a_log, d)
    lens = _i32(context_lens)
    if lens.numel() != x.shape[0] or state_slots.numel() != x.shape[0]:
        raise MvHipError("one length and one state slot per row required")
    a.context_lens = lens.data_ptr()
    _check(_lib.mv_ssm_step(ctypes.byref(a), _dt(x), _stream()), "mv_ssm_step")
    return out


def gated_group_norm(y, z, w, heads: int, p: int, p_true: int, groups: int, eps: float, out_cols: int | None = None):
    """rms over each of ``groups`` equal parts of y * silu(z), times w: [T, heads * p] (p_true of each head's columns count);
    ``out_cols``: rows of that many columns, zeros behind."""
    _need_cuda(y, z, w)
    cols = heads * p
    _rows_ok("y", y, cols)
    _rows_ok("z", z, cols, y.dtype)
    if w.dtype != y.dtype or w.numel() != cols or y.shape[0] != z.shape[0]:
        raise MvHipError(f"norm weight of {cols} {y.dtype} and as many rows of z required")
    wide = out_cols is not None and out_cols > cols
    out = (torch.zeros if wide else torch.empty)((y.shape[0], out_cols if wide else cols), dtype=y.dtype, device=y.device)
    _check(_lib.mv_gated_group_norm(y.data_ptr(), y.stride(0), z.data_ptr(), z.stride(0), w.data_ptr(), out.data_ptr(),
                                    out.stride(0), y.shape[0], heads, p, p_true, groups, float(eps), _dt(y), _stream()),
           "mv_gated_group_norm")
    return out


# ---------------------------------------------------------------- K16
MV_DELTA_SCAN = 1
GATES = {"silu": 0, "sigmoid": 1}


class DeltaShape(NamedTuple):
    """Stored sizes of a gated delta rule: channels [v heads * p | k groups * n | q groups * n] at 0, k_off, q_off."""
    heads: int
    groups: int
    p: int          # columns of a head (p_true of them count)
    n: int          # key channels
    k_off: int
    q_off: int
    p_true: int
    q_scale: float
    channel_decay: bool
    eps: float = 1e-6
    unit_eps: float = 1e-6

    @property
    def channels(self) -> int:
        return self.q_off + self.groups * self.n

    @property
    def conv(self) -> tuple:
        """The same channels as ``causal_conv`` takes them."""
        return self.heads, self.groups, self.p, self.n, self.k_off, self.q_off


def _delta_args(s: DeltaShape, x, beta, a, dt_bias, a_log, state, state_slots, out):
    _need_cuda(x, beta, a, dt_bias, a_log, state, state_slots, out)
    _rows_ok("x", x, s.channels)
    _rows_ok("beta", beta, s.heads, x.dtype)
    width = s.heads * (s.n if s.channel_decay else 1)
    _rows_ok("decay", a, width, x.dtype)
    _rows_ok("out", out, s.heads * s.p, x.dtype)
    if dt_bias.dtype != x.dtype or dt_bias.numel() < width or a_log.dtype != x.dtype or a_log.numel() < s.heads:
        raise MvHipError(f"decay parameters of {x.dtype}, {width} and {s.heads}, required")
    if state_slots.dtype != torch.int32 or not state_slots.is_contiguous():
        raise MvHipError("int32 state slots required")
    g = MvDeltaArgs(x=x.data_ptr(), beta=beta.data_ptr(), a=a.data_ptr(), dt_bias=dt_bias.data_ptr(), a_log=a_log.data_ptr(),
                    state_slots=state_slots.data_ptr(), out=out.data_ptr(), x_stride=x.stride(0), beta_stride=beta.stride(0),
                    a_stride=a.stride(0), out_stride=out.stride(0), n_seqs=state_slots.numel(), total_q=x.shape[0],
                    channels=s.channels, taps=1, heads=s.heads, groups=s.groups, p=s.p, p_true=s.p_true, n=s.n, k_off=s.k_off,
                    q_off=s.q_off, channel_decay=int(s.channel_decay), eps=s.eps, unit_eps=s.unit_eps, q_scale=s.q_scale,
                    out_scale=1.0)
    if state is not None and state.numel():
        if state.dtype != torch.float32 or tuple(state.shape[2:]) != (s.heads, s.n, s.p) or state.shape[0] != 2 or not state.is_contiguous():
            raise MvHipError(f"recurrent state must be dense fp32 [2, slots, {s.heads}, {s.n}, {s.p}]")
        g.state, g.slots = state.data_ptr(), state.shape[1]
    return g


def delta_prefill(s: DeltaShape, x, beta, a, dt_bias, a_log, state, state_slots, cu_q, cu_k, max_q: int, out=None, flags: int = 0):
    """The gated delta rule over convolved channels [T, channels], raw beta [T, heads] and raw decays -> o [T, heads * p]."""
    if out is None:
        out = torch.empty((x.shape[0], s.heads * s.p), dtype=x.dtype, device=x.device)
    g = _delta_args(s, x, beta, a, dt_bias, a_log, state, state_slots, out)
    g.cu_q, g.cu_k, g.max_q = cu_q.data_ptr(), cu_k.data_ptr(), int(max_q)
    n = 0 if flags & MV_DELTA_SCAN else int(_lib.mv_delta_prefill_workspace_bytes(g.n_seqs, g.total_q, s.heads, s.p, s.n, _dt(x)))
    ws = torch.empty((n,), dtype=torch.uint8, device=x.device) if n else None
    g.workspace, g.ws_bytes = _ptr(ws), n
    _check(_lib.mv_delta_prefill(ctypes.byref(g), _dt(x), int(flags), _stream()), "mv_delta_prefill")
    return out


def delta_step(s: DeltaShape, x, beta, a, dt_bias, a_log, conv_w, conv_state, state, state_slots, context_lens, gate, norm_w,
               gate_kind: str = "silu", out_scale: float = 1.0, out=None):
    """One token per sequence, from projected channels [B, channels]: convolution, gated delta rule, ``head_norm_gate``."""
    if out is None:
        out = torch.empty((x.shape[0], s.heads * s.p), dtype=x.dtype, device=x.device)
    g = _delta_args(s, x, beta, a, dt_bias, a_log, state, state_slots, out)
    lens = _i32(context_lens)
    _need_cuda(conv_w, gate, norm_w, lens)
    _rows_ok("gate", gate, s.heads * s.p, x.dtype)
    if lens.numel() != x.shape[0] or state_slots.numel() != x.shape[0]:
        raise MvHipError("one length and one state slot per row required")
    if conv_w.dtype != x.dtype or conv_w.shape[1] != s.channels or norm_w.dtype != x.dtype or norm_w.numel() < s.p:
        raise MvHipError(f"convolution weight [taps, {s.channels}] and norm weight [{s.p}] of {x.dtype} required")
    g.taps = conv_w.shape[0]
    if g.slots and g.taps > 1:
        if conv_state.dtype != x.dtype or tuple(conv_state.shape) != (2, g.slots, g.taps - 1, s.channels) or not conv_state.is_contiguous():
            raise MvHipError(f"convolution state must be dense [2, {g.slots}, {g.taps - 1}, {s.channels}] of {x.dtype}")
        g.conv_state = conv_state.data_ptr()
    g.conv_w, g.norm_w, g.gate, g.gate_stride = conv_w.data_ptr(), norm_w.data_ptr(), gate.data_ptr(), gate.stride(0)
    g.context_lens, g.gate_kind, g.out_scale = lens.data_ptr(), GATES[gate_kind], float(out_scale)
    _check(_lib.mv_delta_step(ctypes.byref(g), _dt(x), _stream()), "mv_delta_step")
    return out


def head_norm_gate(y, gate, w, heads: int, p: int, p_true: int, eps: float, gate_kind: str = "silu", out_scale: float = 1.0, out=None):
    """Per head of [T, heads * p]: rms(y) * w (shared by the heads) * act(gate) * out_scale."""
    _need_cuda(y, gate, w)
    _rows_ok("y", y, heads * p)
    _rows_ok("gate", gate, heads * p, y.dtype)
    if out is None:
        out = torch.empty((y.shape[0], heads * p), dtype=y.dtype, device=y.device)
    _rows_ok("out", out, heads * p, y.dtype)
    if w.dtype != y.dtype or w.numel() < p or gate.shape[0] != y.shape[0] or out.shape[0] != y.shape[0]:
        raise MvHipError(f"norm weight of {p} {y.dtype} and as many rows of the gate and the output required")
    _check(_lib.mv_head_norm_gate(y.data_ptr(), y.stride(0), gate.data_ptr(), gate.stride(0), w.data_ptr(), out.data_ptr(), out.stride(0),
                                  y.shape[0], heads, p, p_true, float(eps), GATES[gate_kind], float(out_scale), _dt(y), _stream()),
           "mv_head_norm_gate")
    return out


# ---------------------------------------------------------------- K17
MV_ROUTE_SIGMOID, MV_ROUTE_RAW = 1, 2


def moe_route(x, w, correction, top: int, groups: int = 1, keep: int = 1, scale: float = 1.0, sigmoid: bool = False, raw: bool = False):
    """x [T, K], w [outputs, K] -> (ids int32 [T, top], weights fp32 [T, top]).  ``sigmoid``: scores are sigmoids, not a softmax;
    ``raw``: weights are the scores, not divided by their sum."""
    _need_cuda(x, w, correction)
    _rows_ok("x", x, w.shape[1])
    if w.dtype != x.dtype or not w.is_contiguous() or (correction is not None and (correction.dtype != x.dtype
                                                                                   or correction.numel() != w.shape[0])):
        raise MvHipError(f"router weight [outputs, K] and correction [outputs] of {x.dtype} required")
    ids = torch.empty((x.shape[0], top), dtype=torch.int32, device=x.device)
    weights = torch.empty((x.shape[0], top), dtype=torch.float32, device=x.device)
    flags = (MV_ROUTE_SIGMOID if sigmoid else 0) | (MV_ROUTE_RAW if raw else 0)
    _check(_lib.mv_moe_route(x.data_ptr(), x.stride(0), w.data_ptr(), _ptr(correction), ids.data_ptr(), weights.data_ptr(),
                             x.shape[0], w.shape[1], w.shape[0], top, groups, keep, float(scale), flags, _dt(x), _stream()), "mv_moe_route")
    return ids, weights


class ExpertGroups(NamedTuple):
    place: torch.Tensor      # int32 [pairs]; -1: no product
    tokens: torch.Tensor     # int32 [pairs], by place
    tiles: torch.Tensor      # int32 [tiles, 3]
    tile_m: int
    weights: torch.Tensor | None = None   # fp32 [pairs], by place


def moe_group(ids, experts: int, tile_m: int, weights=None) -> ExpertGroups:
    """(token, choice) pairs of ids [T, top] sorted by expert; ``weights`` (fp32 [T, top]): sorted along."""
    _need_cuda(ids, weights)
    pairs, n = ids.numel(), ids.numel() // tile_m + experts
    if ids.dtype != torch.int32 or not ids.is_contiguous():
        raise MvHipError("dense int32 choices [T, top] required")
    place, tokens, tiles = (torch.empty(s, dtype=torch.int32, device=ids.device) for s in ((pairs,), (pairs,), (n, 3)))
    by_place = None
    if weights is not None:
        if weights.dtype != torch.float32 or weights.numel() != pairs or not weights.is_contiguous():
            raise MvHipError("a dense fp32 weight per choice required")
        by_place = torch.empty((pairs,), dtype=torch.float32, device=ids.device)
    _check(_lib.mv_moe_group(ids.data_ptr(), pairs, ids.shape[1], experts, tile_m, n, place.data_ptr(), tokens.data_ptr(),
                             tiles.data_ptr(), _ptr(weights), _ptr(by_place), _stream()), "mv_moe_group")
    return ExpertGroups(place, tokens, tiles, tile_m, by_place)


def moe_linear(x, w, n: int, groups: ExpertGroups, act: GateAct | None = None, gather: bool = False, experts: int = 0,
               in_scale=None):
    """Rows by place: out[i] = W[expert of i] x[i] (``gather``: x[token of i]), W the experts' weights [experts, n, K] -- fp32: as
    they are, 16-bit: packed per expert; ``act``: [experts, 2, n, K], out = act(gate, up).  ``in_scale`` (fp32 by
    place): the inputs are multiplied by it."""
    _need_cuda(x, w, in_scale)
    pairs, k = groups.tokens.numel(), x.shape[1]
    _rows_ok("x", x, 1, w.dtype)
    if not w.is_contiguous() or w.numel() != experts * n * k * (2 if act is not None else 1) or (not gather and x.shape[0] < pairs):
        raise MvHipError(f"expert weights of {experts} x {n} outputs and {k} inputs, and a row of x per place, required")
    out = torch.empty((pairs, n), dtype=x.dtype, device=x.device)
    if in_scale is not None and (in_scale.dtype != torch.float32 or in_scale.numel() != pairs or not in_scale.is_contiguous()):
        raise MvHipError("a dense fp32 factor per place required")
    a = MvMoeLinearArgs(x=x.data_ptr(), w=w.data_ptr(), out=out.data_ptr(), in_scale=_ptr(in_scale), tokens=groups.tokens.data_ptr() if gather else None,
                        tiles=groups.tiles.data_ptr(), act=ctypes.addressof(act) if act is not None else None, x_stride=x.stride(0),
                        out_stride=out.stride(0), max_tiles=groups.tiles.shape[0], tile_m=groups.tile_m, n=n, k=k)
    _check(_lib.mv_moe_linear(ctypes.byref(a), _dt(x), _stream()), "mv_moe_linear")
    return out


# ---------------------------------------------------------------- K18
class StreamShift(NamedTuple):
    """Blend of a normed row with the one of the sequence's token before (include/mvhip.h: mv_stream_update)."""
    share: torch.Tensor         # [cols]
    prev: torch.Tensor          # fp32 [2, slots, cols]
    positions: torch.Tensor
    state_slots: torch.Tensor
    cu_q: torch.Tensor | None = None     # None: one row per sequence


def stream_update(streams: int, norm_w, eps: float, x=None, x_out=None, y=None, mix=None, out_w=None, in_w=None, embed=None, ids=None,
                  experts=None, shift: StreamShift | None = None, cols_true: int | None = None, want_out: bool = True):
    """One edge of fp32 residual streams [rows, streams, cols].  ``embed`` / ``ids``: they start from the embedding; else ``x`` is mixed
    (``mix`` [from, to]) and gets ``out_w`` times y: [rows, cols], fp32 partial sums [splits, rows, cols], and / or ``experts`` (rows
    [pairs, cols], place per pair, weight per pair or None).  The new streams go to ``x_out`` (None: nowhere).  -> the rms norm of
    their sum weighted by ``in_w`` (None: 1), times ``norm_w``, blended by ``shift``."""
    rows, cols, dt = (ids.numel() if embed is not None else x.shape[0]), norm_w.numel(), norm_w.dtype
    _need_cuda(norm_w, x, x_out, y, mix, out_w, in_w, embed, ids)
    for name, t in (("streams", x), ("new streams", x_out)):
        if t is not None and (t.dtype != torch.float32 or tuple(t.shape) != (rows, streams, cols) or not t.is_contiguous()):
            raise MvHipError(f"{name}: dense fp32 [{rows}, {streams}, {cols}] required")
    for name, t, n in (("mix", mix, streams * streams), ("out_w", out_w, streams), ("in_w", in_w, streams),
                       ("shift", shift.share if shift else None, cols)):
        if t is not None and (t.dtype != dt or t.numel() != n or not t.is_contiguous()):
            raise MvHipError(f"{name}: {n} elements of {dt} required")
    a = MvStreamArgs(x=_ptr(x), x_out=_ptr(x_out), mix=_ptr(mix), out_w=_ptr(out_w), in_w=_ptr(in_w), norm_w=norm_w.data_ptr(),
                     streams=streams, eps=float(eps))
    if embed is not None:
        if embed.dtype != dt or embed.shape[1] != cols or not embed.is_contiguous() or ids.dtype != torch.int64 or not ids.is_contiguous():
            raise MvHipError(f"embedding table [vocab, {cols}] of {dt} and int64 ids required")
        a.embed, a.ids, a.vocab = embed.data_ptr(), ids.data_ptr(), embed.shape[0]
    if y is not None:
        if y.dim() == 3:
            if y.dtype != torch.float32 or tuple(y.shape[1:]) != (rows, cols) or not y.is_contiguous():
                raise MvHipError("partial sums must be dense fp32 [splits, rows, cols]")
            a.y_splits = y.shape[0]
        elif tuple(y.shape) != (rows, cols) or y.dtype != dt or y.stride(1) != 1:
            raise MvHipError(f"y must be [{rows}, {cols}] of {dt}")
        a.y, a.y_stride = y.data_ptr(), y.stride(-2)
    if experts is not None:
        rows_out, place, weight = experts
        if (rows_out.dtype != dt or rows_out.shape[1] != cols or not rows_out.is_contiguous() or place.dtype != torch.int32
                or place.numel() % rows or not place.is_contiguous() or (weight is not None and (
                    weight.dtype != torch.float32 or weight.numel() != place.numel() or not weight.is_contiguous()))):
            raise MvHipError(f"expert outputs: dense rows of {cols} {dt}, an int32 place (and an fp32 weight) per choice required")
        a.moe_out, a.moe_rows, a.moe_w, a.moe_top = rows_out.data_ptr(), place.data_ptr(), _ptr(weight), place.numel() // rows
    if shift is not None:
        _need_cuda(*shift)
        n = rows if shift.cu_q is None else shift.cu_q.numel() - 1
        slots = shift.prev.shape[1] if shift.prev.numel() else 0
        if (shift.positions.dtype != torch.int64 or shift.positions.numel() != rows or not shift.positions.is_contiguous()
                or shift.state_slots.dtype != torch.int32 or shift.state_slots.numel() != n or not shift.state_slots.is_contiguous()
                or (slots and (shift.prev.dtype != torch.float32 or tuple(shift.prev.shape) != (2, slots, cols)
                               or not shift.prev.is_contiguous()))
                or (shift.cu_q is not None and (shift.cu_q.dtype != torch.int32 or not shift.cu_q.is_contiguous()))):
            raise MvHipError(f"shift: int64 positions, int32 state slots and fp32 kept rows [2, slots, {cols}] required")
        a.shift, a.prev, a.positions = shift.share.data_ptr(), shift.prev.data_ptr() if slots else None, shift.positions.data_ptr()
        a.state_slots, a.cu_q, a.n_seqs, a.slots = shift.state_slots.data_ptr(), _ptr(shift.cu_q), n, slots
    out = torch.empty((rows, cols), dtype=dt, device=norm_w.device) if want_out else None
    a.out, a.out_stride = _ptr(out), cols
    _check(_lib.mv_stream_update(ctypes.byref(a), rows, cols, cols if cols_true is None else int(cols_true), _DTYPES[dt], _stream()),
           "mv_stream_update")
    return out


# ---------------------------------------------------------------- K19
def _gru_args(z, u, g, state, state_slots, out):
    _need_cuda(z, u, g, state, state_slots, out)
    rows, n = z.shape
    for t in (z, u, g, out):
        if tuple(t.shape) != (rows, n) or t.dtype != z.dtype or t.stride(1) != 1 or (t is not out and t.stride(0) != z.stride(0)):
            raise MvHipError(f"z, u and g: [{rows}, {n}] of {z.dtype} at one row stride, and such an output, required")
    if state_slots.dtype != torch.int32 or not state_slots.is_contiguous():
        raise MvHipError("int32 state slots required")
    a = MvGruArgs(z=z.data_ptr(), u=u.data_ptr(), g=g.data_ptr(), state_slots=state_slots.data_ptr(), out=out.data_ptr(),
                  stride=z.stride(0), out_stride=out.stride(0), n_seqs=state_slots.numel(), total_q=rows, n=n)
    if state is not None and state.numel():
        if state.dtype != torch.float32 or state.shape[0] != 2 or state.shape[2:] != (n,) or not state.is_contiguous():
            raise MvHipError(f"recurrent state must be dense fp32 [2, slots, {n}]")
        a.state, a.slots = state.data_ptr(), state.shape[1]
    return a


def gru_prefill(z, u, g, state, state_slots, cu_q, cu_k, max_q: int, out):
    """The gated running mean over raw projections [T, n] of a batch of sequences; ``out`` [T, n] gets S silu(g)."""
    a = _gru_args(z, u, g, state, state_slots, out)
    a.cu_q, a.cu_k, a.max_q = cu_q.data_ptr(), cu_k.data_ptr(), int(max_q)
    size = int(_lib.mv_gru_prefill_workspace_bytes(a.n_seqs, a.total_q, a.max_q, a.n))
    ws = torch.empty((size,), dtype=torch.uint8, device=z.device) if size else None
    a.workspace, a.ws_bytes = _ptr(ws), size
    _check(_lib.mv_gru_prefill(ctypes.byref(a), _dt(z), _stream()), "mv_gru_prefill")
    return out


def gru_step(z, u, g, state, state_slots, context_lens, out):
    """One token per sequence."""
    a = _gru_args(z, u, g, state, state_slots, out)
    lens = _i32(context_lens)
    if lens.numel() != z.shape[0] or state_slots.numel() != z.shape[0]:
        raise MvHipError("one length and one state slot per row required")
    a.context_lens = lens.data_ptr()
    _check(_lib.mv_gru_step(ctypes.byref(a), _dt(z), _stream()), "mv_gru_step")
    return out
