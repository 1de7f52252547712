"""ctypes binding of libmetaseq_amd.so and libmetaseq_hybrid.so (the C ABIs declared in
include/metaseq_amd.h and include/metaseq_hybrid.h).

There is no fallback: if the library is missing or a call fails, an exception is raised.
Shape / argument errors surface as ValueError, capacity overruns as ValueError, HIP
failures as RuntimeError (the reference's serving loop treats a RuntimeError from
``generate`` as a device fault and restarts the worker, metaseq/cli/interactive_hosted.py:161-171).
"""
import ctypes
import os
from ctypes import c_char_p, c_float, c_int, c_int32, c_int64, c_size_t, c_uint, c_void_p

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "csrc", "libmetaseq_amd.so")

MSA_EPI_RELU = 1
MSA_IN_PACKED = 2
MSA_OUT_PACKED = 4
MSA_EMBED_COL_FROM_LEN = 8
MSA_EMBED_ROWS_GIVEN = 32
MSA_ROW_BAN_EARLY = 1
MSA_ROW_ONLY_EOS = 2
MSA_ROW_SKIP = 4

_P = c_void_p
MSA_STEP_NO_ADVANCE = 16


class DecoderConfig(ctypes.Structure):
    """msa_decoder_config"""
    _fields_ = [(n, c_int) for n in ("layers", "d_model", "heads", "ffn", "vocab", "n_pos_rows",
                                     "pad_idx", "int8")]


class LayerWeights(ctypes.Structure):
    """msa_layer_weights: device pointers of one layer's parameters."""
    _fields_ = [(n, c_void_p) for n in (
        "ln1_gamma", "ln1_beta", "qkv_weight", "qkv_scales", "qkv_bias", "out_weight",
        "out_scales", "out_bias", "ln2_gamma", "ln2_beta", "fc1_weight", "fc1_scales",
        "fc1_bias", "fc2_weight", "fc2_scales", "fc2_bias")]


class StepArgs(ctypes.Structure):
    """msa_step_args"""
    _fields_ = [("tokens", c_void_p), ("tok_stride", c_int64), ("n", c_int), ("B", c_int),
                ("k_cache", ctypes.POINTER(c_void_p)), ("v_cache", ctypes.POINTER(c_void_p)),
                ("S0", c_int), ("S_cap", c_int), ("len_dev", c_void_p),
                ("key_pad_mask", c_void_p), ("mask_stride", c_int64), ("flags", c_uint),
                ("workspace", c_void_p), ("workspace_bytes", c_int64), ("logits", c_void_p),
                ("tok", c_void_p), ("tok_stride_out", c_int64), ("score", c_void_p),
                ("score_stride", c_int64), ("temperature", c_float),
                ("banned", ctypes.POINTER(c_int32)), ("n_banned", c_int),
                ("stop", ctypes.POINTER(c_int32)), ("n_stop", c_int), ("finished", c_void_p),
                ("row_mode", c_void_p), ("force_eos_all", c_int), ("eos_idx", c_int),
                ("col_dev", c_void_p)]


# name -> argtypes, in the order of include/metaseq_amd.h
SIGNATURES = {
    "msa_pack_weight_f16": [_P, _P, c_int, c_int, _P],
    "msa_unpack_weight_f16": [_P, _P, c_int, c_int, _P],
    "msa_pack_weight_i8": [_P, _P, c_int, c_int, _P],
    "msa_unpack_weight_i8": [_P, _P, c_int, c_int, _P],
    "msa_expand_weight_w8_f16": [_P, _P, _P, c_int, c_int, _P],
    "msa_layernorm_f16": [_P, _P, _P, _P, c_int64, c_int, c_float, c_uint, _P],
    "msa_residual_layernorm_f16": [_P, c_int, _P, _P, _P, _P, _P, c_int64, c_int, c_float, c_uint,
                                   _P],
    "msa_advance_len": [_P, _P, c_int, c_int, _P],
    "msa_embed_f16": [_P, c_int64, c_int, c_int, c_int, _P, c_int, _P, c_int, c_int, c_int, _P, _P,
                      _P, _P, _P, c_uint, _P],
    "msa_linear_f16": [_P, _P, _P, _P, _P, c_int64, c_int, c_int, c_uint, _P],
    "msa_linear_w8a16": [_P, _P, _P, _P, _P, _P, c_int64, c_int, c_int, c_uint, _P],
    "msa_linear_partial_f16": [_P, _P, _P, c_int64, c_int, c_int, c_int, c_uint, _P],
    "msa_linear_partial_w8a16": [_P, _P, _P, _P, c_int64, c_int, c_int, c_int, c_uint, _P],
    "msa_linear_default_splits": [c_int64, c_int, c_int],
    "msa_linear_default_splits_w8a16": [c_int64, c_int, c_int],
    "msa_linear_default_splits_rows": [c_int64, c_int, c_int],
    "msa_qkv_proj_f16": [_P, _P, _P, _P, _P, _P, c_int, c_int, c_int, c_int, c_int, c_int, c_int,
                         c_uint, _P, _P],
    "msa_qkv_proj_w8a16": [_P, _P, _P, _P, _P, _P, _P, c_int, c_int, c_int, c_int, c_int, c_int,
                           c_int, c_uint, _P, _P],
    "msa_attention_f16": [_P, _P, _P, _P, c_int64, _P, c_int, c_int, c_int, c_int, c_int, c_int,
                          c_uint, _P, _P],
    "msa_attention_split_f16": [_P, _P, _P, _P, c_int64, _P, _P, c_int, c_int, c_int, c_int, c_int,
                                c_uint, _P, _P],
    "msa_attention_prefers_split": [c_int, c_int, c_int, c_int],
    "msa_greedy_select_f16": [_P, c_int64, c_int, c_int, c_float, _P, c_int, _P, c_int, _P, _P,
                              c_int, c_int, _P, c_int64, _P, c_int64, _P, _P],
    "msa_sample_topp_f16": [_P, c_int64, c_int, c_int, c_float, _P, _P, c_int, _P, c_int, _P, _P,
                            c_int, c_int, _P, c_float, _P, _P, _P, c_float, c_float, c_float,
                            c_float, _P, _P, c_int64, _P, c_int64, _P, c_int64, _P],
    "msa_log_softmax_f16": [_P, c_int64, c_int64, c_int, c_int, c_int, c_float, _P, c_int64,
                            c_int64, _P],
    "msa_target_logprob_f16": [_P, c_int64, c_int64, c_int, c_float, _P, _P, _P],
    "msa_lm_head_greedy_select_f16": [_P, _P, _P, _P, c_int, c_int, c_int, c_float, _P, c_int, _P,
                                      c_int, _P, _P, c_int, c_int, _P, c_int64, _P, c_int64, _P,
                                      _P],
    "msa_lm_head_greedy_select_noalloc_f16": [_P, _P, _P, c_int, c_int, c_int, c_float, _P, c_int,
                                              _P, c_int, _P, _P, c_int, c_int, _P, c_int64, _P,
                                              c_int64, _P, _P],
    "msa_decoder_create": [ctypes.POINTER(DecoderConfig), _P, _P, _P, _P, _P,
                           ctypes.POINTER(LayerWeights), ctypes.POINTER(c_void_p)],
    "msa_decoder_step": [_P, ctypes.POINTER(StepArgs), _P],
    "msa_probe_stream_read": [_P, c_int64, _P],
}
for _n in ("msa_greedy_select", "msa_sample_topp", "msa_log_softmax", "msa_target_logprob"):
    SIGNATURES[_n + "_f32"] = SIGNATURES[_n + "_f16"]  # the same over fp32 logits
OTHER_SYMBOLS = ["msa_last_error", "msa_version", "msa_lm_head_select_workspace_bytes",
                 "msa_decoder_destroy", "msa_decoder_step_workspace_bytes",
                 "msa_attention_split_workspace_bytes"]

# ---- the hybrid library (include/metaseq_hybrid.h) -----------------------------------------
HYBRID_LIB_PATH = os.path.join(_HERE, "csrc", "libmetaseq_hybrid.so")
MSA_BF16, MSA_F32 = 0, 1
MSA_GLU_NONE, MSA_GLU_GELU, MSA_GLU_CLAMPED = -1, 0, 1
MSA_ACT_NONE, MSA_ACT_RELU2 = 0, 1
MSA_GATE_SILU, MSA_GATE_SIGMOID = 0, 1
MSA_MIX_LATENT, MSA_MIX_RGLRU, MSA_MIX_DELTA, MSA_MIX_PARALLEL = 0, 1, 2, 3
MSA_FF_NONE, MSA_FF_DENSE, MSA_FF_MOE, MSA_FF_RELU2 = 0, 1, 2, 3
MSA_OUT2_PACKED = 16
_I32P = ctypes.POINTER(c_int32)


def _struct(name, doc, *groups):
    """A ctypes structure from (type, "field field ...") groups."""
    fields = [(n, t) for t, names in groups for n in names.split()]
    return type(name, (ctypes.Structure,), {"_fields_": fields, "__doc__": doc})


Batch = _struct("Batch", "msa_batch", (c_int, "M nseg max_count key_bound"),
                (c_void_p, "tok_slot tok_pos tok_off seg_start seg_slot seg_pos"),
                (_I32P, "host_start host_slot host_pos"))
GroupLinearArgs = _struct(
    "GroupLinearArgs", "msa_group_linear_args", (c_int, "dtype"), (c_void_p, "x"),
    (c_int64, "ldx"), (c_int, "x_group x_groups x_mb"), (c_void_p, "W y"), (c_int64, "ldy"),
    (c_int, "y_group y_mb y_f32 y_row0 N K groups glu"), (c_float, "limit"), (c_int64, "M"),
    (c_void_p, "perm tile_group tile_row n_tiles group_end"),
    (c_int, "rows_per_x max_tiles tile_rows"))
LinearArgs = _struct(
    "LinearArgs", "msa_linear_args", (c_int, "dtype"), (c_void_p, "x W"), (c_int64, "M"),
    (c_int, "N K n32 n2 act"), (c_uint, "flags"), (c_void_p, "bias decay_rate y y2 y32"))
TailArgs = _struct("TailArgs", "msa_tail_args", (c_int, "dtype M D Dp S S2 top h_mb"),
                   (c_float, "eps"), (c_void_p, "part gate pair_w pair_y inverse"),
                   (c_void_p, "bias part2 w_post2 add step probe w_post w_next x h"))
DeltaArgs = _struct(
    "DeltaArgs", "msa_delta_args", (c_int, "dtype heads kv_heads dim dp vdim vp gate_act"),
    (c_void_p, "qkv"), (c_int64, "ld"), (c_void_p, "ba"), (c_int, "ldba"),
    (c_void_p, "decay_rate dt_bias decay state o gate"), (c_int64, "ld_gate"), (c_void_p, "w"),
    (c_float, "eps"), (c_void_p, "out"), (c_int64, "ld_out"), (c_int, "out_mb"))
GroupedArgs = _struct(
    "GroupedArgs", "msa_grouped_args", (c_int, "dtype heads kv_heads hd vd chunk rot_dims rows"),
    (c_float, "scale"), (c_void_p, "inv_freq q k v"), (c_int64, "ld"),
    (c_void_p, "k_cache v_cache gate"), (c_int, "ld_gate"), (c_void_p, "out"), (c_int64, "ldo"),
    (c_int, "out_mb"), (c_void_p, "partial"), (c_int, "splits fused"))
AttentionLayer = _struct(
    "AttentionLayer", "msa_attention_layer", (c_int, "heads kv_heads hd vd chunk rot_dims ko"),
    (c_float, "scale"), (c_void_p, "inv_freq w_out out_norm"))
HybridLayer = _struct(
    "HybridLayer", "msa_hybrid_layer", (c_int, "kind heads hd q_rank qp kv_rank rp kv_from"),
    (c_float, "scale"), (c_void_p, "w_in w_q w_kv w_absorb w_v wq_norm wkv_norm"),
    (c_int, "kv_heads dim dp vdim vp channels blocks taps"),
    (c_void_p, "conv_w conv_b in_bias y_bias gate_bias lam decay_rate dt_bias o_norm w_gates"),
    (AttentionLayer, "att"), (c_int, "lr"), (c_void_p, "w_lr lr_bias lr_rate out_norm w_out"),
    (c_int, "n_in ko"), (c_void_p, "norm1 norm1b norm2 norm2b"),
    (c_int, "ff_kind ff experts top n_groups keep ff_expert ff_shared"),
    (c_float, "router_scale limit_expert limit_shared"), (c_void_p, "w_ff_in"),
    (c_int, "n_ff_in"), (c_void_p, "ff_bias ff_down_bias w_ff_down w_e_in w_e_down"))
HybridConfigC = _struct("HybridConfigC", "msa_hybrid_config",
                        (c_int, "dtype layers D Dp vocab Vp"), (c_float, "eps embed_scale"),
                        (c_void_p, "embed inv_freq final_norm head"), (c_int, "n_runs"),
                        (ctypes.POINTER(ctypes.c_int32), "run_layer run_pass"),
                        (c_void_p, "loop_step"))
HybridState = _struct("HybridState", "msa_hybrid_state", (c_void_p, "latent conv rec keys values"),
                      (c_int, "kv_rows"))
HybridStepArgs = _struct(
    "HybridStepArgs", "msa_hybrid_step_args", (Batch, "batch"), (c_void_p, "tokens"),
    (ctypes.POINTER(HybridState), "state"), (c_int, "capacity"), (c_void_p, "rows"),
    (c_int, "n_rows"), (c_void_p, "logits probe workspace"), (c_int64, "workspace_bytes"))

_BP = ctypes.POINTER(Batch)
HYBRID_SIGNATURES = {
    "msa_linear_bf16": [_P, _P, _P, _P, c_int64, c_int, c_int, c_int, c_int, c_float, c_uint, _P],
    "msa_linear_f32": [_P, _P, _P, _P, c_int64, c_int, c_int, c_int, c_int, c_float, _P],
    "msa_linear": [ctypes.POINTER(LinearArgs), _P],
    "msa_linear_partial_bf16": [_P, _P, _P, c_int64, c_int, c_int, c_int, c_uint, _P],
    "msa_linear_bf16_splits": [c_int64, c_int, c_int, c_int],
    "msa_group_linear": [ctypes.POINTER(GroupLinearArgs), _P],
    "msa_moe_route": [_P, c_int, c_int, c_int, c_int, c_int, c_int, c_float, _P, _P, _P, _P],
    "msa_moe_plan": [_P, c_int, c_int, c_int, _P, _P, _P, _P, _P, _P, c_int, _P],
    "msa_embed_rmsnorm": [c_int, _P, _P, c_int, _P, c_int, c_float, _P, c_int, c_int, c_float, _P,
                          _P, _P, _P, _P, c_int, _P],
    "msa_residual_rmsnorm_tail": [ctypes.POINTER(TailArgs), _P],
    "msa_short_conv": [c_int, _P, c_int64, c_int, c_int, _P, _P, _P, c_int, _P, c_int64, _P, _BP,
                       _P],
    "msa_conv_state": [c_int, _P, c_int64, c_int, c_int, _P, _BP, _P],
    "msa_rglru_chunks": [c_int],
    "msa_rglru_scan": [c_int, _P, _P, _P, _P, c_int64, _P, c_int64, _P, c_int, _P, _P, _P, c_int64,
                       c_int, _BP, _P],
    "msa_delta_scan": [ctypes.POINTER(DeltaArgs), _BP, _P],
    "msa_delta_output": [ctypes.POINTER(DeltaArgs), c_int, _P],
    "msa_delta_step": [ctypes.POINTER(DeltaArgs), _BP, _P],
    "msa_grouped_rotate": [ctypes.POINTER(GroupedArgs), _BP, _P],
    "msa_grouped_append": [ctypes.POINTER(GroupedArgs), _BP, _P],
    "msa_grouped_attention_splits": [ctypes.POINTER(GroupedArgs), c_int, c_int],
    "msa_grouped_fuses": [ctypes.POINTER(GroupedArgs), _BP],
    "msa_grouped_attention": [ctypes.POINTER(GroupedArgs), _BP, c_int, c_int, c_int, _P],
    "msa_latent_norm": [c_int, _P, c_int, c_int, c_int, c_int, c_int, _P, c_int, c_int, _P,
                        c_float, _P, c_int, _P, c_int, _BP, _P],
    "msa_latent_attention_splits": [c_int, c_int, c_int, c_int, c_int],
    "msa_latent_attention": [c_int, _P, _P, c_int, c_int, c_int, c_float, _P, _P, c_int, _P, _P,
                             c_int, _P],
    "msa_flash_attention_bf16": [_P, c_int64, _P, c_int64, _P, c_int64, c_int, c_int, c_int, c_int,
                                 c_int, c_int, c_float, _P],
    "msa_zero_columns": [c_int, _P, c_int64, c_int64, c_int, c_int, c_int, _P],
    "msa_gather_rows": [c_int, _P, c_int, _P, c_int, c_int, _P, c_int, _P],
    "msa_step_positions": [_P, _P, c_int64, c_int64, c_int, _P, _P],
    "msa_advance_active": [_P, _P, c_int, _P],
    "msa_hybrid_create": [ctypes.POINTER(HybridConfigC), ctypes.POINTER(HybridLayer),
                          ctypes.POINTER(c_void_p)],
    "msa_hybrid_step": [_P, ctypes.POINTER(HybridStepArgs), _P],
}
HYBRID_OTHER_SYMBOLS = ["msa_hybrid_destroy", "msa_hybrid_workspace_bytes"]

_lib = None
_hybrid_lib = None


def _open(path):
    if not os.path.exists(path):
        raise RuntimeError(
            "metaseq_amd: %s is missing - build it with `python -m metaseq_amd.csrc.build` "
            "(there is no non-HIP fallback)" % path)
    lib = ctypes.CDLL(path)
    lib.msa_last_error.argtypes = []
    lib.msa_last_error.restype = c_char_p
    lib.msa_version.argtypes = []
    lib.msa_version.restype = c_int
    return lib


def load_hybrid():
    """Loads the hybrid decoders' library once; raises if it has not been built."""
    global _hybrid_lib
    if _hybrid_lib is None:
        lib = _open(HYBRID_LIB_PATH)
        for name, args in HYBRID_SIGNATURES.items():
            fn = getattr(lib, name)
            fn.argtypes = args
            fn.restype = c_int
        lib.msa_hybrid_destroy.argtypes = [_P]
        lib.msa_hybrid_destroy.restype = None
        lib.msa_hybrid_workspace_bytes.argtypes = [_P, ctypes.POINTER(HybridStepArgs)]
        lib.msa_hybrid_workspace_bytes.restype = c_int64
        _hybrid_lib = lib
    return _hybrid_lib


def load():
    """Loads the shared library once; raises if it has not been built."""
    global _lib
    if _lib is not None:
        return _lib
    lib = _open(LIB_PATH)
    for name, args in SIGNATURES.items():
        fn = getattr(lib, name)
        fn.argtypes = args
        fn.restype = c_int
    lib.msa_lm_head_select_workspace_bytes.argtypes = [c_int]
    lib.msa_lm_head_select_workspace_bytes.restype = c_int64
    lib.msa_decoder_destroy.argtypes = [_P]
    lib.msa_decoder_destroy.restype = None
    lib.msa_decoder_step_workspace_bytes.argtypes = [_P, c_int]
    lib.msa_decoder_step_workspace_bytes.restype = c_int64
    lib.msa_attention_split_workspace_bytes.argtypes = [c_int, c_int, c_int]
    lib.msa_attention_split_workspace_bytes.restype = c_int64
    _lib = lib
    return lib


def check(rc, lib=None):
    if rc == 0:
        return
    lib = lib or load()
    msg = lib.msa_last_error().decode("utf-8", "replace")
    if rc == -3:
        raise RuntimeError("metaseq_amd HIP failure: " + msg)
    raise ValueError("metaseq_amd: " + msg)


def for_logits(lib, name, logits):
    """The entry point ``name`` for logits of this dtype (fp16 or fp32)."""
    import torch

    return getattr(lib, name + {torch.float16: "_f16", torch.float32: "_f32"}[logits.dtype])


def ptr(t):
    """Device pointer of a torch tensor (or NULL for None)."""
    return None if t is None else t.data_ptr()


def stream_ptr():
    """hipStream_t of torch's current stream, so kernels order with torch's own work."""
    import torch

    return torch.cuda.current_stream().cuda_stream
