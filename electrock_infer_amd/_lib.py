"""ctypes binding of libelectrock_moe.so (the C ABI declared in include/electrock_moe.h) and of
libelectrock_decoder.so (include/electrock_decoder.h).

Nothing here computes: each wrapper turns torch tensors into raw device
pointers plus the current HIP stream and raises RuntimeError on a non-zero
status.  There is deliberately no CPU or eager-PyTorch fallback.
"""
import ctypes
import os

from ._build import DECODER_LIB_PATH, LIB_PATH

# element / index type codes of the C ABI
DTYPE_F32, DTYPE_BF16, DTYPE_F16 = 0, 1, 2
ITYPE_I32, ITYPE_I64 = 0, 1

NORM_LAYER, NORM_OP = 0, 1   # rounding points of layers/layernorm.py resp. of the native add_rms_norm op

FLAG_OUT_F32 = 1 << 0
FLAG_GATE_F32_LOGITS = 1 << 2
FLAG_W2_F16 = 1 << 3
FLAG_BF16_ACT = 1 << 5        # SiLU*mul activations stored as bf16 between the GEMMs (the reference's storage type)
FLAG_F32_PARTIALS = 1 << 7    # w2 partial sums stored as float32 at every batch size (default: fp16 + escape above 448 tokens)
# diagnostic switches (include/electrock_moe_diag.h): benchmarks and tests only
FLAG_SKIP_ROUTER = 1 << 8
FLAG_SKIP_ALIGN = 1 << 9
FLAG_SKIP_GEMM1 = 1 << 10
FLAG_SKIP_GEMM2 = 1 << 11
FLAG_SKIP_COMBINE = 1 << 12
FLAG_FORCE_GENERIC = 1 << 16
FLAG_NO_PERSIST = 1 << 17      # one workgroup per tile in the 256-row kernels
FLAG_ONE_GROUP_SORT = 1 << 18  # the layer's sort on one workgroup at every batch size

ERR_STATIC_LIMIT = -8
STATIC_SCRATCH_BYTES = 32 << 20   # EM_STATIC_SCRATCH_BYTES

# every symbol include/electrock_moe.h declares
EXPORTED_SYMBOLS = (
    "em_version", "em_error_string", "em_topk_softmax", "em_moe_align_block_size",
    "em_silu_and_mul", "em_moe_sum", "em_moe_workspace_bytes", "em_moe_workspace_layout",
    "em_moe_forward", "em_moe_forward_gated", "em_gate_topk_softmax", "em_rms_norm", "em_add_rms_norm",
    "em_norm_gate_topk_softmax", "em_moe_forward_normed", "em_moe_forward_static", "em_moe_w2_f16_max_tokens",
)


# every function include/electrock_decoder.h declares
DECODER_SYMBOLS = (
    "ed_version", "ed_embed", "ed_residual_norm", "ed_relu_squared", "ed_silu_gate", "ed_gated_norm", "ed_token_gate", "ed_skinny_gemm_splits", "ed_skinny_gemm",
    "ed_token_side_supported", "ed_token_side", "ed_gla_prefill", "ed_gla_step",
    "ed_recur_record", "ed_recur_prefill", "ed_recur_step",
    "ed_attn_row_elems", "ed_attn_prepare", "ed_attn_paged", "ed_attn_prompt_supported", "ed_attn_prompt",
    "ed_latent_row_elems", "ed_latent_prepare", "ed_latent_paged", "ed_head_gemm", "ed_latent_gather",
    "ed_latent_prompt_supported", "ed_latent_prompt",
)


class GlaArgs(ctypes.Structure):
    """Mirror of struct ed_gla_args."""
    _fields_ = ([(n, ctypes.c_void_p) for n in ("q", "k", "v", "g", "a1")] + [("stride", ctypes.c_int64)] +
                [(n, ctypes.c_void_p) for n in ("a2", "bias", "norm_w", "out", "slots", "starts", "states", "log_decay",
                                                "chunks", "seq_chunks", "chunk_states", "chunk_decay")] +
                [(n, ctypes.c_int32) for n in ("n_seqs", "n_chunks", "chunk_tokens", "heads", "dim", "vdim", "rank",
                                               "a2_stride", "dtype")] +
                [(n, ctypes.c_float) for n in ("tau", "q_scale", "eps")])


class RecurArgs(ctypes.Structure):
    """Mirror of struct ed_recur_args."""
    _fields_ = ([(n, ctypes.c_void_p) for n in ("q", "k", "v", "decay_in", "beta_in", "gate")] + [("stride", ctypes.c_int64)] +
                [(n, ctypes.c_void_p) for n in ("conv_w", "conv_b", "a_log", "dt_bias", "skip", "norm_w", "ring", "states", "out",
                                                "slots", "starts", "q_begin", "chunks", "seq_chunks", "q_rows", "k_rows",
                                                "v_rows", "rates", "blocks", "chunk_states", "chunk_trans")] +
                [(n, ctypes.c_int32) for n in ("n_seqs", "n_chunks", "chunk_tokens", "heads", "kv_heads", "dim", "vdim", "taps",
                                               "dtype")] +
                [(n, ctypes.c_float) for n in ("q_scale", "unit_eps", "eps")])


class AttnArgs(ctypes.Structure):
    """Mirror of struct ed_attn_args."""
    _fields_ = ([(n, ctypes.c_void_p) for n in ("q", "k", "v")] + [("stride", ctypes.c_int64), ("v_first", ctypes.c_void_p),
                                                                   ("v_first_stride", ctypes.c_int64)] +
                [(n, ctypes.c_void_p) for n in ("mix", "q_norm", "k_norm", "inv_freq", "positions", "cache_rows", "cache", "q_rows",
                                                "out", "q_begin", "starts", "tables", "part_o", "part_ml")] +
                [("T", ctypes.c_int64)] +
                [(n, ctypes.c_int32) for n in ("n_seqs", "max_q", "table_width", "block_size", "splits", "heads", "kv_heads", "dim",
                                               "vdim", "rot", "window", "dtype")] +
                [(n, ctypes.c_float) for n in ("scale", "softcap", "eps")])


class LatentArgs(ctypes.Structure):
    """Mirror of struct ed_latent_args."""
    _fields_ = ([("q", ctypes.c_void_p), ("q_stride", ctypes.c_int64), ("down", ctypes.c_void_p),
                 ("down_stride", ctypes.c_int64)] +
                [(n, ctypes.c_void_p) for n in ("latent_w", "inv_freq", "positions", "cache_rows", "cache", "q_latent",
                                                "out", "sink", "q_begin", "starts", "tables", "part_o", "part_ml")] +
                [("T", ctypes.c_int64)] +
                [(n, ctypes.c_int32) for n in ("n_seqs", "max_q", "table_width", "block_size", "splits", "heads", "dim",
                                               "rot", "rank", "dtype")] +
                [(n, ctypes.c_float) for n in ("scale", "eps")])


class LatentPromptArgs(ctypes.Structure):
    """Mirror of struct ed_latent_prompt_args."""
    _fields_ = ([(n, t) for name in ("q", "k", "k_rot", "vt") for n, t in
                 ((name, ctypes.c_void_p), (("v" if name == "vt" else name) + "_stride", ctypes.c_int64))] +
                [(n, ctypes.c_void_p) for n in ("out", "sink", "q_begin", "starts", "k_begin")] +
                [(n, ctypes.c_int32) for n in ("n_seqs", "max_q", "heads", "dim", "rot", "vdim")] +
                [("scale", ctypes.c_float)])


class MoeLayout(ctypes.Structure):
    """Mirror of struct em_moe_layout."""
    _fields_ = [(n, ctypes.c_int64) for n in (
        "block_size", "topk_weights_off", "topk_ids_off", "sorted_ids_off", "sorted_len",
        "expert_ids_off", "expert_ids_len", "post_pad_off", "seg_begin_off", "tickets_off", "saturated_off",
        "sort_scratch_off", "act_off", "act_lo_off", "y_off", "ksplit", "y_wide_off",
        "total_bytes")]


_lib = None


def load() -> ctypes.CDLL:
    """Load the built library; raise if it has not been built."""
    global _lib
    if _lib is not None:
        return _lib
    if not os.path.exists(LIB_PATH):
        raise RuntimeError(
            f"{LIB_PATH} is missing: build it with `python -m electrock_infer_amd._build` "
            "(there is no fallback implementation)")
    lib = ctypes.CDLL(LIB_PATH)
    vp, i32, i64, u32, sz = ctypes.c_void_p, ctypes.c_int, ctypes.c_int64, ctypes.c_uint, ctypes.c_size_t
    lib.em_version.restype = i32
    lib.em_version.argtypes = []
    lib.em_error_string.restype = ctypes.c_char_p
    lib.em_error_string.argtypes = [i32]
    lib.em_topk_softmax.restype = i32
    lib.em_topk_softmax.argtypes = [vp, i32, i64, i32, i32, i32, vp, vp, vp]
    lib.em_moe_align_block_size.restype = i32
    lib.em_moe_align_block_size.argtypes = [vp, i32, i64, i32, i32, vp, i64, vp, i64, vp, vp]
    lib.em_silu_and_mul.restype = i32
    lib.em_silu_and_mul.argtypes = [vp, vp, i64, i64, i32, vp]
    lib.em_moe_sum.restype = i32
    lib.em_moe_sum.argtypes = [vp, vp, i64, i32, i64, i32, vp]
    lib.em_moe_w2_f16_max_tokens.restype = i64
    lib.em_moe_w2_f16_max_tokens.argtypes = [i32, i32, i32, i32]
    lib.em_moe_workspace_bytes.restype = sz
    lib.em_moe_workspace_bytes.argtypes = [i64, i32, i32, i32, i32, u32]
    lib.em_moe_workspace_layout.restype = i32
    lib.em_moe_workspace_layout.argtypes = [i64, i32, i32, i32, i32, u32, ctypes.POINTER(MoeLayout)]
    lib.em_moe_forward.restype = i32
    lib.em_moe_forward.argtypes = [vp, vp, i32, vp, vp, vp, i64, i32, i32, i32, i32, i32, vp, sz, u32, vp]
    lib.em_moe_forward_static.restype = i32
    lib.em_moe_forward_static.argtypes = [vp, vp, i32, vp, vp, vp, i64, i32, i32, i32, i32, i32, u32, vp]
    lib.em_moe_forward_gated.restype = i32
    lib.em_moe_forward_gated.argtypes = [vp, vp, vp, vp, vp, i64, i32, i32, i32, i32, i32, vp, sz, u32, vp]
    lib.em_gate_topk_softmax.restype = i32
    lib.em_gate_topk_softmax.argtypes = [vp, vp, i64, i32, i32, i32, i32, i32, vp, vp, vp, vp]
    lib.em_rms_norm.restype = i32
    lib.em_rms_norm.argtypes = [vp, vp, vp, i64, i32, ctypes.c_double, i32, i32, i32, vp]
    lib.em_add_rms_norm.restype = i32
    lib.em_add_rms_norm.argtypes = [vp, vp, vp, vp, vp, i64, i32, ctypes.c_double, i32, i32, i32, vp]
    lib.em_norm_gate_topk_softmax.restype = i32
    lib.em_norm_gate_topk_softmax.argtypes = [vp, vp, vp, i32, ctypes.c_double, i32, vp, vp, vp, i64, i32, i32, i32, i32,
                                              i32, vp, vp, vp, vp]
    lib.em_moe_forward_normed.restype = i32
    lib.em_moe_forward_normed.argtypes = [vp, vp, vp, i32, ctypes.c_double, i32, vp, vp, vp, vp, vp, vp, i64, i32, i32,
                                          i32, i32, i32, vp, sz, u32, vp]
    _lib = lib
    return lib


def check(code: int, what: str) -> None:
    if code != 0:
        msg = load().em_error_string(code).decode()
        raise RuntimeError(f"{what} failed: {msg} (status {code})")


_decoder_lib = None


def load_decoder() -> ctypes.CDLL:
    """Load the built decoder library; raise if it has not been built."""
    global _decoder_lib
    if _decoder_lib is not None:
        return _decoder_lib
    if not os.path.exists(DECODER_LIB_PATH):
        raise RuntimeError(
            f"{DECODER_LIB_PATH} is missing: build it with `python -m electrock_infer_amd._build decoder` "
            "(there is no fallback implementation)")
    lib = ctypes.CDLL(DECODER_LIB_PATH)
    vp, i32, i64, dbl = ctypes.c_void_p, ctypes.c_int, ctypes.c_int64, ctypes.c_double
    signatures = {
        "ed_version": [],
        "ed_embed": [vp, vp, dbl, vp, vp, i64, i64, i32, i32, vp],
        "ed_skinny_gemm_splits": [i64, i32, i32],
        "ed_skinny_gemm": [vp, vp, vp, i32, i32, i64, i32, i32, i32, vp],
        "ed_residual_norm": [i32, vp, vp, i32, i32, vp, vp, vp, i64, i64, i32, dbl, i32, vp],
        "ed_relu_squared": [vp, i64, i32, vp],
        "ed_silu_gate": [vp, vp, i64, i32, i32, vp],
        "ed_gated_norm": [vp, vp, i64, vp, i64, i32, i32, dbl, i32, vp],
        "ed_recur_record": [i32],
        "ed_recur_prefill": [ctypes.POINTER(RecurArgs), vp],
        "ed_recur_step": [ctypes.POINTER(RecurArgs), vp],
        "ed_attn_row_elems": [i32, i32, i32],
        "ed_attn_prepare": [ctypes.POINTER(AttnArgs), vp],
        "ed_attn_paged": [ctypes.POINTER(AttnArgs), vp],
        "ed_attn_prompt_supported": [i32, i32],
        "ed_attn_prompt": [ctypes.POINTER(AttnArgs), vp],
        "ed_token_gate": [vp, vp, vp, vp, i64, i32, vp, i64, i32, i32, i32, vp],
        "ed_token_side_supported": [i32, i32],
        "ed_token_side": [vp, vp, vp, vp, vp, vp, vp, i64, i32, vp, vp, vp, i64, i64, i32, i32, dbl, vp],
        "ed_gla_prefill": [ctypes.POINTER(GlaArgs), vp],
        "ed_gla_step": [ctypes.POINTER(GlaArgs), vp],
        "ed_latent_row_elems": [i32, i32],
        "ed_latent_prepare": [ctypes.POINTER(LatentArgs), vp],
        "ed_latent_paged": [ctypes.POINTER(LatentArgs), vp],
        "ed_head_gemm": [vp, i64, i64, vp, vp, i64, i64, i64, i32, i32, i32, i32, vp],
        "ed_latent_prompt_supported": [i32, i32, i32],
        "ed_latent_prompt": [ctypes.POINTER(LatentPromptArgs), vp],
        "ed_latent_gather": [vp, vp, i32, i32, vp, vp, i32, i32, i32, vp, i32, vp],
    }
    for name, argtypes in signatures.items():
        fn = getattr(lib, name)
        fn.restype, fn.argtypes = i32, argtypes
    _decoder_lib = lib
    return lib


ERROR_TEXT = {-1: "null pointer", -2: "bad shape", -3: "unsupported element type", -4: "unsupported shape or option",
              -5: "workspace missing or too small", -7: "misaligned pointer"}


def check_decoder(code: int, what: str) -> None:
    if code != 0:
        raise RuntimeError(f"{what} failed: {ERROR_TEXT.get(code, 'HIP error')} (status {code})")


def dtype_code(dtype) -> int:
    import torch
    try:
        return {torch.float32: DTYPE_F32, torch.bfloat16: DTYPE_BF16, torch.float16: DTYPE_F16}[dtype]
    except KeyError:
        raise RuntimeError(f"unsupported element type {dtype}") from None


def current_stream(device) -> int:
    import torch
    return torch.cuda.current_stream(device).cuda_stream


def require_device(*tensors) -> None:
    for t in tensors:
        if not t.is_cuda:
            raise RuntimeError("tensor must be on a GPU device (no CPU path exists)")
        if not t.is_contiguous():
            raise RuntimeError("tensor must be contiguous")


def workspace_layout(T: int, H: int, I: int, E: int, top_k: int, flags: int = 0) -> MoeLayout:
    L = MoeLayout()
    check(load().em_moe_workspace_layout(T, H, I, E, top_k, flags, ctypes.byref(L)), "em_moe_workspace_layout")
    return L
