"""ctypes view of the C ABI declared in include/catgrad_hip.h.

The same binding serves any shared library that exports the ABI; the package
itself only ever loads the HIP library (see `catgrad_amd.backend`).
"""
from __future__ import annotations

import ctypes as C

MAX_RANK = 8

# enum cg_dtype — order of `enum Dtype` (catgrad/src/category/core.rs:23-29)
F32, F16, BF16, F8, U32 = 0, 1, 2, 3, 4
DTYPE_NAMES = {F32: "f32", F16: "f16", BF16: "bf16", F8: "f8", U32: "u32"}

# enum cg_status
OK, ERR_SHAPE, ERR_DTYPE, ERR_RANGE, ERR_DEVICE, ERR_UNSUPPORTED, ERR_ARG = range(7)

# enum cg_unary_op / cg_binary_op
NEG, SIN, COS, EXP, LOG, FLOOR, ROUND = range(7)
ADD, SUB, MUL, DIV, POW, LT, GT, GTE, LTE, EQ = range(10)

# enum cg_kernel_class
K_GEMM_MFMA, K_GEMM_SKINNY, K_GEMM_SIMPLE, K_ELEMENTWISE, K_REDUCE, K_GATHER, K_ATTENTION, K_PACK, K_RECURRENCE = range(9)

_P = C.c_void_p
_PP = C.POINTER(C.c_void_p)
_SZ = C.c_size_t
_SZP = C.POINTER(C.c_size_t)
_I = C.c_int


# cg_linear_args, cg_pair_embedding_args, cg_conv_input, cg_conv_linear_args, cg_experts, cg_branch, cg_token_side_args,
# cg_attention_args, cg_channel_delta_args
class LinearArgs(C.Structure):
    _fields_ = [(n, _P) for n in ("x", "x2", "gamma", "w", "bias")] + [("eps", C.c_float), ("scale", C.c_float), ("groups", _SZ)]


class PairEmbeddingArgs(C.Structure):
    _fields_ = [(n, _P) for n in ("ids", "previous", "table", "pairs")] + [("mul_prev", _SZ), ("mul_cur", _SZ)]


class ConvInput(C.Structure):
    _fields_ = [(n, _P) for n in ("gamma", "conv", "w")] + [("keep", _I), ("keep_bf16", _I)]


class ConvLinearArgs(C.Structure):
    _fields_ = [("x", _P), ("state", _P), ("in_", ConvInput * 2), ("n", _SZ), ("groups", _SZ), ("eps", C.c_float)]


class Experts(C.Structure):
    _fields_ = ([(n, _P) for n in ("h", "logits", "correction", "gate_up", "down")] + [(n, _SZ) for n in ("top", "groups", "keep")]
                + [("limit", C.c_float), ("slope", C.c_float)])


class TokenSideArgs(C.Structure):
    _fields_ = ([(n, _P) for n in ("x", "ids", "table", "gate", "proj", "norm")] + [("first", _SZ), ("eps", C.c_float), ("scale", C.c_float)])


class Branch(C.Structure):
    _fields_ = [(n, _P) for n in ("y", "w", "gate", "gate_bias", "poly")]


class AttentionArgs(C.Structure):
    _fields_ = ([(n, _P) for n in ("q", "k", "v", "q_norm", "k_norm", "talk", "k_cache", "v_cache")]
                + [(n, _SZ) for n in ("heads", "kv_heads", "dim", "vdim", "position", "window", "temp_every")]
                + [("scale", C.c_float), ("norm_eps", C.c_float), ("temp_coef", C.c_float), ("distance_bias", _I), ("rot_dims", _SZ),
                   ("rot_base", C.c_double), ("unit_heads", _I), ("mix_scores", _I), ("zero_sink", _I)])


class ChannelDeltaArgs(C.Structure):
    _fields_ = ([(n, _P) for n in ("q", "k", "v", "conv_q", "conv_k", "conv_v", "beta", "decay", "decay_w", "a_log", "dt_bias",
                                   "gate", "gate_w", "norm", "state", "conv_state")]
                + [(n, _SZ) for n in ("heads", "kv_heads", "dim", "vdim")] + [("eps", C.c_float)])


# name -> (restype, argtypes); every symbol the header declares.
SIGNATURES = {
    "cg_backend_create": (_I, [_I, _PP]),
    "cg_backend_destroy": (None, [_P]),
    "cg_last_error": (C.c_char_p, []),
    "cg_backend_name": (C.c_char_p, [_P]),
    "cg_sync": (_I, [_P]),
    "cg_pool_stats": (_I, [_P, _SZP, _SZP]),
    "cg_pool_trim": (_I, [_P]),
    "cg_profile_enable": (_I, [_P, _I, C.c_uint]),
    "cg_realize": (_I, [_P, _P]),
    "cg_program_stats": (_I, [_P, C.POINTER(C.c_uint64), C.POINTER(C.c_uint64), _I]),
    "cg_profile_read": (_I, [_P, _I, C.POINTER(C.c_uint64), C.POINTER(C.c_double), C.POINTER(C.c_double), _I]),
    "cg_tensor_retain": (None, [_P]),
    "cg_tensor_release": (None, [_P]),
    "cg_tensor_rank": (_SZ, [_P]),
    "cg_tensor_shape": (None, [_P, _SZP]),
    "cg_tensor_dtype": (_I, [_P]),
    "cg_tensor_numel": (_SZ, [_P]),
    "cg_tensor_is_contiguous": (_I, [_P]),
    "cg_zeros": (_I, [_P, _I, _SZP, _SZ, _PP]),
    "cg_from_host": (_I, [_P, _I, _P, _SZ, _SZP, _SZ, _PP]),
    "cg_from_host_bf16_as_f32": (_I, [_P, _P, _SZ, _SZP, _SZ, _PP]),
    "cg_arange": (_I, [_P, _SZ, _PP]),
    "cg_to_host": (_I, [_P, _P, _P, _SZ]),
    "cg_to_bool": (_I, [_P, _P, C.POINTER(_I)]),
    "cg_compare": (_I, [_P, _P, _P, C.POINTER(_I)]),
    "cg_format_tensor": (_I, [_P, _P, C.c_char_p, _SZ]),
    "cg_cast": (_I, [_P, _P, _I, _PP]),
    "cg_unary": (_I, [_P, _I, _P, _PP]),
    "cg_binary": (_I, [_P, _I, _P, _P, _PP]),
    "cg_where": (_I, [_P, _P, _P, _P, _PP]),
    "cg_matmul": (_I, [_P, _P, _P, _PP]),
    "cg_sum": (_I, [_P, _P, _PP]),
    "cg_max": (_I, [_P, _P, _PP]),
    "cg_argmax": (_I, [_P, _P, _PP]),
    "cg_noalloc_setup": (_I, [_I]),
    "cg_argmax_rows_noalloc": (_I, [_I, _I, _P, _SZ, _SZ, _P, _P]),
    "cg_topk": (_I, [_P, _P, _SZ, _PP, _PP]),
    "cg_broadcast": (_I, [_P, _P, _SZP, _SZ, _PP]),
    "cg_reshape": (_I, [_P, _P, _SZP, _SZ, _PP]),
    "cg_transpose": (_I, [_P, _P, _SZ, _SZ, _PP]),
    "cg_slice": (_I, [_P, _P, _SZ, _SZ, _SZ, _PP]),
    "cg_concat": (_I, [_P, _P, _P, _SZ, _PP]),
    "cg_index": (_I, [_P, _P, _SZ, _P, _PP]),
    "cg_block_linear": (_I, [_P, C.POINTER(LinearArgs), _PP]),
    "cg_block_pair_embedding": (_I, [_P, C.POINTER(PairEmbeddingArgs), _PP, _PP]),
    "cg_block_conv_linear": (_I, [_P, C.POINTER(ConvLinearArgs), _PP, _PP, _PP]),
    "cg_block_residual": (_I, [_P, _P, C.POINTER(Branch), _SZ, C.c_float, C.c_float, C.POINTER(Experts), _PP]),
    "cg_block_token_side": (_I, [_P, C.POINTER(TokenSideArgs), _PP]),
    "cg_block_attention": (_I, [_P, C.POINTER(AttentionArgs), _PP, _PP, _PP]),
    "cg_block_channel_delta": (_I, [_P, C.POINTER(ChannelDeltaArgs), _PP, _PP, _PP]),
}


def bind(path: str) -> C.CDLL:
    """dlopen `path` (RTLD_LOCAL) and attach the ABI's signatures.

    Raises AttributeError naming the first missing symbol."""
    lib = C.CDLL(path, mode=C.RTLD_LOCAL)
    for name, (res, args) in SIGNATURES.items():
        fn = getattr(lib, name)
        fn.restype = res
        fn.argtypes = args
    return lib


def dims_array(shape):
    shape = tuple(int(s) for s in shape)
    arr = (C.c_size_t * max(len(shape), 1))(*shape)
    return arr, len(shape)
