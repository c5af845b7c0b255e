"""ctypes binding of the operators in include/vkl_stack.h (libvkllama_hip.so).
The one-token step of such a stack is driven by the C++ model classes."""
import ctypes as C

from . import capi

F32, BF16 = 0, 30
vp, sz, u32, i32, f32 = C.c_void_p, C.c_size_t, C.c_uint32, C.c_int, C.c_float


class OutSeg(C.Structure):
    """vkl_out_seg"""
    _fields_ = [("n0", i32), ("n", i32), ("y", vp), ("ys", sz), ("type", i32), ("act", i32), ("residual", vp),
                ("cap", f32)]


class AttnRowsPrep(C.Structure):
    """vkl_attn_rows_prep"""
    _fields_ = [("H", i32), ("G", i32), ("dim", i32), ("n", i32), ("npair", i32), ("freq", vp), ("eps", f32),
                ("q", vp), ("qs", sz), ("qo", vp), ("qos", sz), ("qtype", i32), ("qotype", i32),
                ("k", vp), ("v", vp), ("kvs", sz), ("kvtype", i32), ("ko", vp), ("vo", vp), ("first", vp), ("fdim", i32), ("mix", f32),
                ("ctype", i32)]


class RecurrenceArgs(C.Structure):
    """vkl_recurrence_args"""
    _fields_ = [("H", i32), ("rep", i32), ("dim", i32), ("vdim", i32), ("q", vp), ("k", vp), ("v", vp), ("type", i32),
                ("qs", sz), ("ks", sz), ("vs", sz), ("qscale", f32), ("log_decay", vp), ("z", vp), ("zs", sz), ("a1", vp), ("a_s", sz),
                ("w_a2", vp), ("r_a", i32), ("b", vp), ("bs", sz), ("dt_bias", vp), ("rate", vp), ("unit_eps", f32), ("state", vp), ("out", vp), ("os", sz)]


RECUR_AUTO, RECUR_TOKENS, RECUR_CHUNKS = 0, 1, 2
ACT_NONE, ACT_SILU, ACT_RELU2, ACT_GELU = 0, 1, 2, 3

SIGNATURES = {
    "vkl_project_bf16w": (i32, [vp, i32, sz, vp, i32, i32, i32, C.POINTER(OutSeg), i32, vp]),
    "vkl_embed_norm_bf16": (i32, [vp, u32, i32, i32, vp, u32, vp, f32, vp, sz, vp]),
    "vkl_rmsnorm_f32": (i32, [vp, sz, vp, i32, i32, vp, f32, vp, i32, sz, i32, vp]),
    "vkl_attn_prefill_causal_bf16": (i32, [vp, vp, vp, i32, i32, i32, i32, i32, sz, sz, sz, f32, f32, i32, vp, sz, vp, sz,
                                           vp]),
    "vkl_attn_rows": (i32, [vp, i32, sz, vp, i32, sz, i32, i32, i32, i32, u32, f32, f32, i32, vp, i32, sz, vp, vp]),
    "vkl_attn_rows_scratch_bytes": (sz, [i32, i32, i32, i32, i32]),
    "vkl_embed_rows_bf16": (i32, [vp, u32, i32, i32, vp, u32, f32, vp, sz, vp]),
    "vkl_attn_prepare": (i32, [C.POINTER(AttnRowsPrep), i32, u32, vp]),
    "vkl_attn_kv_rows": (i32, [vp, i32, sz, vp, vp, i32, sz, i32, i32, i32, i32, u32, f32, i32, i32, vp, i32, sz, vp, vp]),
    "vkl_attn_kv_rows_scratch_bytes": (sz, [i32, i32, i32, i32, i32]),
    "vkl_attn_prefill_chunked_bf16": (i32, [vp, vp, vp, i32, i32, i32, i32, i32, sz, sz, sz, f32, i32, i32, vp, sz, vp]),
    "vkl_short_conv_silu": (i32, [vp, i32, sz, vp, i32, i32, vp, u32, i32, vp, sz, vp]),
    "vkl_recurrence": (i32, [C.POINTER(RecurrenceArgs), i32, u32, i32, vp, sz, vp]),
    "vkl_recurrence_scratch_bytes": (sz, [C.POINTER(RecurrenceArgs), i32]),
    "vkl_recurrence_chunked": (i32, [C.POINTER(RecurrenceArgs), i32]),
    "vkl_low_rank_gated_norm": (i32, [vp, sz, i32, i32, i32, vp, f32, vp, sz, vp, i32, i32, i32, vp, sz, vp]),
    "vkl_gated_norm": (i32, [vp, sz, i32, i32, i32, vp, f32, vp, sz, i32, i32, vp, sz, vp]),
    "vkl_head_matvec": (i32, [vp, i32, i32, i32, vp, i32, sz, sz, vp, i32, sz, sz, vp, sz, i32, vp]),
    "vkl_stack_scratch_bytes": (sz, [vp]),
    "vkl_stack_supported": (i32, [vp]),
    "vkl_stack_step": (i32, [vp, vp, u32, vp, vp, vp]),
    "vkl_stack_loop": (i32, [vp, vp, u32, i32, vp, vp]),
    "vkl_stack_loop_sampled": (i32, [vp, vp, u32, i32, vp, i32, f32, C.c_uint64, vp]),
    "vkl_stack_release": (None, [vp]),
}

_lib = None


def lib():
    global _lib
    if _lib is None:
        capi.lib()
        _lib = capi.load_library(capi.HIP_LIB_PATH, SIGNATURES)
    return _lib


def segments(items):
    """items: (n0, n, y, ys, type, act, residual, cap) each"""
    return (OutSeg * len(items))(*[OutSeg(*it) for it in items])
