"""ctypes binding of the gfx950 kernel library (C ABI: include/nanoflow_kernels.h).

Operands are torch CUDA tensors used purely as device buffers; every call enqueues on
torch's current stream and returns without synchronising.  There is no CPU or PyTorch
fallback: if the compiled library is missing or a call is rejected, an exception is raised.
"""
from __future__ import annotations

import ctypes as C
import os

import torch

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "libnf_kernels.so")

SYMBOLS = [
    "nf_abi_version", "nf_last_error", "nf_embedding_f16", "nf_rmsnorm_f16", "nf_gemm_f16", "nf_gemm_bias_f16",
    "nf_gemm_workspace_bytes", "nf_gemm_workspace_bytes_upto", "nf_gemm_f16_ws", "nf_gemm_bias_f16_ws",
    "nf_dual_swiglu_workspace_bytes", "nf_dual_swiglu_workspace_bytes_upto", "nf_dual_swiglu_f16_ws",
    "nf_dual_swiglu_f16", "nf_gemm_bf16", "nf_dual_swiglu_bf16", "nf_quantize_rows_e4m3", "nf_gemm_f8_f16", "nf_gemm_f8w_workspace_bytes",
    "nf_quantize_weight_e4m3", "nf_dual_swiglu_f8_f16", "nf_dual_swiglu_f8w_f16", "nf_move_kv_pages",
    "nf_gemm_f8w_split_workspace_bytes", "nf_gemm_f8w_split_workspace_bytes_upto",
    "nf_dual_swiglu_f8w_split_workspace_bytes", "nf_dual_swiglu_f8w_split_workspace_bytes_upto",
    "nf_gemm_f8w_f16", "nf_rope_append_f16", "nf_attention_workspace_bytes",
    "nf_attention_paged_f16", "nf_keep_token_f16", "nf_argmax_f16",
    "nf_calibrate_mfma", "nf_calibrate_hbm_read", "nf_calibrate_paged_read",
    "nf_gemm_f16_noalloc", "nf_gemm_noalloc_scratch_bytes",
    "nf_split_kqv_f16", "nf_extract_rank_columns_f16", "nf_silu_mul_f16", "nf_transpose_f16", "nf_sleep_us",
    "nf_gemm_tile_menu", "nf_gemm_tiled_workspace_bytes", "nf_gemm_f16_tiled",
    "nf_rmsnorm_quantize_e4m3", "nf_gemm_f8q_f16", "nf_dual_swiglu_f8q_f16",
    "nf_gemm_nk_workspace_bytes_upto", "nf_gemm_nk_bf16", "nf_gemm_nk_relu2_bf16", "nf_gemm_nk_silu_bf16", "nf_gemm_nk_bias_bf16",
    "nf_gemm_nk_f32", "nf_gemm_nk_sums_shares", "nf_gemm_nk_sums_bytes_upto", "nf_gemm_nk_sums_bf16", "nf_routing_max_tiles", "nf_route", "nf_conv_state", "nf_gemm_nk_gelu_bf16",
    "nf_grouped_tile_rows", "nf_gemm_grouped", "nf_norm_rows", "nf_residual_rows", "nf_token_gate_rows", "nf_gated_norm_rows",
    "nf_embed_rows", "nf_token_shift", "nf_tanh_rows", "nf_argmax_f32", "nf_kv_page_elements", "nf_qkv_append",
    "nf_window_attention", "nf_latent_layout_of", "nf_latent_append", "nf_latent_gather", "nf_latent_pack", "nf_latent_queries", "nf_latent_workspace_bytes", "nf_latent_attention",
    "nf_recurrence_state_elements", "nf_recurrence_workspace_bytes", "nf_linear_recurrence",
]


# structs of the layer-stack operators (nf_rotation, nf_kv_layout, ...)
class Rotation(C.Structure):
    _fields_ = [("table", C.c_void_p), ("dims", C.c_int), ("interleaved", C.c_int)]


class KVLayout(C.Structure):
    _fields_ = [(n, C.c_int) for n in ("dtype", "heads", "kv_heads", "dim", "vdim", "k_pad", "v_pad", "page", "maps")]


class WindowAttentionArgs(C.Structure):
    _fields_ = [("kv", KVLayout), ("window", C.c_int), ("keep_first", C.c_int), ("chunk", C.c_int), ("scale", C.c_float),
                ("out_scale", C.c_float), ("softcap", C.c_float), ("map_weight", C.c_float), ("head_eps", C.c_float),
                ("head_norm", C.c_int), ("sink", C.c_void_p), ("out_rot", Rotation), ("gate", C.c_void_p), ("gate_ld", C.c_int), ("q", C.c_void_p),
                ("out", C.c_void_p), ("out_ld", C.c_int), ("out_col", C.c_int), ("kv_data", C.c_void_p)] + \
        [(n, C.c_void_p) for n in ("input_indptr", "kv_indptr", "kv_indices", "rev_input_indptr", "positions")] + \
        [(n, C.c_int) for n in ("req_begin", "req_num", "row_begin", "max_rows", "decode")]


class QueryTemperature(C.Structure):
    _fields_ = [("coef", C.c_float), ("every", C.c_int)]


class ValueForm(C.Structure):
    _fields_ = [("norm", C.c_int), ("rot", Rotation)]


class ShortConv(C.Structure):
    _fields_ = [("taps", C.c_int)] + [(n, C.c_void_p) for n in ("weight", "state", "input_indptr", "state_slots")]


class LatentLayout(C.Structure):
    _fields_ = [(n, C.c_int) for n in ("dtype", "heads", "kv_rank", "rank_pad", "rot_dim", "row_ld", "page")]


class LatentExpandArgs(C.Structure):
    _fields_ = [("layout", LatentLayout), ("kv", KVLayout), ("dim_pad", C.c_int)] + \
        [(n, C.c_void_p) for n in ("kv_data", "kv_indptr", "kv_indices")] + [(n, C.c_int) for n in ("req_begin", "req_end", "max_pages")] + \
        [(n, C.c_void_p) for n in ("rows", "page_ids", "products")] + [(n, C.c_int) for n in ("ld", "k_col", "v_col")] + [("pages", C.c_void_p)]


class LatentAttentionArgs(C.Structure):
    _fields_ = [("layout", LatentLayout), ("window", C.c_int), ("scale", C.c_float), ("q", C.c_void_p), ("out", C.c_void_p), ("kv_data", C.c_void_p)] + \
        [(n, C.c_void_p) for n in ("input_indptr", "kv_indptr", "kv_indices", "rev_input_indptr", "positions")] + \
        [(n, C.c_int) for n in ("req_begin", "req_num", "row_begin", "max_rows", "decode")] + \
        [("workspace", C.c_void_p), ("workspace_bytes", C.c_size_t)]


class Norm(C.Structure):
    _fields_ = [("kind", C.c_int), ("weight", C.c_void_p), ("bias", C.c_void_p), ("eps", C.c_float)]


class Routing(C.Structure):
    _fields_ = [(n, C.c_void_p) for n in ("choice", "weight", "place", "row_of", "offsets", "tile_group", "tile_row", "n_tiles")] + \
        [("tile_rows", C.c_int), ("row_weight", C.c_void_p)]


class RouteArgs(C.Structure):
    _fields_ = [("z", C.c_void_p)] + \
        [(n, C.c_int) for n in ("shares", "ld", "rows", "outputs", "experts", "top", "always", "groups", "keep_groups")] + \
        [("correction", C.c_void_p), ("scale", C.c_float), ("scores", C.c_int), ("always_plain", C.c_int)]


class GatedAct(C.Structure):
    _fields_ = [("slope", C.c_float), ("shift", C.c_float), ("limits", C.c_void_p)]


class GroupedGemmArgs(C.Structure):
    _fields_ = [(n, C.c_int) for n in ("dtype", "act", "groups", "M", "N", "K")] + \
        [("a", C.c_void_p), ("lda", C.c_int), ("a_group", C.c_size_t), ("b", C.c_void_p), ("d", C.c_void_p), ("ldd", C.c_int),
         ("d_group", C.c_size_t), ("routing", Routing), ("gather", C.c_int), ("max_rows", C.c_int), ("weigh", C.c_int),
         ("gated", GatedAct)]


class ResidualArgs(C.Structure):
    _fields_ = [(n, C.c_int) for n in ("rows", "width", "ld", "y_dtype", "shares")] + \
        [("y", C.c_void_p), ("routing", C.POINTER(Routing)), ("top", C.c_int), ("y_ld", C.c_int), ("identity", C.c_void_p),
         ("y_norm", Norm), ("next", Norm), ("y_scale", C.c_float), ("x", C.c_void_p), ("dtype", C.c_int), ("act", C.c_void_p),
         ("add", C.c_void_p), ("table", C.c_void_p), ("tokens", C.c_void_p), ("table_scale", C.c_float)]


class RecurrenceArgs(C.Structure):
    _fields_ = [(n, C.c_int) for n in ("dtype", "kind", "heads", "dim", "vdim")] + \
        [(n, C.c_void_p) for n in ("q", "k", "v", "g")] + [(n, C.c_int) for n in ("q_ld", "k_ld", "v_ld", "g_ld")] + \
        [("rot", Rotation), ("k_scale", C.c_float), ("log2_decay", C.c_void_p), ("z", C.c_void_p), ("z_ld", C.c_int),
         ("z_shares", C.c_int), ("w0", C.c_void_p), ("u", C.c_void_p), ("norm_weight", C.c_void_p), ("eps", C.c_float),
         ("out_scale", C.c_float), ("state", C.c_void_p), ("out", C.c_void_p), ("out_ld", C.c_int), ("out_col", C.c_int),
         ("shift_x", C.c_void_p), ("shift_state", C.c_void_p), ("shift_ld", C.c_int), ("input_indptr", C.c_void_p),
         ("positions", C.c_void_p), ("state_slots", C.c_void_p)] + \
        [(n, C.c_int) for n in ("req_begin", "req_num", "row_begin", "rows", "total_rows")] + \
        [("workspace", C.c_void_p), ("workspace_bytes", C.c_size_t)]


class NanoflowKernelError(RuntimeError):
    pass


_lib = None


def lib() -> C.CDLL:
    """Loads libnf_kernels.so (built by ``make -C nanoflow_amd/csrc`` / ``__graft_entry__.build``)."""
    global _lib
    if _lib is None:
        if not os.path.exists(LIB_PATH):
            raise NanoflowKernelError(
                f"{LIB_PATH} is missing: build it with `make -C nanoflow_amd/csrc` "
                "(there is no fallback path)")
        l = C.CDLL(LIB_PATH)
        vp, i32, f32, sz = C.c_void_p, C.c_int, C.c_float, C.c_size_t
        l.nf_abi_version.restype = i32
        l.nf_last_error.restype = C.c_char_p
        l.nf_embedding_f16.argtypes = [vp, vp, vp, i32, i32, vp]
        l.nf_rmsnorm_f16.argtypes = [vp, vp, vp, i32, i32, f32, vp]
        l.nf_gemm_f16.argtypes = [vp, vp, vp, vp, i32, i32, i32, f32, f32, i32, vp]
        l.nf_gemm_workspace_bytes.restype = sz
        l.nf_gemm_workspace_bytes.argtypes = [i32, i32, i32]
        l.nf_gemm_workspace_bytes_upto.restype = sz
        l.nf_gemm_workspace_bytes_upto.argtypes = [i32, i32, i32]
        l.nf_gemm_f16_ws.argtypes = [vp, vp, vp, vp, i32, i32, i32, f32, f32, i32, vp, sz, vp]
        l.nf_dual_swiglu_workspace_bytes.restype = sz
        l.nf_dual_swiglu_workspace_bytes.argtypes = [i32, i32, i32]
        l.nf_dual_swiglu_workspace_bytes_upto.restype = sz
        l.nf_dual_swiglu_workspace_bytes_upto.argtypes = [i32, i32, i32]
        l.nf_dual_swiglu_f16_ws.argtypes = [vp, vp, vp, vp, i32, i32, i32, i32, vp, sz, vp]
        l.nf_gemm_bias_f16_ws.argtypes = [vp, vp, vp, vp, i32, i32, i32, f32, f32, i32, vp, sz, vp]
        l.nf_gemm_bias_f16.argtypes = [vp, vp, vp, vp, i32, i32, i32, f32, f32, i32, vp]
        l.nf_dual_swiglu_f16.argtypes = [vp, vp, vp, vp, i32, i32, i32, i32, vp]
        l.nf_gemm_bf16.argtypes = [vp, vp, vp, vp, i32, i32, i32, f32, f32, i32, vp]
        l.nf_dual_swiglu_bf16.argtypes = [vp, vp, vp, vp, i32, i32, i32, vp]
        l.nf_quantize_rows_e4m3.argtypes = [vp, vp, vp, i32, i32, vp]
        l.nf_gemm_f8_f16.argtypes = [vp, vp, vp, vp, vp, vp, i32, i32, i32, f32, f32, vp]
        l.nf_gemm_f8w_workspace_bytes.restype = C.c_size_t
        l.nf_gemm_f8w_workspace_bytes.argtypes = [i32, i32]
        l.nf_gemm_f8w_f16.argtypes = [vp, vp, vp, vp, vp, i32, i32, i32, f32, f32, vp, C.c_size_t, vp]
        for name in ("nf_gemm_f8w_split_workspace_bytes", "nf_gemm_f8w_split_workspace_bytes_upto",
                     "nf_dual_swiglu_f8w_split_workspace_bytes", "nf_dual_swiglu_f8w_split_workspace_bytes_upto"):
            getattr(l, name).restype = sz
            getattr(l, name).argtypes = [i32, i32, i32]
        l.nf_quantize_weight_e4m3.argtypes = [vp, vp, vp, i32, i32, vp]
        l.nf_rmsnorm_quantize_e4m3.argtypes = [vp, vp, vp, vp, vp, i32, i32, f32, vp]
        l.nf_gemm_f8q_f16.argtypes = [vp, vp, vp, vp, vp, vp, i32, i32, i32, f32, f32, vp, C.c_size_t, vp]
        l.nf_dual_swiglu_f8q_f16.argtypes = [vp, vp, vp, vp, vp, vp, vp, i32, i32, i32, vp, C.c_size_t, vp]
        l.nf_dual_swiglu_f8_f16.argtypes = [vp, vp, vp, vp, vp, vp, vp, i32, i32, i32, vp]
        l.nf_dual_swiglu_f8w_f16.argtypes = [vp, vp, vp, vp, vp, vp, i32, i32, i32, vp, C.c_size_t, vp]
        l.nf_move_kv_pages.argtypes = [i32, vp, vp, vp, vp, vp, sz, i32, vp]
        l.nf_rope_append_f16.argtypes = [vp] * 7 + [i32] * 5 + [f32] * 4 + [vp]
        l.nf_gemm_f16_noalloc.argtypes = [vp, vp, vp, vp, i32, i32, i32, f32, f32, i32, vp]
        l.nf_gemm_noalloc_scratch_bytes.restype = sz
        l.nf_gemm_noalloc_scratch_bytes.argtypes = []
        l.nf_split_kqv_f16.argtypes = [vp, vp, vp, vp, i32, i32, i32, i32, vp]
        l.nf_extract_rank_columns_f16.argtypes = [vp, vp, i32, i32, i32, i32, vp]
        l.nf_silu_mul_f16.argtypes = [vp, vp, i32, i32, vp]
        l.nf_transpose_f16.argtypes = [vp, vp, i32, i32, vp]
        l.nf_sleep_us.argtypes = [i32, vp]
        ip = C.POINTER(C.c_int)
        l.nf_gemm_tile_menu.argtypes = [i32, ip, ip, ip]
        l.nf_gemm_tiled_workspace_bytes.restype = sz
        l.nf_gemm_tiled_workspace_bytes.argtypes = [i32, i32, i32, i32]
        l.nf_gemm_f16_tiled.argtypes = [vp, vp, vp, vp, i32, i32, i32, f32, f32, i32, i32, i32, i32, i32, vp, sz, vp]
        dp = C.POINTER(C.c_double)
        l.nf_calibrate_mfma.argtypes = [i32, i32, i32, vp, sz, dp, dp, vp]
        l.nf_calibrate_hbm_read.argtypes = [vp, sz, i32, vp, sz, dp, vp]
        l.nf_calibrate_paged_read.argtypes = [vp, vp, vp, vp, i32, i32, sz, i32, vp, sz, dp, vp]
        l.nf_attention_workspace_bytes.restype = sz
        l.nf_attention_workspace_bytes.argtypes = [i32, i32, i32]
        l.nf_attention_paged_f16.argtypes = [vp] * 7 + [i32] * 8 + [vp, sz, vp]
        l.nf_keep_token_f16.argtypes = [vp, vp, vp, i32, i32, vp]
        l.nf_argmax_f16.argtypes = [vp, vp, vp, i32, i32, vp]
        for name in ("nf_gemm_nk_bf16", "nf_gemm_nk_relu2_bf16", "nf_gemm_nk_silu_bf16", "nf_gemm_nk_gelu_bf16"):
            getattr(l, name).argtypes = [vp, vp, vp, i32, i32, i32, vp, sz, vp]
        l.nf_gemm_nk_bias_bf16.argtypes = [vp, vp, vp, vp, i32, i32, i32, vp, sz, vp]
        l.nf_gemm_nk_f32.argtypes = [vp, vp, vp, vp, i32, i32, i32, i32, vp]
        l.nf_routing_max_tiles.argtypes = l.nf_grouped_tile_rows.argtypes = [i32] * 3
        l.nf_route.argtypes = [vp, vp, vp]
        l.nf_conv_state.argtypes = [i32, vp, i32, vp, vp, i32, i32, vp]
        l.nf_gemm_grouped.argtypes = l.nf_residual_rows.argtypes = l.nf_latent_attention.argtypes = [vp, vp]
        l.nf_norm_rows.argtypes = [i32, vp, vp, vp, vp, i32, i32, i32, vp]
        l.nf_token_gate_rows.argtypes = [i32, vp, i32, vp, vp, i32, i32, i32, vp, i32, i32, vp]
        l.nf_gated_norm_rows.argtypes = [i32, vp, i32, vp, i32, vp, i32, i32, f32, vp]
        l.nf_latent_gather.argtypes = l.nf_latent_pack.argtypes = [vp, vp]
        l.nf_latent_queries.argtypes = [vp, i32, vp, i32, i32, i32, vp, vp, vp, i32, i32, vp]
        l.nf_latent_layout_of.argtypes = [i32] * 5 + [vp]
        l.nf_latent_append.argtypes = [vp, vp, i32, i32, i32, vp, f32] + [vp] * 7 + [i32, i32, vp]
        l.nf_gemm_nk_sums_shares.argtypes = [i32] * 4
        l.nf_gemm_nk_sums_bf16.argtypes = [vp, vp, vp, sz, i32, i32, i32, i32, vp]
        l.nf_embed_rows.argtypes = [i32, vp, vp, vp, vp, f32, vp, vp, i32, i32, vp]
        l.nf_token_shift.argtypes = [i32, vp, vp, vp, vp, i32, vp, vp, vp, vp, i32, i32, vp]
        l.nf_tanh_rows.argtypes = [i32, vp, i32, vp, i32, i32, vp]
        l.nf_argmax_f32.argtypes = [vp, vp, i32, i32, i32, vp]
        l.nf_qkv_append.argtypes = [C.POINTER(KVLayout), vp, i32, i32, i32, i32, vp, vp, f32, C.POINTER(Rotation), vp, vp, vp, vp, vp,
                                    vp, vp, vp, vp, i32, vp]
        l.nf_window_attention.argtypes = [C.POINTER(WindowAttentionArgs), vp]
        l.nf_linear_recurrence.argtypes = [C.POINTER(RecurrenceArgs), vp]
        size_calls = {"nf_kv_page_elements": [C.POINTER(KVLayout)], "nf_recurrence_state_elements": [i32, i32],
                      "nf_recurrence_workspace_bytes": [i32] * 5, "nf_gemm_nk_workspace_bytes_upto": [i32] * 3,
                      "nf_gemm_nk_sums_bytes_upto": [i32] * 4, "nf_latent_workspace_bytes": [vp, i32]}
        for name, types in size_calls.items():
            getattr(l, name).restype = sz
            getattr(l, name).argtypes = types
        for name in SYMBOLS:
            if name not in size_calls and name not in ("nf_last_error", "nf_attention_workspace_bytes", "nf_gemm_workspace_bytes",
                            "nf_gemm_workspace_bytes_upto", "nf_gemm_f8w_workspace_bytes", "nf_gemm_tiled_workspace_bytes",
                            "nf_dual_swiglu_workspace_bytes", "nf_dual_swiglu_workspace_bytes_upto",
                            "nf_gemm_f8w_split_workspace_bytes", "nf_gemm_f8w_split_workspace_bytes_upto",
                            "nf_dual_swiglu_f8w_split_workspace_bytes", "nf_dual_swiglu_f8w_split_workspace_bytes_upto"):
                getattr(l, name).restype = i32
        _lib = l
    return _lib


def _check(rc: int, what: str):
    if rc != 0:
        raise NanoflowKernelError(f"{what} failed ({rc}): {lib().nf_last_error().decode()}")


def _p(t):
    if t is None:
        return None
    assert t.is_cuda and t.is_contiguous(), "device-resident contiguous tensor required"
    return t.data_ptr()


def _stream():
    return torch.cuda.current_stream().cuda_stream


def _f16(t):
    assert t.dtype == torch.float16, t.dtype


def _i32(t):
    assert t.dtype == torch.int32, t.dtype


def embedding(tokens, table, out=None):
    _i32(tokens); _f16(table)
    T, H = tokens.numel(), table.shape[1]
    out = torch.empty((T, H), dtype=torch.float16, device=table.device) if out is None else out
    _check(lib().nf_embedding_f16(_p(tokens), _p(table), _p(out), T, H, _stream()), "nf_embedding_f16")
    return out


def rmsnorm(x, w, eps=1e-5, out=None):
    _f16(x); _f16(w)
    rows, H = x.shape
    out = torch.empty_like(x) if out is None else out
    _check(lib().nf_rmsnorm_f16(_p(out), _p(x), _p(w), rows, H, eps, _stream()), "nf_rmsnorm_f16")
    return out


def rmsnorm_quantize_e4m3(x, w, eps=1e-5):
    """(fp16 RMSNorm output, its e4m3 bytes, fp32 row scales) from one launch."""
    _f16(x); _f16(w)
    rows, H = x.shape
    out = torch.empty_like(x)
    q = torch.empty((rows, H), dtype=torch.uint8, device=x.device)
    scale = torch.empty((rows,), dtype=torch.float32, device=x.device)
    _check(lib().nf_rmsnorm_quantize_e4m3(_p(out), _p(x), _p(w), _p(q), _p(scale), rows, H, eps, _stream()),
           "nf_rmsnorm_quantize_e4m3")
    return out, q, scale


def _elem(t, dtype):
    assert t.is_cuda and t.dtype == dtype and t.is_contiguous(), (t.dtype, t.device)


def gemm(A, B, Cmat=None, alpha=1.0, beta=0.0, b_col_major=False, out=None, bias=None):
    """fp16 operands run nf_gemm_f16, bfloat16 operands nf_gemm_bf16 (same kernels, other element type).
    bias [N] (fp16 only, instead of Cmat): beta * bias is added to every row (nf_gemm_bias_f16)."""
    dt = A.dtype
    assert dt in (torch.float16, torch.bfloat16), dt
    _elem(A, dt); _elem(B, dt)
    M, K = A.shape
    N = B.shape[0] if b_col_major else B.shape[1]
    assert tuple(B.shape) == ((N, K) if b_col_major else (K, N)), (A.shape, B.shape)
    if bias is not None:
        assert Cmat is None and dt == torch.float16 and bias.numel() == N
        _elem(bias, dt)
        out = torch.empty((M, N), dtype=dt, device=A.device) if out is None else out
        _elem(out, dt)
        _check(lib().nf_gemm_bias_f16(_p(A), _p(B), _p(bias), _p(out), M, N, K, alpha, beta, int(b_col_major),
                                      _stream()), "nf_gemm_bias_f16")
        return out
    if Cmat is not None:
        _elem(Cmat, dt)
        assert tuple(Cmat.shape) == (M, N)
    out = torch.empty((M, N), dtype=dt, device=A.device) if out is None else out
    _elem(out, dt)
    fn, name = (lib().nf_gemm_f16, "nf_gemm_f16") if dt == torch.float16 else (lib().nf_gemm_bf16, "nf_gemm_bf16")
    _check(fn(_p(A), _p(B), _p(Cmat), _p(out), M, N, K, alpha, beta, int(b_col_major), _stream()), name)
    return out


def gemm_ws(A, B, Cmat=None, alpha=1.0, beta=0.0, b_col_major=False, out=None, workspace=None, bias=None):
    """nf_gemm_f16_ws: fp16 GEMM that is split over K through a workspace when few rows against a narrow
    N would leave most of the chip idle.  Returns (out, shares_bytes) where shares_bytes is the
    workspace the shape asked for (0: not split)."""
    _f16(A); _f16(B)
    M, K = A.shape
    N = B.shape[0] if b_col_major else B.shape[1]
    assert tuple(B.shape) == ((N, K) if b_col_major else (K, N)), (A.shape, B.shape)
    if Cmat is not None:
        _f16(Cmat)
        assert tuple(Cmat.shape) == (M, N)
    need = lib().nf_gemm_workspace_bytes(M, N, K)
    if workspace is None:
        workspace = torch.empty((max(need, 16),), dtype=torch.uint8, device=A.device)
    out = torch.empty((M, N), dtype=torch.float16, device=A.device) if out is None else out
    if bias is not None:          # one row [N] added (times beta) to every row: nf_gemm_bias_f16_ws
        assert Cmat is None and bias.numel() == N
        _f16(bias)
        _check(lib().nf_gemm_bias_f16_ws(_p(A), _p(B), _p(bias), _p(out), M, N, K, alpha, beta, int(b_col_major),
                                         _p(workspace), workspace.numel(), _stream()), "nf_gemm_bias_f16_ws")
        return out, need
    _check(lib().nf_gemm_f16_ws(_p(A), _p(B), _p(Cmat), _p(out), M, N, K, alpha, beta, int(b_col_major),
                                _p(workspace), workspace.numel(), _stream()), "nf_gemm_f16_ws")
    return out, need


def gemm_tile_menu():
    """[(tile_m, tile_n, takes k-contiguous weights only)] of the tiles nf_gemm_f16_tiled chooses from."""
    m, n, c = C.c_int(), C.c_int(), C.c_int()
    out = []
    for i in range(lib().nf_gemm_tile_menu(-1, None, None, None)):
        lib().nf_gemm_tile_menu(i, C.byref(m), C.byref(n), C.byref(c))
        out.append((m.value, n.value, bool(c.value)))
    return out


def gemm_tiled(A, B, tile, split_k=1, Cmat=None, alpha=1.0, beta=0.0, b_col_major=False, out=None, bias=None,
               workspace=None):
    """nf_gemm_f16_tiled: the GEMM on the menu tile closest to ``tile`` = (m, n), K cut into ``split_k`` shares."""
    _f16(A); _f16(B)
    M, K = A.shape
    N = B.shape[0] if b_col_major else B.shape[1]
    assert tuple(B.shape) == ((N, K) if b_col_major else (K, N))
    need = lib().nf_gemm_tiled_workspace_bytes(M, N, K, split_k)
    if workspace is None:
        workspace = torch.empty((max(need, 16),), dtype=torch.uint8, device=A.device)
    out = torch.empty((M, N), dtype=torch.float16, device=A.device) if out is None else out
    c = bias if bias is not None else Cmat
    _check(lib().nf_gemm_f16_tiled(_p(A), _p(B), _p(c), _p(out), M, N, K, alpha, beta, int(b_col_major),
                                   int(bias is not None), tile[0], tile[1], split_k, _p(workspace), workspace.numel(),
                                   _stream()), "nf_gemm_f16_tiled")
    return out


def dual_swiglu_ws(A, Bg, Bu, out=None, workspace=None, b_col_major=False):
    """nf_dual_swiglu_f16_ws; returns (out, bytes of workspace the shape asks for: 0 = not split).
    b_col_major: Bg / Bu are [N, K] (k contiguous) instead of [K, N]."""
    _f16(A); _f16(Bg); _f16(Bu)
    M, K = A.shape
    N = Bg.shape[0] if b_col_major else Bg.shape[1]
    assert tuple(Bg.shape) == ((N, K) if b_col_major else (K, N)) and Bu.shape == Bg.shape
    need = lib().nf_dual_swiglu_workspace_bytes(M, N, K)
    if workspace is None:
        workspace = torch.empty((max(need, 16),), dtype=torch.uint8, device=A.device)
    out = torch.empty((M, N), dtype=torch.float16, device=A.device) if out is None else out
    _check(lib().nf_dual_swiglu_f16_ws(_p(A), _p(Bg), _p(Bu), _p(out), M, N, K, int(b_col_major), _p(workspace),
                                       workspace.numel(), _stream()), "nf_dual_swiglu_f16_ws")
    return out, need


def dual_swiglu(A, Bg, Bu, out=None, b_col_major=False):
    """b_col_major (fp16 only): Bg / Bu are [N, K] (k contiguous) instead of [K, N]."""
    dt = A.dtype
    assert dt in (torch.float16, torch.bfloat16), dt
    _elem(A, dt); _elem(Bg, dt); _elem(Bu, dt)
    M, K = A.shape
    N = Bg.shape[0] if b_col_major else Bg.shape[1]
    assert tuple(Bg.shape) == ((N, K) if b_col_major else (K, N)) and Bu.shape == Bg.shape
    out = torch.empty((M, N), dtype=dt, device=A.device) if out is None else out
    _elem(out, dt)
    if dt == torch.float16:
        _check(lib().nf_dual_swiglu_f16(_p(A), _p(Bg), _p(Bu), _p(out), M, N, K, int(b_col_major), _stream()),
               "nf_dual_swiglu_f16")
    else:
        assert not b_col_major, "the bf16 pair takes [K, N] weights only"
        _check(lib().nf_dual_swiglu_bf16(_p(A), _p(Bg), _p(Bu), _p(out), M, N, K, _stream()), "nf_dual_swiglu_bf16")
    return out


def quantize_rows_e4m3(X):
    """fp16 [M,K] -> (e4m3 bytes [M,K], fp32 row scales [M])."""
    _f16(X)
    M, K = X.shape
    Xq = torch.empty((M, K), dtype=torch.uint8, device=X.device)
    scale = torch.empty((M,), dtype=torch.float32, device=X.device)
    _check(lib().nf_quantize_rows_e4m3(_p(X), _p(Xq), _p(scale), M, K, _stream()), "nf_quantize_rows_e4m3")
    return Xq, scale


def gemm_f8(Aq, a_scale, Bq_nk, b_scale, Cmat=None, alpha=1.0, beta=0.0, out=None):
    """Aq e4m3 bytes [M,K], Bq_nk e4m3 bytes [N,K] (one row per output channel)."""
    assert Aq.dtype == torch.uint8 and Bq_nk.dtype == torch.uint8
    assert a_scale.dtype == torch.float32 and b_scale.dtype == torch.float32
    M, K = Aq.shape
    N = Bq_nk.shape[0]
    assert tuple(Bq_nk.shape) == (N, K) and a_scale.numel() == M and b_scale.numel() == N
    assert Aq.is_contiguous() and Bq_nk.is_contiguous()
    out = torch.empty((M, N), dtype=torch.float16, device=Aq.device) if out is None else out
    _check(lib().nf_gemm_f8_f16(_p(Aq), _p(a_scale), _p(Bq_nk), _p(b_scale), _p(Cmat), _p(out), M, N, K,
                                alpha, beta, _stream()), "nf_gemm_f8_f16")
    return out


def gemm_f8w(A, Bq_nk, b_scale, Cmat=None, alpha=1.0, beta=0.0, out=None, workspace=None):
    """fp16 activations [M,K] against e4m3 weights [N,K] with per-output-channel scales."""
    _f16(A)
    assert Bq_nk.dtype == torch.uint8 and b_scale.dtype == torch.float32 and Bq_nk.is_contiguous()
    M, K = A.shape
    N = Bq_nk.shape[0]
    assert tuple(Bq_nk.shape) == (N, K) and b_scale.numel() == N
    need = lib().nf_gemm_f8w_split_workspace_bytes(M, N, K)      # quantised rows (+ the sums of a split over K)
    if workspace is None:
        workspace = torch.empty((max(need, 16),), dtype=torch.uint8, device=A.device)
    out = torch.empty((M, N), dtype=torch.float16, device=A.device) if out is None else out
    _check(lib().nf_gemm_f8w_f16(_p(A), _p(Bq_nk), _p(b_scale), _p(Cmat), _p(out), M, N, K, alpha, beta,
                                 _p(workspace), workspace.numel() * workspace.element_size(), _stream()),
           "nf_gemm_f8w_f16")
    return out


def gemm_f8q(Aq, a_scale, Bq_nk, b_scale, Cmat=None, alpha=1.0, beta=0.0, out=None, workspace=None):
    """nf_gemm_f8w_f16 on rows that are quantised already; the workspace only holds the sums of a split over K."""
    M, K = Aq.shape
    N = Bq_nk.shape[0]
    need = lib().nf_gemm_f8w_split_workspace_bytes(M, N, K)
    if workspace is None:
        workspace = torch.empty((max(need, 16),), dtype=torch.uint8, device=Aq.device)
    out = torch.empty((M, N), dtype=torch.float16, device=Aq.device) if out is None else out
    _check(lib().nf_gemm_f8q_f16(_p(Aq), _p(a_scale), _p(Bq_nk), _p(b_scale), _p(Cmat), _p(out), M, N, K, alpha, beta,
                                 _p(workspace), workspace.numel(), _stream()), "nf_gemm_f8q_f16")
    return out


def dual_swiglu_f8q(Aq, a_scale, Gq, g_scale, Uq, u_scale, out=None, workspace=None):
    M, Kd = Aq.shape
    N = Gq.shape[0]
    need = lib().nf_dual_swiglu_f8w_split_workspace_bytes(M, N, Kd)
    if workspace is None:
        workspace = torch.empty((max(need, 16),), dtype=torch.uint8, device=Aq.device)
    out = torch.empty((M, N), dtype=torch.float16, device=Aq.device) if out is None else out
    _check(lib().nf_dual_swiglu_f8q_f16(_p(Aq), _p(a_scale), _p(Gq), _p(g_scale), _p(Uq), _p(u_scale), _p(out), M, N,
                                        Kd, _p(workspace), workspace.numel(), _stream()), "nf_dual_swiglu_f8q_f16")
    return out


def quantize_weight_e4m3(W):
    """W fp16 [K,N] (the pipeline's weight orientation) -> (Wq e4m3 bytes [N,K], col_scale fp32 [N])."""
    _f16(W)
    Kd, N = W.shape
    Wq = torch.empty((N, Kd), dtype=torch.uint8, device=W.device)
    scale = torch.empty((N,), dtype=torch.float32, device=W.device)
    _check(lib().nf_quantize_weight_e4m3(_p(W), _p(Wq), _p(scale), Kd, N, _stream()), "nf_quantize_weight_e4m3")
    return Wq, scale


def dual_swiglu_f8(Aq, a_scale, Gq, g_scale, Uq, u_scale, out=None):
    assert Aq.dtype == torch.uint8 and Gq.dtype == torch.uint8 and Uq.dtype == torch.uint8
    M, Kd = Aq.shape
    N = Gq.shape[0]
    assert tuple(Gq.shape) == (N, Kd) and tuple(Uq.shape) == (N, Kd)
    assert a_scale.numel() == M and g_scale.numel() == N and u_scale.numel() == N
    out = torch.empty((M, N), dtype=torch.float16, device=Aq.device) if out is None else out
    _check(lib().nf_dual_swiglu_f8_f16(_p(Aq), _p(a_scale), _p(Gq), _p(g_scale), _p(Uq), _p(u_scale), _p(out),
                                       M, N, Kd, _stream()), "nf_dual_swiglu_f8_f16")
    return out


def dual_swiglu_f8w(A, Gq, g_scale, Uq, u_scale, out=None, workspace=None):
    """fp16 activations [M,K] against e4m3 gate/up weights [N,K] with per-output-channel scales."""
    _f16(A)
    M, Kd = A.shape
    N = Gq.shape[0]
    assert tuple(Gq.shape) == (N, Kd) and tuple(Uq.shape) == (N, Kd)
    need = lib().nf_dual_swiglu_f8w_split_workspace_bytes(M, N, Kd)
    if workspace is None:
        workspace = torch.empty((max(need, 16),), dtype=torch.uint8, device=A.device)
    out = torch.empty((M, N), dtype=torch.float16, device=A.device) if out is None else out
    _check(lib().nf_dual_swiglu_f8w_f16(_p(A), _p(Gq), _p(g_scale), _p(Uq), _p(u_scale), _p(out), M, N, Kd,
                                        _p(workspace), workspace.numel() * workspace.element_size(), _stream()),
           "nf_dual_swiglu_f8w_f16")
    return out


def rope_append(kqv, kv_data, kv_indices, kv_indptr, rev_input_indptr, per_token_offset, Hq, Hkv,
                d=128, page_size=16, rope_scale=1.0, rope_theta=1e4, smooth_a=0.0, smooth_b=0.0,
                q_out=None, n_tokens=None):
    """Appends K/V into kv_data IN PLACE and returns the rotated Q rows."""
    _f16(kqv); _f16(kv_data)
    for t in (kv_indices, kv_indptr, rev_input_indptr, per_token_offset):
        _i32(t)
    T = kqv.shape[0] if n_tokens is None else n_tokens
    assert kqv.shape[1] == (Hq + 2 * Hkv) * d
    q_out = torch.empty((kqv.shape[0], Hq * d), dtype=torch.float16, device=kqv.device) \
        if q_out is None else q_out
    _check(lib().nf_rope_append_f16(_p(kqv), _p(q_out), _p(kv_data), _p(kv_indices), _p(kv_indptr),
                                    _p(rev_input_indptr), _p(per_token_offset), T, Hq, Hkv, d,
                                    page_size, rope_scale, rope_theta, smooth_a, smooth_b, _stream()),
           "nf_rope_append_f16")
    return q_out


def attention_paged(q, qo_indptr, kv_data, kv_indptr, kv_indices, kv_last_page_len, Hq, Hkv, d=128,
                    page_size=16, causal=False, out=None, batch=None, max_qo_rows=None,
                    num_blocks=0, workspace=None):
    _f16(q); _f16(kv_data)
    for t in (qo_indptr, kv_indptr, kv_indices, kv_last_page_len):
        _i32(t)
    batch = kv_last_page_len.numel() if batch is None else batch
    max_qo_rows = q.shape[0] if max_qo_rows is None else max_qo_rows
    out = torch.zeros_like(q) if out is None else out
    need = lib().nf_attention_workspace_bytes(batch, max_qo_rows, Hq)
    if workspace is None:
        workspace = torch.empty((max(need, 1),), dtype=torch.uint8, device=q.device)
    _check(lib().nf_attention_paged_f16(_p(q), _p(out), _p(qo_indptr), _p(kv_data), _p(kv_indptr),
                                        _p(kv_indices), _p(kv_last_page_len), batch, max_qo_rows,
                                        Hq, Hkv, d, page_size, int(bool(causal)), num_blocks,
                                        _p(workspace), workspace.numel(), _stream()),
           "nf_attention_paged_f16")
    return out


def move_kv_pages(req_idx, kv_indptr, kv_indices, staging, kv_data, to_pool: bool):
    """Pages of the requests in req_idx between one layer's pool kv_data [pages, 2, page, Hkv, d] and
    staging [len(kv_indices), 2, page, Hkv, d] (page j of staging <-> pool page kv_indices[j])."""
    for t in (req_idx, kv_indptr, kv_indices):
        _i32(t)
    _f16(staging); _f16(kv_data)
    page_bytes = kv_data[0].numel() * 2
    assert staging[0].numel() * 2 == page_bytes and staging.shape[0] >= kv_indices.numel()
    _check(lib().nf_move_kv_pages(req_idx.numel(), _p(req_idx), _p(kv_indptr), _p(kv_indices), _p(staging),
                                  _p(kv_data), page_bytes, int(bool(to_pool)), _stream()), "nf_move_kv_pages")


def split_kqv(kqv, k_dim, q_dim, v_dim):
    """(k, q, v): the three column ranges of kqv [rows, k_dim + q_dim + v_dim], in that order."""
    _f16(kqv)
    rows = kqv.shape[0]
    assert kqv.shape[1] == k_dim + q_dim + v_dim
    outs = [torch.empty((rows, d), dtype=torch.float16, device=kqv.device) for d in (k_dim, q_dim, v_dim)]
    _check(lib().nf_split_kqv_f16(_p(kqv), *[_p(o) if o.numel() else None for o in outs], rows, k_dim, q_dim, v_dim,
                                  _stream()), "nf_split_kqv_f16")
    return tuple(outs)


def extract_rank_columns(x, nranks, rank):
    _f16(x)
    rows, cols = x.shape[0], x.shape[1] // nranks
    assert x.shape[1] == nranks * cols
    out = torch.empty((rows, cols), dtype=torch.float16, device=x.device)
    _check(lib().nf_extract_rank_columns_f16(_p(x), _p(out), rows, cols, nranks, rank, _stream()),
           "nf_extract_rank_columns_f16")
    return out


def silu_mul(x):
    """[rows, 2 * cols] -> [rows, cols]: x[:, :cols] * silu(x[:, cols:])."""
    _f16(x)
    rows, cols = x.shape[0], x.shape[1] // 2
    assert x.shape[1] == 2 * cols
    out = torch.empty((rows, cols), dtype=torch.float16, device=x.device)
    _check(lib().nf_silu_mul_f16(_p(x), _p(out), rows, cols, _stream()), "nf_silu_mul_f16")
    return out


def transpose(x):
    _f16(x)
    rows, cols = x.shape
    out = torch.empty((cols, rows), dtype=torch.float16, device=x.device)
    _check(lib().nf_transpose_f16(_p(x), _p(out), rows, cols, _stream()), "nf_transpose_f16")
    return out


def sleep_us(us):
    _check(lib().nf_sleep_us(int(us), _stream()), "nf_sleep_us")


def keep_token(x, input_indptr, req_num, out=None):
    _f16(x); _i32(input_indptr)
    H = x.shape[1]
    out = torch.empty((req_num, H), dtype=torch.float16, device=x.device) if out is None else out
    _check(lib().nf_keep_token_f16(_p(x), _p(out), _p(input_indptr), req_num, H, _stream()),
           "nf_keep_token_f16")
    return out


def argmax(logits, rows=None):
    _f16(logits)
    rows = logits.shape[0] if rows is None else rows
    cols = logits.shape[1]
    mv = torch.empty((rows,), dtype=torch.float16, device=logits.device)
    arg = torch.empty((rows,), dtype=torch.int32, device=logits.device)
    _check(lib().nf_argmax_f16(_p(logits), _p(mv), _p(arg), rows, cols, _stream()), "nf_argmax_f16")
    return arg, mv


# ---------------------------------------------------------------- calibration micro-benchmarks

def calibrate_mfma(fp8: bool = False, random_operands=True, iters: int = 20000):
    """(TFLOP/s, shader clock in MHz) of an MFMA loop on this device.  random_operands: False = zero
    operands in registers, True = pseudo-random ones, 2 = pseudo-random ones re-read from LDS before
    every 16 MFMAs (fp16 only), as a GEMM's main loop reads its fragments, 3 = with the operand loads
    of a 256x256 tile (L2 -> LDS) beside them as well, 4 = as True with 16x16 MFMAs."""
    scratch = torch.zeros(8192 + ((8 << 20) if int(random_operands) == 3 else 0), dtype=torch.uint8, device="cuda")
    tf, mhz = C.c_double(), C.c_double()
    _check(lib().nf_calibrate_mfma(int(fp8), int(random_operands), iters, scratch.data_ptr(), scratch.numel(),
                                   C.byref(tf), C.byref(mhz), _stream()), "nf_calibrate_mfma")
    return tf.value, mhz.value


def calibrate_hbm_read(gib: float = 8.0, reps: int = 4) -> float:
    """GB/s of all CUs streaming a buffer of `gib` GiB (freed again before returning)."""
    n = int(gib * (1 << 30)) // 16 * 16
    buf = torch.empty(n, dtype=torch.uint8, device="cuda")
    buf.random_()   # touched: every page is backed
    scratch = torch.zeros(8192, dtype=torch.uint8, device="cuda")
    g = C.c_double()
    _check(lib().nf_calibrate_hbm_read(buf.data_ptr(), n, reps, scratch.data_ptr(), scratch.numel(), C.byref(g), _stream()),
           "nf_calibrate_hbm_read")
    del buf
    torch.cuda.empty_cache()
    return g.value


def calibrate_paged_read(pool, kv_indptr, kv_indices, kv_last_page_len, batch: int, num_kv_heads: int,
                         kv_bytes: int, reps: int = 10) -> float:
    """GB/s of paged decode attention's load pattern with the arithmetic removed."""
    scratch = torch.zeros(8192, dtype=torch.uint8, device="cuda")
    g = C.c_double()
    _check(lib().nf_calibrate_paged_read(pool.data_ptr(), kv_indptr.data_ptr(), kv_indices.data_ptr(),
                                         kv_last_page_len.data_ptr(), batch, num_kv_heads, kv_bytes, reps,
                                         scratch.data_ptr(), scratch.numel(), C.byref(g), _stream()), "nf_calibrate_paged_read")
    return g.value


# ---------------------------------------------------------------- layer-stack operators
# Activations are float32 or bfloat16 tensors (the operators' dtype follows them); see the C header for
# the layouts.

F32, BF16 = 0, 1
FIXED_DECAY, TOKEN_DECAY = 0, 1


def _dt(t):
    return {torch.float32: F32, torch.bfloat16: BF16}[t.dtype]


def _call(name, *args):
    _check(getattr(lib(), name)(*args), name)


ACT_NONE, ACT_SQUARED_RELU, ACT_SILU, ACT_GELU, ACT_GATED = 0, 1, 2, 3, 4
SCORES_SOFTMAX, SCORES_SIGMOID = 0, 1
NORM_NONE, NORM_RMS, NORM_LAYER = 0, 1, 2


def gemm_nk(a, b, squared_relu=False, workspace=None, act=None, bias=None):
    """act(a . b^T + bias), b [N, K], in the type of a (bf16: an activation or a bias, not both)."""
    act = act or (ACT_SQUARED_RELU if squared_relu else ACT_NONE)
    M, K = a.shape
    N = b.shape[0]
    d = torch.empty((M, N), dtype=a.dtype, device=a.device)
    if a.dtype == torch.float32:
        _call("nf_gemm_nk_f32", _p(a), _p(b), _p(bias), _p(d), M, N, K, act, _stream())
    else:
        ws_bytes = workspace.numel() * workspace.element_size() if workspace is not None else 0
        tail = (_p(d), M, N, K, _p(workspace), ws_bytes, _stream())
        if bias is not None:
            _call("nf_gemm_nk_bias_bf16", _p(a), _p(b), _p(bias), *tail)
        else:
            name = {ACT_NONE: "nf_gemm_nk_bf16", ACT_SQUARED_RELU: "nf_gemm_nk_relu2_bf16", ACT_SILU: "nf_gemm_nk_silu_bf16",
                    ACT_GELU: "nf_gemm_nk_gelu_bf16"}[act]
            _call(name, _p(a), _p(b), *tail)
    return d


def gemm_nk_sums(a, b, max_shares=1):
    """fp32 sums [shares, M, N] of a . b^T (bf16 operands)."""
    M, K = a.shape
    N = b.shape[0]
    shares = lib().nf_gemm_nk_sums_shares(M, N, K, max_shares)
    p = torch.empty((shares, M, N), dtype=torch.float32, device=a.device)
    _call("nf_gemm_nk_sums_bf16", _p(a), _p(b), _p(p), p.numel() * 4, M, N, K, max_shares, _stream())
    return p


def embed_rows(tokens, positions, embed, pos, scale=1.0):
    """(fp32 rows, rows in the tables' type); the embedding is multiplied by scale"""
    T, ld = tokens.numel(), embed.shape[1]
    x = torch.empty((T, ld), dtype=torch.float32, device=embed.device)
    act = torch.empty((T, ld), dtype=embed.dtype, device=embed.device)
    _call("nf_embed_rows", _dt(embed), _p(tokens), _p(positions), _p(embed), _p(pos), scale, _p(x), _p(act), T, ld, _stream())
    return x, act


def norm(kind, weight=None, bias=None, eps=0.0) -> Norm:
    n = Norm(kind, _p(weight), _p(bias), eps)
    n.tensors = (weight, bias)      # the struct holds addresses only
    return n


def residual_rows(y, x, act, width, y_norm=None, next_norm=None, y_scale=1.0, add=None, table=None, tokens=None, table_scale=1.0):
    """x += y_scale * y_norm(y) in place; y [shares, T, ld] fp32 or [T, ld] bf16 (or None); then x += add + table_scale * table[tokens];
    act (or None) receives next_norm(x) in its type."""
    shares = y.shape[0] if y is not None and y.dim() == 3 else 1
    T, ld = x.shape
    a = ResidualArgs(rows=T, width=width, ld=ld, y_dtype=F32 if y is None else _dt(y), shares=shares, y=_p(y), y_norm=y_norm or Norm(),
                     next=next_norm or Norm(), y_scale=y_scale, x=_p(x), dtype=_dt(act) if act is not None else F32, act=_p(act), add=_p(add),
                     table=_p(table), tokens=_p(tokens), table_scale=table_scale)
    _call("nf_residual_rows", C.byref(a), _stream())


def mixture_rows(y, routing, top, identity, x, act, width, next_norm=None, y_scale=1.0, y_norm=None, plain=False):
    """x += y_scale * y_norm of the weighted sum (plain: the sum) of every token's sorted rows of y [sorted, ld] and of identity
    [T, ld] (or None)."""
    T, ld = x.shape
    if plain:
        routing = Routing.from_buffer_copy(routing)
        routing.weight = None
    a = ResidualArgs(rows=T, y_norm=y_norm or Norm(), width=width, ld=ld, y=_p(y), routing=C.pointer(routing), top=top, y_ld=y.shape[1], identity=_p(identity),
                     next=next_norm or Norm(), y_scale=y_scale, x=_p(x), dtype=_dt(y), act=_p(act))
    _call("nf_residual_rows", C.byref(a), _stream())


def norm_rows(x, index, n, width, dtype):
    out = torch.empty((x.shape[0] if index is None else index.numel(), x.shape[1]), dtype=dtype, device=x.device)
    _call("nf_norm_rows", _dt(out), _p(x), _p(index), C.byref(n), _p(out), out.shape[0], width, x.shape[1], _stream())
    return out


def norm_add_rows(y, weight, x, act, width, eps):
    """x += RMS norm of y, times weight, in place; act receives x in its type."""
    residual_rows(y, x, act, width, norm(NORM_RMS, weight, None, eps))


def gather_norm_rows(x, index, weight, width, eps, dtype):
    return norm_rows(x, index, norm(NORM_RMS, weight, None, eps), width, dtype)


def gated_norm_rows(o, g, weight, width, eps):
    """RMS norm of the rows of o, times weight and sigmoid(g), in place."""
    _call("nf_gated_norm_rows", _dt(o), _p(o), o.shape[1], _p(g), g.shape[1], _p(weight), o.shape[0], width, eps, _stream())


def token_gate_rows(sums, tokens, table, col0, dim):
    out = torch.empty(sums.shape[1:], dtype=table.dtype, device=sums.device)
    _call("nf_token_gate_rows", _dt(table), _p(sums), sums.shape[0], _p(tokens), _p(table), table.shape[1], col0, dim, _p(out),
          sums.shape[1], sums.shape[2], _stream())
    return out


def route(z, outputs, experts, top, correction, scale, tile_rows, groups=1, keep_groups=1, always=0, scores=SCORES_SOFTMAX, always_plain=False):
    """(Routing, dict of its tensors) of router outputs z [shares, T, ld] fp32; always: experts of every token behind the chosen
    ones, weighed by the column after the outputs (always_plain: by 1)."""
    shares, T, ld = z.shape
    n, e = T * (top + always), experts + always
    i32 = lambda k: torch.full((k,), -7, dtype=torch.int32, device=z.device)
    t = {"choice": i32(n), "weight": torch.empty(n, dtype=torch.float32, device=z.device), "place": i32(n), "row_of": i32(n),
         "offsets": i32(e + 1), "tile_group": i32(lib().nf_routing_max_tiles(n, e, tile_rows)), "n_tiles": i32(1),
         "row_weight": torch.full((n,), -7.0, dtype=torch.float32, device=z.device)}
    t["tile_row"] = torch.empty_like(t["tile_group"])
    r = Routing(**{k: _p(v) for k, v in t.items()}, tile_rows=tile_rows)
    a = RouteArgs(z=_p(z), shares=shares, ld=ld, rows=T, outputs=outputs, experts=experts, top=top, always=always, groups=groups,
                  keep_groups=keep_groups, correction=_p(correction), scale=scale, scores=scores, always_plain=int(always_plain))
    _call("nf_route", C.byref(a), C.byref(r), _stream())
    return r, t


def gemm_grouped_heads(a, b, d, a_group, d_group):
    """D_g = A_g . B_g^T for b [groups, N, K]: all rows of a, columns from g * a_group, to d's from g * d_group."""
    g, N, Kd = b.shape
    args = GroupedGemmArgs(dtype=_dt(a), groups=g, M=a.shape[0], N=N, K=Kd, a=_p(a), lda=a.shape[1], a_group=a_group, b=_p(b), d=_p(d),
                           ldd=d.shape[1], d_group=d_group)
    _call("nf_gemm_grouped", C.byref(args), _stream())
    return d


def gemm_grouped_experts(a, b, d, routing, max_rows, gather, act=ACT_NONE, weigh=False, gated=(1.0, 0.0, None)):
    """Sorted rows d = act(A . B_e^T): a holds tokens (gather) or sorted rows.  weigh: the product's rows are multiplied by their
    weights first; gated: slope, shift and limits per expert of ACT_GATED."""
    e, N, Kd = b.shape
    args = GroupedGemmArgs(dtype=_dt(a), act=act, groups=e, M=a.shape[0], N=N, K=Kd, a=_p(a), lda=a.shape[1], b=_p(b), d=_p(d),
                           ldd=d.shape[1], routing=routing, gather=int(gather), max_rows=max_rows, weigh=int(weigh),
                           gated=GatedAct(gated[0], gated[1], _p(gated[2])))
    _call("nf_gemm_grouped", C.byref(args), _stream())
    return d


def token_shift(x, shift_state, mu, input_indptr, rev_input_indptr, positions, state_slots, dtype):
    T, ld = x.shape
    out = torch.empty((mu.shape[0], T, ld), dtype=dtype, device=x.device)
    _call("nf_token_shift", _dt(out), _p(x), _p(shift_state), _p(mu), _p(out), mu.shape[0], _p(input_indptr),
          _p(rev_input_indptr), _p(positions), _p(state_slots), T, ld, _stream())
    return out


def tanh_rows(sums, dtype):
    out = torch.empty(sums.shape[1:], dtype=dtype, device=sums.device)
    _call("nf_tanh_rows", _dt(out), _p(sums), sums.shape[0], _p(out), sums.shape[1], sums.shape[2], _stream())
    return out


def argmax_f32(logits, cols=None):
    out = torch.empty((logits.shape[0],), dtype=torch.int32, device=logits.device)
    _call("nf_argmax_f32", _p(logits), _p(out), logits.shape[0], cols or logits.shape[1], logits.shape[1], _stream())
    return out


def kv_layout(dtype, heads, kv_heads, dim, vdim, maps=1) -> KVLayout:
    return KVLayout(BF16 if dtype == torch.bfloat16 else F32, heads, kv_heads, dim, vdim, (dim + 31) // 32 * 32,
                    (vdim + 15) // 16 * 16, 16, maps)


def kv_pool(layout: KVLayout, pages, device="cuda"):
    n = lib().nf_kv_page_elements(C.byref(layout))
    return torch.zeros((pages, n), dtype=torch.bfloat16 if layout.dtype == BF16 else torch.float32, device=device)


def rotation(table=None, dims=0, interleaved=False) -> Rotation:
    """table: fp32 [positions, dims / 2, 2] of (cos, sin)."""
    r = Rotation(_p(table) if table is not None else None, dims, int(interleaved))
    r.tensors = (table,)            # the struct holds addresses only
    return r


def short_conv(weight, state, input_indptr, state_slots) -> ShortConv:
    """weight [taps, columns], state [slots, taps - 1, columns] in the type of the projected rows."""
    c = ShortConv(weight.shape[0], _p(weight), _p(state), _p(input_indptr), _p(state_slots))
    c.tensors = (weight, state, input_indptr, state_slots)      # the struct holds addresses only
    return c


def qkv_append(layout, proj, cols, q_norm, k_norm, eps, rot, pool, kv_indptr, kv_indices, rev_input_indptr, positions, q_temp=None, conv=None,
               value_norm=False, value_rot=None):
    """Returns the normed, rotated queries [T, heads * maps, k_pad]; keys and values go to the pool's pages, what a convolution
    needs of these rows to its state."""
    T = proj.shape[0]
    q = torch.empty((T, layout.heads * layout.maps, layout.k_pad), dtype=proj.dtype, device=proj.device)
    _call("nf_qkv_append", C.byref(layout), _p(proj), proj.shape[1], *cols, _p(q_norm), _p(k_norm), eps, C.byref(rot),
          C.byref(QueryTemperature(*q_temp)) if q_temp else None,
          C.byref(ValueForm(int(value_norm), value_rot or Rotation())) if value_norm or value_rot else None, C.byref(conv) if conv else None, _p(q), _p(pool), _p(kv_indptr),
          _p(kv_indices), _p(rev_input_indptr), _p(positions), T, _stream())
    if conv:
        _call("nf_conv_state", _dt(proj), _p(proj), proj.shape[1], C.byref(conv), _p(positions), 0, kv_indptr.numel() - 1, _stream())
    return q


def window_attention(layout, q, pool, batch, *, window, keep_first, scale, sink=None, out_scale=1.0, decode=0, gate=None, softcap=0.0,
                     map_weight=0.0, head_eps=None, chunk=0, out_rot=None):
    """batch: dict of device arrays input_indptr, kv_indptr, kv_indices, rev_input_indptr, positions; the first
    `decode` requests have one row each.  Returns [T, heads * vdim]."""
    T = q.shape[0]
    out = torch.zeros((T, layout.heads * layout.vdim), dtype=q.dtype, device=q.device)
    n_req = batch["input_indptr"].numel() - 1
    a = WindowAttentionArgs(kv=layout, window=window, keep_first=keep_first, chunk=chunk, out_rot=out_rot or Rotation(), scale=scale, out_scale=out_scale, softcap=softcap,
                            map_weight=map_weight, head_norm=int(head_eps is not None), head_eps=head_eps or 0.0, sink=_p(sink),
                            gate=_p(gate), gate_ld=gate.shape[1] if gate is not None else 0, q=_p(q), out=_p(out), out_ld=out.shape[1], out_col=0, kv_data=_p(pool))
    for n in ("input_indptr", "kv_indptr", "kv_indices", "rev_input_indptr", "positions"):
        setattr(a, n, _p(batch[n]))
    for first, n, rows, dec in ((0, decode, decode, 1), (decode, n_req - decode, T - decode, 0)):
        if n:
            a.req_begin, a.req_num, a.row_begin, a.max_rows, a.decode = first, n, first, rows, dec
            _call("nf_window_attention", C.byref(a), _stream())
    return out


def latent_layout(dtype, heads, kv_rank, rot_dim) -> LatentLayout:
    l = LatentLayout()
    _call("nf_latent_layout_of", BF16 if dtype == torch.bfloat16 else F32, heads, kv_rank, rot_dim, 16, C.byref(l))
    return l


def latent_pool(layout: LatentLayout, pages, device="cuda"):
    return torch.zeros((pages, 16, layout.row_ld), dtype=torch.bfloat16 if layout.dtype == BF16 else torch.float32, device=device)


def latent_append(layout, proj, cols, weight, eps, rot, q, pool, batch):
    """cols: (rotated query parts, latent); q [T, heads, row_ld] receives its columns from rank_pad on."""
    _call("nf_latent_append", C.byref(layout), _p(proj), proj.shape[1], *cols, _p(weight), eps, C.byref(rot), _p(q), _p(pool),
          *(_p(batch[n]) for n in ("kv_indptr", "kv_indices", "rev_input_indptr", "positions")), proj.shape[0], proj.shape[0], _stream())


def latent_expand(layout, dim_pad, vdim_pad, weight, pool, batch, req_begin, req_end, max_pages):
    """Keys and values of all heads of the requests' positions: (KVLayout, pages, page_ids); weight [heads * (dim_pad + vdim_pad),
    rank_pad], keys first."""
    H = layout.heads
    kv = kv_layout(pool.dtype, H, H, dim_pad + layout.rot_dim, vdim_pad)
    new = lambda *shape: torch.full(shape, 3.0, dtype=pool.dtype, device=pool.device)
    rows, pages = new(max_pages * 16, layout.rank_pad), new(max_pages, lib().nf_kv_page_elements(C.byref(kv)))
    ids = torch.zeros_like(batch["kv_indices"])
    a = LatentExpandArgs(layout=layout, kv=kv, dim_pad=dim_pad, kv_data=_p(pool), kv_indptr=_p(batch["kv_indptr"]), kv_indices=_p(batch["kv_indices"]),
                         req_begin=req_begin, req_end=req_end, max_pages=max_pages, rows=_p(rows), page_ids=_p(ids), ld=weight.shape[0], k_col=0,
                         v_col=H * dim_pad, pages=_p(pages))
    _call("nf_latent_gather", C.byref(a), _stream())
    products = gemm_nk(rows, weight)
    a.products = _p(products)
    _call("nf_latent_pack", C.byref(a), _stream())
    return kv, pages, ids


def latent_queries(kv, dim_pad, proj, q_col, rot_dim, rot, positions, row_begin, rows):
    q = torch.zeros((proj.shape[0], kv.heads, kv.k_pad), dtype=proj.dtype, device=proj.device)
    _call("nf_latent_queries", C.byref(kv), dim_pad, _p(proj), proj.shape[1], q_col, rot_dim, C.byref(rot), _p(positions), _p(q), row_begin, rows,
          _stream())
    return q


def latent_attention(layout, q, pool, batch, *, scale, decode=0, workspace=True, window=0):
    """q [T, heads, row_ld]; returns [T, heads, rank_pad]."""
    T = q.shape[0]
    out = torch.zeros((T, layout.heads, layout.rank_pad), dtype=q.dtype, device=q.device)
    n_req = batch["input_indptr"].numel() - 1
    ws = torch.empty((max(lib().nf_latent_workspace_bytes(C.byref(layout), T), 16),), dtype=torch.uint8, device=q.device) if workspace else None
    a = LatentAttentionArgs(layout=layout, window=window, scale=scale, q=_p(q), out=_p(out), kv_data=_p(pool), workspace=_p(ws),
                            workspace_bytes=ws.numel() if workspace else 0)
    for n in ("input_indptr", "kv_indptr", "kv_indices", "rev_input_indptr", "positions"):
        setattr(a, n, _p(batch[n]))
    for first, n, rows, dec in ((0, decode, decode, 1), (decode, n_req - decode, T - decode, 0)):
        if n:
            a.req_begin, a.req_num, a.row_begin, a.max_rows, a.decode = first, n, first, rows, dec
            _call("nf_latent_attention", C.byref(a), _stream())
    return out


def linear_recurrence(kind, q, k, v, g, heads, dim, vdim, state, batch, *, eps, decode=0, rot=None, k_scale=1.0,
                      log2_decay=None, z=None, w0=None, u=None, norm_weight=None, out_scale=1.0, shift_x=None,
                      shift_state=None):
    """q, k, v, g: 2-d tensors of rows; batch: device arrays input_indptr, positions, state_slots.  Returns
    [T, heads * vdim]; the state is updated in place."""
    T = q.shape[0]
    out = torch.zeros((T, heads * vdim), dtype=q.dtype, device=q.device)
    n_req = batch["input_indptr"].numel() - 1
    ws = torch.empty((max(lib().nf_recurrence_workspace_bytes(heads, dim, vdim, T, n_req), 16),), dtype=torch.uint8, device=q.device)
    a = RecurrenceArgs(dtype=_dt(q), kind=kind, heads=heads, dim=dim, vdim=vdim, q=_p(q), k=_p(k), v=_p(v), g=_p(g),
                       q_ld=q.shape[1], k_ld=k.shape[1], v_ld=v.shape[1], g_ld=g.shape[1] if g is not None else 0, rot=rot or Rotation(),
                       k_scale=k_scale, log2_decay=_p(log2_decay), z=_p(z), z_ld=z.shape[1] if z is not None else 0,
                       z_shares=1, w0=_p(w0), u=_p(u), norm_weight=_p(norm_weight), eps=eps, out_scale=out_scale,
                       state=_p(state), out=_p(out), out_ld=out.shape[1], out_col=0, shift_x=_p(shift_x),
                       shift_state=_p(shift_state), shift_ld=shift_x.shape[1] if shift_x is not None else 0, total_rows=T,
                       workspace=_p(ws), workspace_bytes=ws.numel())
    for n in ("input_indptr", "positions", "state_slots"):
        setattr(a, n, _p(batch[n]))
    for first, n, rows in ((0, decode, decode), (decode, n_req - decode, T - decode)):
        if n:
            a.req_begin, a.req_num, a.row_begin, a.rows = first, n, first, rows
            _call("nf_linear_recurrence", C.byref(a), _stream())
    return out
