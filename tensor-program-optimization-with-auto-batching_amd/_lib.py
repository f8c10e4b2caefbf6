"""ctypes binding of the kernel libraries (the C ABI declared in include/mlora.h and include/mlora_decoder.h): one library
per element type, with the same entry points.

There is no fallback: if a library has not been built, loading it raises and every operator fails.
"""
from __future__ import annotations

import ctypes as C
import os

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "libmlora_hip.so")
LIB_PATHS = {"float16": LIB_PATH, "bfloat16": os.path.join(_HERE, "libmlora_bf16.so"), "float32": os.path.join(_HERE, "libmlora_f32.so")}

F16, F32 = 0, 1          # F16: the library's own 16-bit element type (in the fp32 library: fp32)
GLU_SILU, GLU_CLIPPED = 0, 1
ACT_NONE, ACT_RELU2, ACT_GLU = 0, 1, 2
MOE_UP, MOE_DOWN = 0, 1
ROWMAJOR, FRAG = 0, 1
STORE, ACCUMULATE = 0, 1
PAGE_SIZE = 16

_p, _i, _f, _z, _l = C.c_void_p, C.c_int, C.c_float, C.c_size_t, C.c_long

# name -> (restype, argtypes); mirrors include/mlora.h one to one
SIGNATURES = {
    "mlora_version": (_i, []),
    "mlora_last_error": (C.c_char_p, []),
    "mlora_gather_mm_workspace_bytes": (_z, [_i, _i, _i]),
    "mlora_gather_mm": (_i, [_p, _i, _i, _p, _i, _p, _p, _p, _f, _i, _i, _i, _i, _i, _p, _z, _p]),
    "mlora_gather_mm_static_max_bytes": (_z, []),
    "mlora_gather_mm_static": (_i, [_p, _i, _i, _p, _i, _p, _p, _p, _f, _i, _i, _i, _i, _i, _p]),
    "mlora_gather_mm_multi": (_i, [_p, _i, _i, _p, _i, _p, _i, _p, _p, _i, _i, _i, _p, _z, _p]),
    "mlora_gather_mm_multi_proj": (_i, [_p, _i, _i, _p, _i, _p, _i, _i, _p, _p, _p, _p, _i, _i, _p, _z, _p]),
    "mlora_gather_mm_batch": (_i, [_p, _i, _i, _i, _i, _p, _f, _i, _i, _i, _i, _i, _p, _z, _p]),
    "mlora_lora_shrink": (_i, [_p, _p, _i, _p, _p, _i, _i, _i, _i, _p]),
    "mlora_lora_expand": (_i, [_p, _i, _i, _p, _p, _p, _f, _i, _i, _i, _i, _i, _p]),
    "mlora_write_tensor_part": (_i, [_p, _p, _p, _p, _i, _i, _i, _p]),
    "mlora_gemv": (_i, [_p, _i, _i, _p, _i, _p, _i, _i, _i, _p]),
    "mlora_gemm": (_i, [_p, _i, _i, _p, _i, _p, _i, _i, _i, _p]),
    "mlora_linear": (_i, [_p, _i, _i, _p, _i, _p, _i, _i, _i, _p]),
    "mlora_packed_weight_elems": (_z, [_i, _i]),
    "mlora_pack_weight": (_i, [_p, _p, _i, _i, _p]),
    "mlora_gemv_packed": (_i, [_p, _i, _i, _p, _i, _p, _i, _i, _i, _p]),
    "mlora_gemm_packed": (_i, [_p, _i, _i, _p, _i, _p, _i, _i, _i, _p]),
    "mlora_linear_packed": (_i, [_p, _i, _i, _p, _i, _p, _i, _i, _i, _p]),
    "mlora_frag_activation_elems": (_z, [_i, _i]),
    "mlora_pack_activation": (_i, [_p, _p, _i, _i, _i, _p]),
    "mlora_gemv_frag": (_i, [_p, _i, _i, _p, _p, _i, _i, _i, _p]),
    "mlora_linear_frag": (_i, [_p, _i, _i, _p, _p, _i, _i, _i, _p]),
    "mlora_gemm_frag_preferred": (_i, [_i, _i, _i]),
    "mlora_lora_block_adapters": (_i, [_p, _p, _p, _i, _i, _p]),
    "mlora_lora_shrink_split": (_i, [_p, _p, _p, _i, _p, _i, _p, _f, _i, _i, _i, _i, _p, _z, _p]),
    "mlora_linear_frag_lora": (_i, [_p, _i, _i, _p, _p, _i, _i, _i, _p, _i, _p, _i, _p]),
    "mlora_linear_frag_silu": (_i, [_p, _p, _p, _i, _i, _i, _p, _i, _p, _i, _p]),
    "mlora_gemv_frag_lora": (_i, [_p, _i, _i, _p, _p, _i, _i, _i, _p, _p, _i, _p, _i, _i, _p]),
    "mlora_gemv_frag_silu": (_i, [_p, _p, _p, _i, _i, _i, _p]),
    "mlora_gemv_frag_clipglu": (_i, [_p, _p, _p, _i, _i, _i, _f, _f, _f, _p]),
    "mlora_linear_frag_clipglu": (_i, [_p, _p, _p, _i, _i, _i, _f, _f, _f, _p]),
    "mlora_clipglu_mul": (_i, [_p, _i, _p, _p, _i, _i, _i, _f, _f, _f, _p]),
    "mlora_gemv_frag_split": (_i, [_p, _i, _i, _p, _p, _p, _i, _i, _i, _i, _p]),
    "mlora_gemv_split_kq": (_i, [_i, _i, _i, _i]),
    "mlora_gemv_frag_split_kq": (_i, [_p, _p, _i, _p, _p, _i, _i, _i, _i, _p]),
    "mlora_rope_kv_append_lora": (_i, [_p, _p, _p, _p, _i, _p, _p, _p, _p, _i, _i, _i, _i, _i, _i, _i, _p, _i, _p, _p, _f, _i, _i, _i, _p]),
    "mlora_rope_attn_decode": (_i, [_p, _i, _p, _p, _p, _p, _i, _p, _p, _p, _p, _p, _i, _i, _i, _i, _i, _i, _i, _p, _i, _p, _p, _f, _i, _i, _i, _p]),
    "mlora_gemv_ksplit": (_i, [_i, _i, _i]),
    "mlora_gemv_ksplit_bytes": (_z, [_i, _i, _i]),
    "mlora_gemv_shrink_rows": (_i, [_i, _i, _i]),
    "mlora_gemv_frag_acc_ksplit": (_i, [_p, _p, _p, _i, _p, _p, _i, _i, _i, _i, _p, _p, _i, _p, _i, _i, _p]),
    "mlora_gemv_delta_ride_ksplit": (_i, [_i, _i, _i, _i]),
    "mlora_gemv_frag_acc_ksplit_delta": (_i, [_p, _p, _i, _p, _p, _i, _i, _i, _p, _i, _p, _p, _f, _i, _i, _p]),
    "mlora_rope_attn_oshrink_ok": (_i, [_i, _i, _i, _i, _i]),
    "mlora_paged_attn_decode_oshrink": (_i, [_p, _i, _p, _p, _p, _p, _i, _p, _p, _i, _i, _i, _i, _i, _i, _p, _i, _i, _p, _p, _p]),
    "mlora_lora_expand_shares_ok": (_i, [_i, _i]),
    "mlora_lora_expand_shares": (_i, [_p, _p, _i, _p, _p, _f, _i, _i, _i, _i, _p]),
    "mlora_rope_attn_decode_oshrink": (_i, [_p, _i, _p, _p, _p, _p, _i, _p, _p, _p, _p, _p, _i, _i, _i, _i, _i, _i, _i, _p, _i, _p, _p, _f, _i, _i, _i, _p, _p, _p]),
    "mlora_rmsnorm_ksplit": (_i, [_p, _i, _p, _p, _i, _i, _p, _f, _i, _i, _p, _i, _p, _p, _f, _i, _i, _i, _p]),
    "mlora_lora_expand_rmsnorm": (_i, [_p, _i, _p, _p, _i, _p, _p, _f, _p, _f, _i, _i, _i, _i, _i, _p]),
    "mlora_rmsnorm": (_i, [_p, _i, _p, _i, _p, _f, _i, _i, _p]),
    "mlora_silu_mul": (_i, [_p, _i, _p, _p, _i, _i, _i, _p]),
    "mlora_embed": (_i, [_p, _i, _p, _p, _i, _i, _i, _p]),
    "mlora_argmax": (_i, [_p, _p, _i, _i, _p]),
    "mlora_rope_kv_append": (_i, [_p, _p, _p, _p, _i, _p, _p, _p, _p, _i, _i, _i, _i, _i, _i, _i, _p]),
    "mlora_paged_attn_decode": (_i, [_p, _i, _p, _p, _p, _p, _i, _p, _p, _i, _i, _i, _i, _i, _i, _p]),
    "mlora_paged_attn_prefill": (_i, [_p, _i, _p, _p, _p, _p, _i, _p, _p, _i, _i, _i, _i, _i, _i, _p]),
}



class LoraBucket(C.Structure):
    _fields_ = [("A", _p), ("B", _p), ("r", _i), ("n_ad", _i), ("scaling", _f)]


class FusedLora(C.Structure):
    _fields_ = [("B", _p), ("v_hi", _p), ("v_lo", _p), ("n_begin", _i), ("n_rows", _i)]


class LoraProj(C.Structure):
    _fields_ = [("A", _p), ("B", _p)]


class Layer(C.Structure):
    _fields_ = [("qkv_p", _p), ("o_p", _p), ("gate_up_p", _p), ("gate_up_il_p", _p), ("down_p", _p), ("ln1", _p), ("ln2", _p),
                ("lora", LoraProj * 7), ("k_cache", _p), ("v_cache", _p)]


class DecodePlan(C.Structure):
    _fields_ = [("n_layers", _i), ("hidden", _i), ("inter", _i), ("n_q_heads", _i), ("n_kv_heads", _i), ("head_dim", _i),
                ("vocab", _i), ("eps", _f), ("lora_r", _i), ("lora_n_ad", _i), ("lora_scaling", _f), ("lora_dense", _i),
                ("layers", C.POINTER(Layer)), ("embed", _p), ("norm", _p), ("lm_head_p", _p),
                ("rope_cos", _p), ("rope_sin", _p), ("max_pos", _i),
                ("block_table", _p), ("max_blocks", _i), ("n_pages", _i), ("n_seq", _i),
                ("T", _i), ("tokens", _p), ("rows", _p), ("pos", _p), ("ctx", _p), ("tok_adapter", _p),
                ("resid", _p), ("xn", _p), ("qkv", _p), ("attn", _p), ("gate_up", _p), ("act", _p), ("logits", _p),
                ("lora_ws", _p), ("lora_ws_bytes", _z), ("ksplit_ws", _p), ("ksplit_ws_bytes", _z)]


SIGNATURES["mlora_decode_step"] = (_i, [C.POINTER(DecodePlan), _p])


class TanhNorm(C.Structure):
    _fields_ = [("w", _p), ("b", _p), ("alpha", _f)]


class StreamStep(C.Structure):
    _fields_ = [("x_out", _p), ("x", _p), ("y", _p), ("part", _p), ("rows", _p), ("out_frag", _p), ("out_row", _p), ("mu", _p), ("shift", _p),
                ("tok_seq", _p), ("tok_pos", _p), ("tok_last", _p), ("post", TanhNorm), ("pre", TanhNorm), ("mix_stride", _l),
                ("n_part", _i), ("top", _i), ("T", _i), ("Hp", _i), ("ld_row", _i), ("n_seq", _i), ("mult", _f), ("row_weight", _f)]


# mirrors include/mlora_decoder.h (the bfloat16 and fp32 libraries)
DECODER_SIGNATURES = {
    "mlora_stream_norm": (_i, [_p, _p, _p, _p, _i, _p, _p, _f, _f, _i, _i, _i, _i, _p]),
    "mlora_stream_step": (_i, [C.POINTER(StreamStep), _p]),
    "mlora_embed_scaled": (_i, [_p, _p, _p, _i, _p, _p, _f, _i, _i, _i, _p]),
    "mlora_linear_ksplit_store": (_i, [_p, _p, _i, _p, _p, _i, _i, _i, _p]),
    "mlora_gemm_frag_groups": (_i, [_p, _p, _l, _i, _p, _i, _i, _i, _p]),
    "mlora_narrow_linear": (_i, [_p, _p, _p, _i, _i, _i, _p]),
    "mlora_gemv_groups_parts": (_i, [_i]),
    "mlora_gemv_frag_groups": (_i, [_p, _p, _p, _l, _i, _p, _i, _i, _i, _i, _p]),
    "mlora_time_mix": (_i, [_p, _i, _i, _p, _p, _p, _p, _i, _p, _i, _i, _i, _p, _i, _p, _p, _p, _f, _p, _i, _p, _i, _p, _p, _i, _i, _i, _p]),
    "mlora_tanh_parts": (_i, [_p, _p, _p, _i, _i, _i, _p]),
    "mlora_time_mix_prompt_served": (_i, [_i]),
    "mlora_time_mix_prompt": (_i, [_p, _i, _i, _p, _p, _p, _p, _i, _p, _i, _p, _p, _p, _p, _f, _p, _i, _p, _i, _p, _i, _p, _z, _i, _i, _i, _i, _p]),
    "mlora_tied_prep": (_i, [_p, _p, _p, _p, _i, _p, _p, _f, _f, _f, _p, _i, _p, _p, _i, _i, _i, _i, _i, _i, _p]),
    "mlora_tied_attn_splits": (_i, [_i, _i, _i, _i]),
    "mlora_tied_attn": (_i, [_p, _i, _p, _p, _p, _p, _i, _p, _p, _p, _f, _i, _i, _i, _i, _i, _i, _i, _p, _z, _p]),
    "mlora_tied_prefill_served": (_i, [_i]),
    "mlora_tied_prefill_scratch_elems": (_z, [_i, _i, _i]),
    "mlora_tied_prefill": (_i, [_p, _i, _i, _p, _p, _p, _p, _i, _p, _i, _p, _f, _i, _i, _i, _i, _i, _p, _z, _p]),
    "mlora_token_gate": (_i, [_p, _p, _p, _p, _i, _i, _i, _p, _i, _i, _i, _i, _p]),
    "mlora_token_gate_mul": (_i, [_p, _p, _p, _i, _i, _i, _p, _i, _i, _i, _p]),
    "mlora_latent_prep": (_i, [_p, _i, _i, _p, _p, _i, _i, _i, _i, _f, _p, _f, _p, _i, _p, _p, _p, _p, _i, _i, _i, _i, _i, _i, _i, _p, _i, _p]),
    "mlora_head_linear": (_i, [_p, _i, _l, _l, _p, _l, _l, _p, _i, _i, _i, _i, _f, _p]),
    "mlora_latent_attn_splits": (_i, [_i, _i, _i]),
    "mlora_latent_attn_workspace_bytes": (_z, [_i, _i, _i, _i]),
    "mlora_latent_attn": (_i, [_p, _p, _p, _p, _i, _p, _p, _p, _f, _i, _i, _i, _i, _i, _i, _i, _p, _z, _p]),
    "mlora_latent_attn_out": (_i, [_p, _i, _l, _p, _i, _p, _p, _p, _i, _p, _p, _p, _f, _i, _i, _i, _i, _i, _i, _i, _p, _z, _p]),
    "mlora_latent_prefill_tile_tokens": (_i, []),
    "mlora_latent_prefill_served": (_i, [_i, _i, _i]),
    "mlora_latent_prefill_scratch_elems": (_z, [_i, _i, _i, _i, _i]),
    "mlora_latent_prefill": (_i, [_p, _i, _i, _p, _i, _p, _p, _p, _i, _p, _i, _p, _p, _p, _f, _i, _i, _i, _i, _i, _i, _i, _p, _z, _p]),
    "mlora_moe_route": (_i, [_p, _p, _p, _i, _p, _f, _i, _i, _i, _p]),
    "mlora_moe_tile_rows": (_i, [_i, _i, _i]),
    "mlora_moe_max_tiles": (_i, [_i, _i, _i]),
    "mlora_moe_max_places": (_i, [_i, _i, _i]),
    "mlora_moe_plan": (_i, [_p, _p, _p, _p, _i, _i, _i, _p]),
    "mlora_moe_table_plan": (_i, [_p, _p, _p, _p, _p, _i, _i, _i, _i, _i, _p]),
    "mlora_moe_linear": (_i, [_p, _p, _p, _p, _p, _p, _i, _i, _i, _i, _i, _i, _i, _i, _i, _f, _p, _z, _p]),
    "mlora_moe_combine": (_i, [_p, _p, _i, _p, _p, _i, _i, _i, _p, _p]),
}

# ... and those that the fp32 library does not have
MATRIX_CORE_ONLY = ("mlora_token_gate", "mlora_latent_attn_out", "mlora_latent_prefill", "mlora_latent_prefill_tile_tokens", "mlora_latent_prefill_served",
                    "mlora_latent_prefill_scratch_elems", "mlora_tied_prefill", "mlora_tied_prefill_served", "mlora_tied_prefill_scratch_elems",
                    "mlora_linear_ksplit_store", "mlora_gemv_frag_groups", "mlora_gemv_groups_parts", "mlora_gemm_frag_groups",
                    "mlora_narrow_linear", "mlora_tanh_parts", "mlora_time_mix_prompt", "mlora_time_mix_prompt_served")

_libs = {}


class MloraError(RuntimeError):
    def __init__(self, code: int, msg: str):
        super().__init__(f"mlora error {code}: {msg}")
        self.code = code


def lib(dtype: str = "float16") -> C.CDLL:
    """The loaded library of an element type; raises if it is missing (build it with build.py).  The bfloat16 and fp32
    libraries hold the decoder kernels and those of mlora.h that their sources give (no adapter kernels)."""
    l = _libs.get(dtype)
    if l is None:
        path = LIB_PATHS[dtype]
        if not os.path.exists(path):
            raise RuntimeError(f"{path} not found: the HIP library is not built (run build.py). There is no CPU fallback.")
        l = C.CDLL(path)
        table = SIGNATURES if dtype == "float16" else {**{n: v for n, v in SIGNATURES.items() if hasattr(l, n)}, **DECODER_SIGNATURES}
        if dtype == "float32":
            table = {n: v for n, v in table.items() if n not in MATRIX_CORE_ONLY}
        for name, (res, args) in table.items():
            fn = getattr(l, name)
            fn.restype = res
            fn.argtypes = args
        _libs[dtype] = l
    return l


def loaded() -> C.CDLL:
    """A library for what does not depend on the element type: one that is loaded already, else the fp16 one."""
    return next(iter(_libs.values()), None) or lib()


def check(code: int, dtype: str = "float16") -> None:
    if code != 0:
        raise MloraError(code, lib(dtype).mlora_last_error().decode())
