"""ctypes binding of ``libzipage_hip.so`` and of the model-side libraries (the C ABIs in
``include/zipage_hip.h`` and ``include/zipage_models.h``).

The product path has no CPU fallback: if the shared object is missing or a symbol cannot
be resolved, importing a kernel wrapper raises.  ctypes releases the GIL for the duration
of every call, so the wrappers can be driven from a worker thread while another thread
runs the model forward (the reference calls this path from a ThreadPoolExecutor worker,
zipage/engine/zipage_engine.py:153-166).
"""
from __future__ import annotations

import ctypes as C
import os

import torch

_HERE = os.path.dirname(os.path.abspath(__file__))
LIB_PATH = os.path.join(_HERE, "libzipage_hip.so")

ZP_BF16, ZP_F16, ZP_F32 = 0, 1, 2
_DTYPES = {torch.bfloat16: ZP_BF16, torch.float16: ZP_F16, torch.float32: ZP_F32}

i32, i64, f32, f64, ptr = C.c_int32, C.c_int64, C.c_float, C.c_double, C.c_void_p

# name -> argument types, in the order of include/zipage_hip.h
SIGNATURES = {
    "zp_store_query": [ptr, ptr, ptr, i32, i32, i32, i32, i32, i64, i64, i64, i64, i64, i32, ptr],
    "zp_attention_score": [ptr, ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i32,
                           i32, i32, i64, i64, i64, i64, f32, i32, i32, ptr, i64, ptr],
    "zp_global_score": [ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i64, i64, f32, i32, i32,
                        i32, ptr],
    "zp_pool_scores": [ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i32, ptr],
    "zp_key_norm": [ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i64, i64, f32, i32, ptr],
    "zp_redundancy_lightning": [ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i64, i64,
                                f32, f64, i32, ptr],
    "zp_redundancy_raw": [ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i64, i64, f32,
                          f64, i32, ptr, i64, ptr],
    "zp_score_epilogue": [ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, f64, i32, i32, i32,
                          i32, ptr],
    "zp_topk_mask": [ptr, ptr, i32, i32, i32, i32, ptr],
    "zp_select_topk": [ptr, ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i32, i32,
                       f64, i32, i32, i32, i32, i32, ptr],
    "zp_compress_kv": [ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i32,
                       i64, i64, i64, i64, i64, i64, i64, i64, i32, ptr],
    "zp_compress_score": [ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i64, i64, i64,
                          i64, i32, ptr],
    "zp_store_kvcache": [ptr, ptr, ptr, ptr, ptr, i32, i32, i64, i64, i64, i32, ptr],
    "zp_paged_decode_attention": [ptr, ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32,
                                  i64, i64, f32, i32, ptr],
    "zp_add_rms_norm": [ptr, ptr, ptr, ptr, i32, i32, i64, i64, i64, f32, i32, ptr],
    "zp_silu_and_mul": [ptr, ptr, i32, i32, i64, i64, i32, ptr],
    "zp_qk_norm_rope_store": [ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, i32, i32,
                              i32, i32, i32, i64, i64, i32, i32, i64, i64, f32, i32, ptr],
}


class CompressConfigC(C.Structure):
    """zp_compress_config of include/zipage_hip.h."""
    _fields_ = [("budget_blocks", i32), ("query_cache_len", i32), ("softmax_scale", f32),
                ("reduced", i32), ("use_global_score", i32), ("decay_factor", f32),
                ("activate_method", i32), ("max_norm", i32), ("use_redundancy", i32),
                ("lightning", i32), ("redundancy_lambda", f64), ("redundancy_temperature", f64),
                ("redundancy_threshold", f32), ("pooling_size", i32), ("continues_pooling", i32),
                ("pooling_mode", i32), ("sink_len", i32), ("deterministic_carry", i32)]


# stage order of the ZP_STAGE_* enum, under the names the reference's timers use
# (zipage/engine/model_runner.py:424-429); the one-launch selection has its own name
STAGE_NAMES = ("attention_score", "global_score", "pooling", "redudancy_score", "window_mask",
               "topk_mask", "pooling+window_mask+topk_mask", "compress_kv", "compress_global_score")

SIGNATURES["zp_compress_layers"] = (
    [ptr] * 9 + [i32] * 11 + [C.POINTER(i64), i32, C.POINTER(CompressConfigC), ptr, i64,
                              C.POINTER(ptr), ptr])
SIGNATURES["zp_compress_layers_static"] = (
    [ptr] * 9 + [i32] * 11 + [C.POINTER(i64), i32, C.POINTER(CompressConfigC), ptr])
SIGNATURES["zp_static_scratch_init"] = []
STATIC_SCRATCH_BYTES = 32 << 20
I64_RETURNING = {
    "zp_compress_layers_workspace": [i32, i32, i32, i32, i32, i32, i32, i32,
                                     C.POINTER(CompressConfigC), i32],
    "zp_attention_score_workspace": [i32, i32, i32, i32, i32, i32, i32],
    "zp_attention_score_workspace_for": [i32, i32, i32, i32, i32, i32, i32, i32],
    "zp_redundancy_raw_workspace": [i32, i32, i32, i32, i32],
}
EXPORTS = sorted(list(SIGNATURES) + list(I64_RETURNING) + ["zp_abi_version", "zp_last_error"])

class Branch(C.Structure):
    """zp_branch of include/zipage_models.h."""
    _fields_ = [("y", ptr), ("weight", ptr), ("planes", i32)]


class Segments(C.Structure):
    """zp_segments of include/zipage_models.h."""
    _fields_ = [(n, ptr) for n in ("rows", "counts", "slots", "starts")] + \
        [(n, i32) for n in ("n", "max_count", "num_slots", "num_rows")]


class MlstmArgs(C.Structure):
    """zp_mlstm."""
    _fields_ = [("seg", Segments)] + \
        [(n, ptr) for n in ("inp", "gates", "i_bias", "f_bias", "norm", "state", "out")] + \
        [(n, i64) for n in ("in_stride", "gate_stride", "out_stride")] + \
        [(n, i32) for n in ("heads", "dk", "dv", "vdim", "q_at", "k_at", "v_at", "g_at")] + \
        [(n, f32) for n in ("cap", "q_scale", "eps", "out_scale")]


class DeltaArgs(C.Structure):
    """zp_delta."""
    _fields_ = [("seg", Segments)] + \
        [(n, ptr) for n in ("inp", "low", "filters", "a_log", "dt_bias", "norm", "state", "conv_state", "out")] + \
        [(n, i64) for n in ("in_stride", "low_stride", "out_stride")] + \
        [(n, i32) for n in ("heads", "kv_heads", "dk", "dv", "vdim", "taps", "b_at", "g_at")] + \
        [(n, f32) for n in ("q_scale", "eps", "out_scale")]


class LinearArgs(C.Structure):
    """zp_linear."""
    _fields_ = [("seg", Segments)] + \
        [(n, ptr) for n in ("inp", "low", "decay", "freqs", "norm", "state", "out")] + \
        [(n, i64) for n in ("in_stride", "low_stride", "out_stride")] + \
        [(n, i32) for n in ("heads", "dk", "dv", "vdim", "rot", "q_at", "k_at", "v_at", "g_at")] + \
        [(n, f32) for n in ("q_scale", "k_scale", "inv_tau", "eps")]


class AttentionForm(C.Structure):
    """zp_attention_form."""
    _fields_ = [("softcap", f32), ("maps", i32), ("balance", f32), ("eps", f32), ("vdim", i32), ("gate", ptr),
                ("gate_stride", i64), ("turns", ptr)]


class StoreForm(C.Structure):
    """zp_store_form."""
    _fields_ = [("norm", ptr), ("q_norm", i32), ("k_norm", i32), ("eps", f32), ("tied", i32), ("V", i32),
                ("value_freqs", ptr), ("turns", ptr)]


SCORE_SOFTMAX, SCORE_SIGMOID = 0, 1      # ZP_SCORE_*
GATE_CLAMPED, GATE_SILU = 0, 1           # ZP_GATE_*
form_ptr = C.POINTER(AttentionForm)

# the model-side libraries, in the order of include/zipage_models.h: name -> (entry points, those that
# return an int64 count instead of a status)
MODEL_LIBS = {
    "models": ({
        "zp_embed_norm": [ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i64, i64, f32, f32, f32, f32, i32, ptr],
        "zp_residual_norm": [ptr, C.POINTER(Branch), i32, ptr, i64, ptr, i32, ptr, ptr, ptr, ptr, ptr, ptr, i32, i32, i32,
                             f32, f32, f32, f32, i32, ptr],
        "zp_normed_powers": [ptr, ptr, i32, i32, i32, i64, i64, f32, f32, f32, f32, f32, i32, ptr],
        "zp_xielu": [ptr, ptr, i64, f32, f32, i32, ptr],
        "zp_relu_square": [ptr, ptr, i64, i32, ptr],
        "zp_softcap": [ptr, ptr, i64, f32, i32, ptr],
        "zp_gather_rows": [ptr, ptr, ptr, i32, i32, i64, ptr],
        "zp_run_attention": [ptr, ptr, ptr, ptr, ptr, ptr, ptr, form_ptr, i32, i32, i32, i32, i32, i32, i32, i32, i64,
                             i64, i64, i64, i64, i64, f32, f32, i32, ptr],
    }, {}),
    "latent": ({
        "zp_latent_norm_store": [ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i64,
                                 f32, i32, ptr],
        "zp_rotate_heads": [ptr, ptr, ptr, i32, i32, i32, i32, i32, i64, i32, ptr],
        "zp_headwise_linear": [ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, ptr],
        "zp_latent_rows_attention": [ptr, ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i32, i32, f32,
                                     i32, ptr, i64, ptr],
    }, {"zp_latent_rows_workspace": [i32, i32, i32, i32, i32, i32, i32]}),
    "grouped": ({
        "zp_rotary_store": [ptr, ptr, ptr, ptr, C.POINTER(StoreForm), ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i64,
                            i64, i32, ptr],
        "zp_grouped_rows_attention": [ptr, ptr, ptr, ptr, ptr, ptr, form_ptr, ptr, i32, i32, i32, i32, i32, i32, i32,
                                      i32, i32, i32, i32, i64, f32, f32, i32, ptr, i64, ptr],
    }, {"zp_grouped_rows_workspace": [i32, i32, i32, i32, i32, i32, i32, i32, i32, i32, i32]}),
    "recurrent": ({
        "zp_mlstm_scan": [C.POINTER(MlstmArgs), i32, ptr],
        "zp_mlstm_runs": [C.POINTER(MlstmArgs), i32, i32, ptr, i64, i32, ptr],
        "zp_delta_scan": [C.POINTER(DeltaArgs), i32, ptr],
        "zp_delta_runs": [C.POINTER(DeltaArgs), i32, i32, ptr, i64, i32, ptr],
    }, {"zp_mlstm_runs_workspace": [i32, i32, i32], "zp_delta_runs_workspace": [i32, i32, i32, i32, i32]}),
    "linear": ({
        "zp_linear_scan": [C.POINTER(LinearArgs), i32, ptr],
        "zp_linear_runs": [C.POINTER(LinearArgs), i32, i32, ptr, i64, i32, ptr],
    }, {"zp_linear_runs_workspace": [i32, i32, i32, i32]}),
    "moe": ({
        "zp_small_linear": [ptr, ptr, ptr, i32, i32, i32, i64, i32, ptr],
        "zp_moe_select": [ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, ptr],
        "zp_moe_plan": [ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, ptr, i64, ptr],
        "zp_moe_gate_up": [ptr, ptr, ptr, ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i32, i32, i64,
                           i64, i32, f32, f32, i32, ptr],
        "zp_moe_down": [ptr, ptr, ptr, ptr, ptr, ptr, ptr, i32, i32, i32, i32, i32, i32, i32, i32, i32, i64, i64, i32,
                        ptr],
    }, {"zp_moe_tile_rows": [i32, i32, i32, i32], "zp_moe_max_tiles": [i32, i32, i32, i32, i32],
        "zp_moe_plan_workspace": [i32, i32, i32]}),
}
MODEL_EXPORTS = {lib: sorted([*calls, *sizes]) for lib, (calls, sizes) in MODEL_LIBS.items()}
_LIB_OF = {name: lib for lib, (calls, _) in MODEL_LIBS.items() for name in calls}

_lib = None
_models: dict[str, C.CDLL] = {}


def _open(path: str, signatures: dict, i64_returning: dict) -> C.CDLL:
    if not os.path.exists(path):
        raise RuntimeError(
            f"{path} is missing: build it with `python -m zipage_amd.build` "
            "(there is no CPU fallback for the HIP kernels)")
    lib = C.CDLL(path)
    for name, args in signatures.items():
        fn = getattr(lib, name)
        fn.argtypes, fn.restype = args, i32
    for name, args in i64_returning.items():
        fn = getattr(lib, name)
        fn.argtypes, fn.restype = args, i64
    lib.zp_abi_version.argtypes, lib.zp_abi_version.restype = [], i32
    lib.zp_last_error.argtypes, lib.zp_last_error.restype = [], C.c_char_p
    return lib


def load() -> C.CDLL:
    """Load the compression library once and type every entry point.  Raises if absent."""
    global _lib
    if _lib is None:
        _lib = _open(LIB_PATH, SIGNATURES, I64_RETURNING)
    return _lib


def model_lib_path(name: str) -> str:
    return os.path.join(_HERE, f"libzipage_{name}.so")


def load_models(name: str = "models") -> C.CDLL:
    """The same for a model-side library."""
    if name not in _models:
        _models[name] = _open(model_lib_path(name), *MODEL_LIBS[name])
    return _models[name]


def _check(lib, name: str, rc: int) -> None:
    if rc != 0:
        raise RuntimeError(f"{name} failed ({rc}): {lib.zp_last_error().decode()}")


def call(name: str, *args) -> None:
    lib = load()
    _check(lib, name, getattr(lib, name)(*args))


def call_models(name: str, *args) -> None:
    lib = load_models(_LIB_OF[name])
    _check(lib, name, getattr(lib, name)(*args))


def dtype_tag(t: torch.Tensor) -> int:
    try:
        return _DTYPES[t.dtype]
    except KeyError:
        raise TypeError(f"unsupported cache dtype {t.dtype}; use bfloat16, float16 or float32")


def dev_ptr(t) -> int:
    if t is None:
        return 0
    if not t.is_cuda:
        raise RuntimeError("the compression kernels need device tensors (no CPU fallback)")
    return t.data_ptr()


def stream_ptr(t: torch.Tensor) -> int:
    return torch.cuda.current_stream(t.device).cuda_stream
