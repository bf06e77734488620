"""The C-ABI library loads and exports every symbol include/zipage_hip.h declares.
No compute calls: this runs without a GPU."""
import ctypes
import os
import re

import pytest

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _declared(header="zipage_hip.h"):
    text = open(os.path.join(ROOT, "include", header)).read()
    text = re.sub(r"/\*.*?\*/", "", text, flags=re.S)
    return sorted(set(re.findall(r"\b(zp_[a-z_0-9]+)\s*\(", text)))


def test_header_declares_expected_entry_points():
    names = _declared()
    for n in ["zp_store_query", "zp_attention_score", "zp_global_score", "zp_pool_scores",
              "zp_key_norm", "zp_redundancy_lightning", "zp_redundancy_raw", "zp_score_epilogue",
              "zp_topk_mask", "zp_compress_kv", "zp_compress_score", "zp_last_error",
              "zp_abi_version"]:
        assert n in names


def test_library_exports_every_declared_symbol():
    from zipage_amd import _lib
    if not os.path.exists(_lib.LIB_PATH):
        pytest.fail(f"{_lib.LIB_PATH} not built (python -m zipage_amd.build)")
    lib = ctypes.CDLL(_lib.LIB_PATH)
    for name in _declared():
        assert hasattr(lib, name), f"{name} declared in the header but not exported"
    assert sorted(_lib.EXPORTS) == _declared()


def test_models_library_exports_every_declared_symbol():
    from zipage_amd import _lib
    names = _declared("zipage_models.h")
    assert sorted(n for names in _lib.MODEL_EXPORTS.values() for n in names) == names
    for part, exported in _lib.MODEL_EXPORTS.items():
        lib = _lib.load_models(part)
        for name in exported:
            assert hasattr(lib, name), f"{name} declared in the header but not exported"
    lib = _lib.load_models("latent")
    # bad arguments are refused on the host, before any launch
    assert lib.zp_headwise_linear(None, None, None, None, None, 1, 2, 33, 16, 0, 0, 0, None) != 0
    assert b"multiples of 32" in lib.zp_last_error()
    assert lib.zp_latent_rows_attention(None, None, None, None, None, None, 1, 1, 32, 0, 16, 1, 1, 1, -1, 1.0, 0,
                                        None, 0, None) == 1
    lib = _lib.load_models("models")
    assert lib.zp_embed_norm(None, None, None, None, None, None, None, None, None, None, 1, 12, 12, 5, 5, 1.0, 1e-6, 0.0, 0.0, 0, None) != 0
    assert lib.zp_run_attention(None, None, None, None, None, None, None, None, 1, 4, 3, 32, 0, 32, 0, 0, 1, 1, 128, 256, 0,
                                128, 1.0, 1.0, 0, None) == 1
    lib = _lib.load_models("grouped")
    two = _lib.AttentionForm(0.0, 2, 0.5, 1e-6, 0, None, 0)                              # a mean over nothing
    assert lib.zp_grouped_rows_attention(1, 1, 1, 1, 1, None, ctypes.byref(two), 1, 1, 2, 2, 32, 32, 16, 1, 1, 1, 0, 0,
                                         64, 1.0, 1.0, 0, None, 0, None) == 1
    assert b"mean over the values" in lib.zp_last_error()
    lib = _lib.load_models("moe")
    assert lib.zp_moe_select(None, None, None, None, 1, 12, 5, 3, 1, 0, 12, None) == 1      # five of a group of four
    assert lib.zp_small_linear(None, None, None, 1, 40, 4, 40, 0, None) != 0
    lib = _lib.load_models("recurrent")
    bad = _lib.MlstmArgs(heads=2, dk=48, dv=32, vdim=32, cap=1.0, gate_stride=4, out_stride=64,
                         seg=_lib.Segments(n=1, num_slots=1, num_rows=1))
    assert lib.zp_mlstm_scan(ctypes.byref(bad), 0, None) != 0 and b"48" in lib.zp_last_error()
    bad = _lib.DeltaArgs(heads=3, kv_heads=2, dk=32, dv=32, vdim=32, taps=4, out_stride=96,
                         seg=_lib.Segments(n=1, num_slots=1, num_rows=1))
    assert lib.zp_delta_scan(ctypes.byref(bad), 0, None) == 1
    lib = _lib.load_models("linear")
    bad = _lib.LinearArgs(heads=2, dk=48, dv=32, vdim=32, in_stride=512, out_stride=64, seg=_lib.Segments(n=1, num_slots=1, num_rows=1))
    assert lib.zp_linear_scan(ctypes.byref(bad), 0, None) != 0 and b"48" in lib.zp_last_error()
    bad.dk, bad.rot = 32, 34                                                             # more than a head has
    assert lib.zp_linear_runs(ctypes.byref(bad), 0, 16, None, 0, 0, None) == 1


def test_version_and_error_string():
    from zipage_amd import _lib
    lib = _lib.load()
    assert lib.zp_abi_version() >= 2
    assert isinstance(lib.zp_last_error(), bytes)


def test_argument_validation_needs_no_gpu():
    """Bad arguments are rejected on the host before any launch."""
    from zipage_amd import _lib
    lib = _lib.load()
    rc = lib.zp_topk_mask(None, None, 4, 16, 17, 0, None)
    assert rc == 1 and b"k=17" in lib.zp_last_error()
    rc = lib.zp_global_score(1, 1, 1, 1, 1, 1, 1, 256, 8, 4, 0, 0, 1.5, 0, 1, 0, None)
    assert rc == 1 and b"decay_factor" in lib.zp_last_error()


def test_product_has_no_cpu_fallback():
    import torch
    from zipage_amd.kernel import topk_mask
    with pytest.raises(RuntimeError, match="device tensors"):
        topk_mask(torch.zeros(2, 8), 3)
