"""C ABI of libslm_mixers.so: exports match include/slm_mixers.h, arguments are validated before anything is launched."""
import ctypes as C
import os
import re
import subprocess

import pytest

from scalellm_amd import _lib

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
HEADER = os.path.join(ROOT, "include", "slm_mixers.h")


def _header():
    return re.sub(r"/\*.*?\*/", "", open(HEADER).read(), flags=re.S)


def test_library_exports_what_the_header_declares():
    want = set(re.findall(r"SLM_API\s+[\w\s\*]+?\b(slm_\w+)\s*\(", _header()))
    out = subprocess.check_output(["nm", "-D", "--defined-only", _lib.MIXERS_LIB_PATH], text=True)
    assert set(re.findall(r"\sT\s+(slm_\w+)", out)) == want
    L = _lib.mixers_lib()
    assert b"gfx950" in L.slm_mixers_version() and L.slm_mixers_status_string(-1) == b"invalid argument"


@pytest.mark.parametrize("name,mirror", [("slm_recurrent_args", _lib.RecurrentArgs), ("slm_gated_norm_args", _lib.GatedNormArgs),
                                         ("slm_window_append_args", _lib.WindowAppendArgs), ("slm_window_attn_args", _lib.WindowAttnArgs),
                                         ("slm_window_prefill_args", _lib.WindowPrefillArgs)])
def test_ctypes_mirrors_have_the_header_layout(name, mirror):
    body = re.search(r"typedef struct %s \{(.*?)\} %s;" % (name, name), _header(), flags=re.S).group(1)
    kinds = {"int64_t": C.c_int64, "int32_t": C.c_int32, "float": C.c_float, "size_t": C.c_size_t}
    fields = []
    for decl in body.split(";"):
        decl = " ".join(decl.split()).replace("const ", "")
        if not decl:
            continue
        base, rest = decl.split(" ", 1) if "*" not in decl.split(" ")[0] else (decl.split("*")[0], "*" + decl.split("*", 1)[1])
        for v in rest.split(","):
            ptr = "*" in v or base.endswith("*")
            fields.append((v.replace("*", "").strip(), C.c_void_p if ptr else kinds[base.rstrip("*")]))
    assert fields == list(mirror._fields_)


def test_invalid_arguments_come_back_as_status():
    L = _lib.mixers_lib()
    assert [L.slm_recurrent_dim_pad(d) for d in (0, 1, 33, 65, 129, 256, 257)] == [0, 32, 64, 128, 192, 256, 0]
    for fn, args in ((L.slm_recurrent_step, _lib.RecurrentArgs), (L.slm_recurrent_prepare, _lib.RecurrentArgs),
                     (L.slm_recurrent_scan, _lib.RecurrentArgs), (L.slm_gated_norm, _lib.GatedNormArgs),
                     (L.slm_window_append, _lib.WindowAppendArgs), (L.slm_window_attn, _lib.WindowAttnArgs)):
        assert fn(None, None) == -1 and fn(C.byref(args()), None) == -1
    p = _lib.WindowPrefillArgs()
    assert L.slm_window_prefill(C.byref(p), None) == -1
    assert L.slm_window_prefill_supported(128, 96) == 1 and L.slm_window_prefill_supported(160, 128) == 0
    a = _lib.RecurrentArgs()
    for name in "proj state positions q_cu state_slots decay o".split():
        setattr(a, name, 4096)
    a.mode, a.dtype, a.batch, a.rows, a.heads, a.qk_heads, a.dim, a.vdim, a.dim_pad, a.v_pad = _lib.REC_LIGHTNING, _lib.SLM_BF16, 1, 0, 4, 4, 20, 20, 32, 32
    assert L.slm_recurrent_step(C.byref(a), None) == 0          # (no single rows: nothing is launched)
    for field, bad in (("qk_heads", 3), ("dim_pad", 64), ("v_pad", 20), ("v_pad", 272), ("mode", 2), ("dtype", 0), ("n_single", 2), ("decay", None)):
        keep = getattr(a, field)
        setattr(a, field, bad)
        assert L.slm_recurrent_step(C.byref(a), None) == -1, field
        setattr(a, field, keep)


def test_split_plan_sizes_its_workspace():
    L = _lib.mixers_lib()
    b = _lib.WindowAttnArgs()
    for name in "q key_cache value_cache out positions q_cu block_table block_cu".split():
        setattr(b, name, 4096)
    b.rows, b.batch, b.heads, b.kv_heads, b.d_pad, b.v_pad, b.block_size, b.dtype = 2, 2, 16, 4, 128, 128, 64, _lib.SLM_BF16
    b.max_kv_len = 4096
    many = L.slm_window_attn_workspace_bytes(C.byref(b))
    assert many > 0
    b.window = 256                     # a window bounds the range that can be split
    assert 0 < L.slm_window_attn_workspace_bytes(C.byref(b)) < many
    b.window = 64
    assert L.slm_window_attn_workspace_bytes(C.byref(b)) == 0
    b.window, b.dtype = 0, _lib.SLM_F32
    assert L.slm_window_attn_workspace_bytes(C.byref(b)) == 0
