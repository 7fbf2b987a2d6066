"""C ABI of libslm_latent.so: exports match include/slm_latent.h, arguments are validated before anything is launched."""
import ctypes as C
import os
import re
import subprocess

import pytest

from scalellm_amd import _lib

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
HEADER = os.path.join(ROOT, "include", "slm_latent.h")


def _header():
    return re.sub(r"/\*.*?\*/", "", open(HEADER).read(), flags=re.S)


def test_library_exports_what_the_header_declares():
    want = set(re.findall(r"SLM_API\s+[\w\s\*]+?\b(slm_\w+)\s*\(", _header()))
    out = subprocess.check_output(["nm", "-D", "--defined-only", _lib.LATENT_LIB_PATH], text=True)
    assert set(re.findall(r"\sT\s+(slm_\w+)", out)) == want
    L = _lib.latent_lib()
    assert b"gfx950" in L.slm_latent_version() and L.slm_latent_status_string(-1) == b"invalid argument"


@pytest.mark.parametrize("name,mirror", [("slm_residual_norm_args", _lib.ResidualNormArgs), ("slm_linear_args", _lib.LinearArgs),
                                         ("slm_latent_append_args", _lib.LatentAppendArgs),
                                         ("slm_latent_attn_args", _lib.LatentAttnArgs),
                                         ("slm_latent_prefill_args", _lib.LatentPrefillArgs)])
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
            v = v.strip()
            ptr = "*" in v or base.endswith("*")
            fields.append((v.replace("*", "").strip(), C.c_void_p if ptr else kinds[base.rstrip("*")]))
    assert fields == list(mirror._fields_)


def test_invalid_arguments_come_back_as_status():
    L = _lib.latent_lib()
    assert L.slm_residual_norm(None, None) == -1
    a = _lib.LinearArgs()
    assert L.slm_linear(C.byref(a), None) == -1
    a.x = a.w = a.y = 4096
    a.M, a.N, a.K, a.ldx, a.ldw, a.ldy, a.batch, a.n_splits, a.dtype = 1, 16, 64, 64, 64, 16, 1, 1, _lib.SLM_BF16
    for field, bad, rc in (("K", 63, -1), ("N", 15, -1), ("ldx", 32, -1), ("dtype", 0, -2), ("ldw", 68, -5), ("n_splits", 2, -1),
                           ("epilogue", 9, -1)):
        keep = getattr(a, field)
        setattr(a, field, bad)
        assert L.slm_linear(C.byref(a), None) == rc, field
        setattr(a, field, keep)
    b = _lib.LatentAttnArgs()
    b.rows, b.batch, b.heads, b.c_pad, b.r_pad, b.block_size, b.dtype = 3, 1, 4, 64, 32, 16, _lib.SLM_BF16
    assert L.slm_latent_attn(C.byref(b), None) == -1          # null pointers
    b.block_size = 24
    assert L.slm_latent_attn(C.byref(b), None) == -1
    b.block_size, b.dtype = 16, 0
    assert L.slm_latent_attn(C.byref(b), None) == -2
    assert L.slm_latent_gather(None, None, None, 1, 64, None) == -1
    assert L.slm_clamped_glu(4096, 4096, 1, 6, 12, 8, 1.0, 1.0, 1.0, _lib.SLM_BF16, None) == -1
    p = _lib.LatentPrefillArgs()
    assert L.slm_latent_prefill(C.byref(p), None) == -1
    assert L.slm_latent_prefill_supported(128, 64, 128) == 1 and L.slm_latent_prefill_supported(250, 96, 128) == 0


def test_split_plan_sizes_its_workspace():
    L = _lib.latent_lib()
    b = _lib.LatentAttnArgs()
    b.rows, b.batch, b.heads, b.c_pad, b.r_pad, b.block_size, b.dtype = 2, 2, 16, 512, 64, 64, _lib.SLM_BF16
    b.max_kv_len = 4096
    many = L.slm_latent_attn_workspace_bytes(C.byref(b))
    assert many > 0
    b.window = 64                      # a window bounds the range that can be split
    assert L.slm_latent_attn_workspace_bytes(C.byref(b)) < many
    b.window, b.rows = 0, 4096
    assert L.slm_latent_attn_workspace_bytes(C.byref(b)) == 0
    b.rows, b.dtype = 2, _lib.SLM_F32
    assert L.slm_latent_attn_workspace_bytes(C.byref(b)) == 0
