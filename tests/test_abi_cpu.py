"""CPU-only checks of the C-ABI library: it loads, exports every symbol the header declares, the
ctypes table matches the header, and argument validation fails loudly without touching a GPU."""
import ctypes as C
import os
import re

import pytest

from msa_amd import _lib

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def _declared(header="msa_amd.h"):
    text = open(os.path.join(ROOT, "include", header)).read()
    text = re.sub(r"/\*.*?\*/", "", text, flags=re.S)
    return sorted(set(re.findall(r"\b(msa_[a-z0-9_]+)\s*\(", text)))


def test_header_symbols_exported_and_bound():
    lib = _lib.load()
    names = _declared()
    assert len(names) >= 16
    for n in names:
        assert hasattr(lib, n), f"{n} declared in the header but not exported"
    assert sorted(_lib.SIGNATURES) == names
    assert lib.msa_abi_version() == 1


def test_seq_header_symbols_exported_and_bound():
    lib = _lib.load_seq()
    names = _declared("msa_seq.h")
    assert len(names) >= 12
    for n in names + list(_lib.SEQ_SHARED):
        assert hasattr(lib, n), f"{n} not exported"
    assert sorted(_lib.SEQ_SIGNATURES) == names
    assert lib.msa_abi_version() == 1


@pytest.mark.parametrize("header,table", [("msa_amd.h", _lib.SIGNATURES), ("msa_seq.h", _lib.SEQ_SIGNATURES)])
def test_header_arity_matches_ctypes_table(header, table):
    text = open(os.path.join(ROOT, "include", header)).read()
    text = re.sub(r"/\*.*?\*/", "", text, flags=re.S)
    for name, (_, args) in table.items():
        m = re.search(r"\b%s\s*\(([^;]*?)\)\s*;" % name, text, flags=re.S)
        assert m, name
        params = m.group(1).strip()
        n = 0 if params in ("", "void") else len(params.split(","))
        assert n == len(args), f"{name}: header has {n} parameters, ctypes table {len(args)}"


def test_seq_structures_match_the_header(tmp_path):
    """Sizes and field offsets of the structures handed over by pointer, against the host compiler's."""
    import subprocess
    structs = {"msa_seq_batch": _lib.SeqBatch, "msa_dyn_tanh": _lib.DynTanh, "msa_rows_args": _lib.RowsArgs,
               "msa_qk_rope_args": _lib.QKRopeArgs, "msa_kv_attn_args": _lib.KVAttnArgs, "msa_delta_args": _lib.DeltaArgs}
    src = ['#include <stdio.h>', '#include "msa_seq.h"', "int main() {"]
    for c_name, py in structs.items():
        src.append(f'printf("{c_name} %zu\\n", sizeof({c_name}));')
        src += [f'printf("{c_name}.{f[0]} %zu\\n", offsetof({c_name}, {f[0]}));' for f in py._fields_]
    src.append("return 0; }")
    (tmp_path / "s.c").write_text("\n".join(src))
    subprocess.run(["gcc", "-I", os.path.join(ROOT, "include"), str(tmp_path / "s.c"), "-o", str(tmp_path / "s")], check=True)
    got = dict(l.split() for l in subprocess.run([str(tmp_path / "s")], check=True, capture_output=True, text=True).stdout.splitlines())
    for c_name, py in structs.items():
        assert int(got[c_name]) == C.sizeof(py), c_name
        for f in py._fields_:
            assert int(got[f"{c_name}.{f[0]}"]) == getattr(py, f[0]).offset, f"{c_name}.{f[0]}"


def test_seq_validation_errors_without_gpu():
    lib = _lib.load_seq()
    a = _lib.RowsArgs()
    assert lib.msa_rows_linear(C.byref(a), 0, None) == -1
    a.x = a.w = a.out = 4096
    a.M, a.N, a.K, a.groups, a.n_b, a.x_stride, a.out_stride = 17, 16, 64, 1, 16, 64, 16
    assert lib.msa_rows_linear(C.byref(a), 0, None) == -1 and b"M=17" in lib.msa_last_error()
    a.M, a.K, a.x_stride = 16, 60, 64
    assert lib.msa_rows_linear(C.byref(a), 0, None) == -1 and b"multiple of 8" in lib.msa_last_error()
    a.K, a.n_b = 64, 8
    assert lib.msa_rows_linear(C.byref(a), 0, None) == -1 and b"second operand" in lib.msa_last_error()
    assert lib.msa_seq_softcap(None, 0, 1, 0.0, None, None) == -1
    b = _lib.SeqBatch(4096, 4096, 4096, 4096, 1, 4, 4, 0)
    flash = lambda H, G, D, chunk: lib.msa_seq_flash(4096, 96, 4096, 96, 4096, 96, 4096, 4096, 1.0, 0, H, G, D, 96, chunk, None, 0, 4096, C.byref(b), None)
    assert flash(1, 1, 300, 0) == -1 and b"D=300" in lib.msa_last_error()
    assert flash(3, 2, 96, 0) == -1 and b"3 heads over 2" in lib.msa_last_error()
    assert flash(1, 1, 96, -1) == -1 and b"chunk" in lib.msa_last_error()
    kv = _lib.KVAttnArgs(4096, 4096, 4096, None, 4096, 64, 0, 65, 4, 2, 64, 64, 0, 1.0)
    assert lib.msa_seq_kv_decode(C.byref(kv), C.byref(b), None, 0, None) == -1 and b"65 keys" in lib.msa_last_error()
    kv.max_keys, kv.D = 64, 60
    assert lib.msa_seq_kv_decode(C.byref(kv), C.byref(b), None, 0, None) == -1 and b"D=60" in lib.msa_last_error()
    rope = _lib.QKRopeArgs(4096, None, None, 128, 0, 0, 4096, None, 4096, 4096, None, None, 0, 2, 1, 64, 64, 33, 1e-5)
    assert lib.msa_seq_qk_rope_append(C.byref(rope), 0, C.byref(b), None) == -1 and b"33 pairs" in lib.msa_last_error()
    d = _lib.DeltaArgs(4096, 4096, 4096, 4096, 192, 64, 1, 64, 4096, 4096, 4096, 4096, 4096, 1, 1, 64, 64, 1e-5, 0)
    size = lambda rows: lib.msa_seq_delta_chunked_workspace_bytes(C.byref(d), rows, 1)
    assert size(640) == 10 * size(64) > 0 and size(64 * 23) == 24 * size(64)          # (two segments of twelve chunks)
    d.H = d.G = 64
    assert size(1 << 20) <= 2 * (88 << 20)                                             # long portions take no more
    d.H = d.G = 1
    assert lib.msa_seq_delta_chunked(C.byref(d), C.byref(b), 4096, 16, None) == -3 and b"workspace" in lib.msa_last_error()
    d.D = 520
    assert lib.msa_seq_delta_scan(C.byref(d), 0, C.byref(b), None) == -1 and b"D=520" in lib.msa_last_error()
    a.K, a.n_b, a.N, a.M = 64, 15, 15, 4
    assert lib.msa_rows_linear(C.byref(a), 5, None) == -1 and b"gated unit" in lib.msa_last_error()
    assert lib.msa_seq_min_gru(4096, 96, 4096, 4096, 0, 32, 4096, 4096, C.byref(_lib.SeqBatch(4096, 4096, 4096, 4096, 1, 999, 999, 0)),
                               None, 0, None) == -3 and b"workspace" in lib.msa_last_error()


def test_validation_errors_without_gpu():
    lib = _lib.load()
    # wrong head dim
    rc = lib.msa_pool_chunks(None, None, None, 0, 10, 8, 64, None, None, None, 1, None, None, None, 0, 0, 0, None,
                             None, None, None)
    assert rc == -1 and b"head dim" in lib.msa_last_error()
    # null bank
    rc = lib.msa_route_topk(None, 0, None, None, 1, 1, 32, 0, 1.0, 16, C.c_void_p(8), C.c_void_p(8), None, None, 0,
                            None)
    assert rc == -1 and b"null bank" in lib.msa_last_error()
    rc = lib.msa_route_topk(None, 0, None, None, 1, 1, 32, 0, 1.0, 65, C.c_void_p(8), C.c_void_p(8), None, None, 0,
                            None)
    assert rc == -1 and b"topk" in lib.msa_last_error()
    # bank tables that do not add up are rejected before any device call
    off = (C.c_int32 * 3)(0, 2, 5)
    gid = (C.c_int64 * 2)(7, 9)
    h = C.c_void_p()
    rc = lib.msa_bank_create(C.byref(h), 1, 6, 8, 128, 0, C.addressof(off), C.addressof(gid), 2)
    assert rc == -1 and b"doc_chunk_off" in lib.msa_last_error()
    assert lib.msa_route_workspace_bytes(16, 128, 32, 8, 128, 1000, 50, 16) > 16 * 128 * 1024 * 2
    assert lib.msa_attn_workspace_bytes(4, 32, 8, 128, 1000) > 0
    # many query rows: one pass over the keys, so the workspace stays linear in the rows
    assert lib.msa_attn_workspace_bytes(65536, 32, 8, 128, 4400) < 2 * 65536 * 32 * 130 * 4
    with pytest.raises(TypeError):
        import torch
        _lib.dtype_code(torch.float16)


def test_product_does_not_import_oracle():
    """Nothing under msa_amd/ may reach into oracle/."""
    pkg = os.path.join(ROOT, "msa_amd")
    for dirpath, _, files in os.walk(pkg):
        for f in files:
            if f.endswith((".py", ".hip", ".h", ".cpp")):
                src = open(os.path.join(dirpath, f)).read()
                assert "oracle" not in src.replace("ORACLE", ""), f"{f} mentions the oracle"


@pytest.mark.parametrize("tiles_m,tiles_n,grid,copy_wg,pool_n", [
    (8, 6271, 256, 1, 783), (8, 6271, 256, 0, 783), (8, 6271, 256, 1, 0),      # the 100M-token bank, B = 16 x 128
    (16, 628, 256, 0, 78), (16, 628, 256, 1, 0),                                # the 10M-token bank, B = 32 x 128
    (1, 40, 256, 0, 0), (2, 3, 16, 1, 0), (3, 100, 64, 1, 12), (11, 37, 256, 0, 4), (11, 37, 24, 1, 18),
    (20, 999, 248, 1, 124), (256, 628, 256, 0, 78), (9, 5, 1024, 1, 0), (5, 1, 16, 0, 0), (7, 200, 16, 1, 25),
])
def test_scan_tile_order_covers_every_tile_once(tiles_m, tiles_n, grid, copy_wg, pool_n):
    """The persistent scan's tile order (fixed shares per XCD walked by an incremental cursor, then the pool):
    every tile exactly once, for grids with and without the copying workgroup and with and without a pool."""
    lib = _lib.load()
    visits = (C.c_int32 * (tiles_m * tiles_n))()
    rc = lib.msa_diag_scan_walk(tiles_m, tiles_n, grid, copy_wg, pool_n, C.addressof(visits))
    assert rc == 0, lib.msa_last_error()
    v = list(visits)
    assert min(v) == 1 and max(v) == 1, f"{v.count(0)} tiles unvisited, {sum(1 for x in v if x > 1)} visited twice"


def test_tile_pool_switch_is_exported():
    lib = _lib.load()
    assert lib.msa_route_set_tile_pool(0) == 0
    assert lib.msa_route_set_tile_pool(1) == 0


def test_build_guard_flags_compiler_code_in_the_asm_statements_registers():
    """The build checks the device assembly of the hand-scheduled scan: code the compiler generated for it (outside
    the inline-asm regions) must stay below v128, leave the accumulation registers alone and use no scratch."""
    from msa_amd import build as B
    ok = """
_ZN12_GLOBAL__N_118score_scan4_kernelILb1EEEvPKt:
	v_add_u32_e32 v5, v4, v3
	;;#ASMSTART
	v_mfma_f32_32x32x16_bf16 a[0:15], v[128:131], v[144:147], a[0:15]
	;;#ASMEND
	s_endpgm
"""
    assert B.check_kernel_contracts(ok, "score_scan4_kernel", max_compiler_vgpr=127, no_agpr=True) == []
    bad = ok.replace("v_add_u32_e32 v5, v4, v3", "v_accvgpr_write_b32 a3, v7\n\tv_mov_b32_e32 v130, v2\n\tscratch_store_dword off, v1, s32")
    problems = B.check_kernel_contracts(bad, "score_scan4_kernel", max_compiler_vgpr=127, no_agpr=True)
    assert len(problems) == 3, problems
    assert B.check_kernel_contracts(ok, "no_such_kernel") != []


def test_build_guard_fails_on_a_forced_spill():
    """With the compiler's share of the scan kernel's registers cut to 24 the kernel spills, and the check that
    build() runs on the device assembly reports it (this compiles route_score.hip once: about 15 s)."""
    from msa_amd import build as B
    src = open(os.path.join(B.CSRC, "route_score.hip")).read()
    assert "constexpr int kScan4CompilerVgprs = 128;" in src
    tmp = os.path.join(B.CSRC, "_guard_probe.hip")            # beside the sources: it includes its neighbours
    try:
        open(tmp, "w").write(src.replace("constexpr int kScan4CompilerVgprs = 128;", "constexpr int kScan4CompilerVgprs = 24;"))
        asm = B._device_asm(tmp)
    finally:
        if os.path.exists(tmp):
            os.remove(tmp)
    problems = B.check_kernel_contracts(asm, "score_scan4_kernel", max_compiler_vgpr=127, no_agpr=True)
    assert problems, "a spilling build passed the check"
    assert any("spill" in p or "scratch" in p or "private_segment" in p or "accumulation" in p for p in problems), problems[:5]


@pytest.mark.parametrize("gen", ["gen_scan_asm.py", "gen_flash_asm.py"])
def test_generated_asm_includes_are_what_their_generators_emit(gen):
    """The committed scan_asm.inc / flash_asm.inc are the generators' output (the build refuses a stale one too)."""
    import subprocess
    import sys
    csrc = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "msa_amd", "csrc")
    assert subprocess.run([sys.executable, os.path.join(csrc, gen), "--check"]).returncode == 0


def test_build_guard_covers_the_wide_flash_kernel():
    from msa_amd import build
    names = [k for k, _ in build.CONTRACTS["flash_attn.hip"]]
    assert "flash_wide_kernel" in names and "flash_attn_kernel" in names
    rules = dict(build.CONTRACTS["flash_attn.hip"])["flash_wide_kernel"]
    assert rules == {"max_compiler_vgpr": 55, "no_agpr": True}
