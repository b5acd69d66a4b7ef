"""scripts/rocpd_sites.py: the join of the engine's launch list with a rocprofv3 kernel trace, on a synthetic trace."""
import sqlite3
import subprocess
import sys
from pathlib import Path

ROOT = Path(__file__).resolve().parent.parent


def test_sites_join_by_position(tmp_path):
    ll = [("prepare", "k_lm_prepare"), ("L.in_proj", "k_gemm_xp"), ("L.ffn_in", "k_gemm_xp"), ("L.in_proj", "k_gemm_xp"),
          ("L.ffn_in", "k_gemm_xp"), ("commit", "k_lm_commit")]
    (tmp_path / "launch_list_lm.tsv").write_text("".join(f"{s}\t{k}\n" for s, k in ll))
    db = tmp_path / "t.db"
    c = sqlite3.connect(db)
    c.execute("create table kernels (name text, start integer, end integer)")
    t = 0
    full = {"k_lm_prepare": "k_lm_prepare(TokArgs, int const*)", "k_gemm_xp": "void k_gemm_xp<32, 1, 1, 8, 4, 0>(GemmArgs)",
            "k_lm_commit": "k_lm_commit(TokArgs)"}
    for step in range(4):
        c.execute("insert into kernels values (?,?,?)", ("__amd_rocclr_fillBufferAligned", t, t + 1000)); t += 2000
        for site, k in ll:
            d = {"prepare": 5000, "L.in_proj": 20000, "L.ffn_in": 40000, "commit": 7000}[site]
            c.execute("insert into kernels values (?,?,?)", (full[k], t, t + d)); t += d + 500
    c.commit(); c.close()
    r = subprocess.run([sys.executable, str(ROOT / "scripts" / "rocpd_sites.py"), str(db), str(tmp_path)], capture_output=True, text=True)
    assert r.returncode == 0, r.stderr
    rows = {ln.split(",")[1]: ln.split(",") for ln in r.stdout.splitlines() if ln.startswith("lm,")}
    assert rows["L.in_proj"][2] == "2" and abs(float(rows["L.in_proj"][3]) - 40.0) < 1e-6 and abs(float(rows["L.in_proj"][4]) - 20.0) < 1e-6
    assert abs(float(rows["L.ffn_in"][4]) - 40.0) < 1e-6
    assert abs(float(rows["L.ffn_in"][6]) - 2 * 2 * 11264 * 4096 / 40e-6 / 1e9) < 1.0      # GB/s of the 7B shape


def test_sites_take_bytes_from_the_launch_list_and_match_per_stream(tmp_path):
    """Quantised weights: the GB/s column uses the bytes the engine recorded (third column), not the bf16 table; and a program
    is found on its own stream although another stream's kernels interleave in time (the pipelined duplex step)."""
    ll = [("prepare", "k_lm_prepare", 0), ("L.ffn_in", "k_gemm_xp", 1000000), ("commit", "k_lm_commit", 0)]
    (tmp_path / "launch_list_lm.tsv").write_text("".join(f"{s}\t{k}" + (f"\t{b}" if b else "") + "\n" for s, k, b in ll))
    db = tmp_path / "t.db"
    c = sqlite3.connect(db)
    c.execute("create table kernels (name text, start integer, end integer, stream_id integer)")
    t = 0
    for step in range(4):
        for site, k, _ in ll:
            d = {"prepare": 5000, "L.ffn_in": 10000, "commit": 7000}[site]
            c.execute("insert into kernels values (?,?,?,?)", (k + "(Args)", t, t + d, 3))
            c.execute("insert into kernels values (?,?,?,?)", ("k_conv_wide(ConvGemmArgs)", t + 100, t + 900, 4))   # another stream, overlapping
            t += d + 500
    c.commit(); c.close()
    r = subprocess.run([sys.executable, str(ROOT / "scripts" / "rocpd_sites.py"), str(db), str(tmp_path)], capture_output=True, text=True)
    assert r.returncode == 0, r.stderr
    rows = {ln.split(",")[1]: ln.split(",") for ln in r.stdout.splitlines() if ln.startswith("lm,")}
    assert abs(float(rows["L.ffn_in"][4]) - 10.0) < 1e-6 and abs(float(rows["L.ffn_in"][5]) - 1.0) < 1e-6
    assert abs(float(rows["L.ffn_in"][6]) - 100.0) < 1e-3


def test_pmc_summary_clusters_a_kernels_dispatches_by_shape(tmp_path):
    """scripts/rocpd_pmc.py --clusters: one kernel name serves several GEMM shapes; its dispatches are grouped by counter value
    (FETCH_SIZE, KiB, doubled on gfx950) - or, for cycle counters, by duration - one line per shape."""
    import sqlite3
    db = tmp_path / "pmc.db"
    c = sqlite3.connect(db)
    c.execute("create table counters_collection (kernel_name text, counter_name text, value real, duration real)")
    name = "void k_gemm_xlds<1, 64, 3, true, 0>(GemmArgs)"
    for i in range(32):
        c.execute("insert into counters_collection values (?,?,?,?)", (name, "FETCH_SIZE", 93159.0 + i % 3, 35000.0))
        c.execute("insert into counters_collection values (?,?,?,?)", (name, "FETCH_SIZE", 55626.0 + i % 3, 23000.0))
    c.execute("insert into counters_collection values (?,?,?,?)", ("k_other(int)", "FETCH_SIZE", 10.0, 5000.0))
    c.commit()
    c.close()
    script = str(ROOT / "scripts" / "rocpd_pmc.py")
    r = subprocess.run([sys.executable, script, str(db), "--header", "synthetic", "--clusters", "k_gemm_xlds"], capture_output=True, text=True)
    assert r.returncode == 0, r.stderr
    lines = r.stdout.splitlines()
    assert lines[0] == "# synthetic"
    rows = [l for l in lines[lines.index([l for l in lines if l.startswith("# clusters")][0]) + 1:] if l]
    assert len(rows) == 2 and all(row.split(",")[-4] == "32" for row in rows), rows
    big = [row for row in rows if ",93160." in row or ",93159." in row][0]
    assert abs(float(big.split(",")[-2]) - 93160.0 * 1024 * 2) < 4096          # bytes_corrected = KiB x 1024 x 2
    r = subprocess.run([sys.executable, script, str(db), "--clusters", "k_gemm_xlds", "--by-duration"], capture_output=True, text=True)
    assert r.returncode == 0 and sum(l.startswith('"k_gemm_xlds') for l in r.stdout.splitlines()) == 2


def test_built_library_has_no_in_place_cross_swizzled_packed_fp32_instruction():
    """The instruction form that stood in k_gemm_xp's RoPE epilogue when its output was not reproducible (round 4's driver failure;
    HISTORY.md round 5 10a: `v_pk_mul_f32 v[14:15], v[30:31], v[14:15] op_sel:[0,1] op_sel_hi:[1,0]`) must not come back through a
    compiler update or a new epilogue: the gfx950 code objects of the library `build()` produced are disassembled and scanned
    (scripts/isa_scan_packed_swizzle.py).  The build also switches packed fp32 math off altogether (moshi_amd/build.py)."""
    import subprocess
    import sys
    from pathlib import Path
    root = Path(__file__).resolve().parent.parent
    lib = root / "moshi_amd" / "libmoshi_mi.so"
    if not lib.exists():
        import pytest
        pytest.skip("the HIP library is not built")
    r = subprocess.run([sys.executable, str(root / "scripts" / "isa_scan_packed_swizzle.py"), str(lib)], capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr
    assert r.stdout.strip().splitlines()[-1].startswith("0 kernel(s)"), r.stdout[-2000:]
