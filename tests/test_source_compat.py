"""Source drop-in check: the reference's own programs compile against include/turboinfer/**.

the reference's benchmarks/benchmark_inference.cpp and
tests/test_tensor_engine.cpp (and every other test / benchmark / example program of the
reference) are compiled, unmodified, against this repository's headers; three of them are also
linked against the in-tree libturboinfer_amd.so (undefined symbols would fail the link).  Only
the profiler test is expected to fail: util/profiler.hpp is out of scope.

CPU only; skipped where /root/reference holds no sources (the GPU box).  Binary drop-in (VERDICT r4 item
7): the public classes have the reference's layout (tests/cpp/layout/layout_probe.cpp, compiled
against both header sets, prints identical sizes and offsets), and the reference's
tests/test_inference_engine.cpp compiled against the REFERENCE's headers links against this
library; that binary (tests/cpp/bin/ref_test_inference_engine) runs on the GPU in
tests/test_cpp_api.py::test_reference_built_program_runs_against_our_library.
"""
import os
import pathlib
import shutil
import subprocess
from concurrent.futures import ThreadPoolExecutor

import pytest

REPO = pathlib.Path(__file__).resolve().parents[1]
REF = pathlib.Path("/root/reference")
LIB = REPO / "turboinfer_amd" / "lib" / "libturboinfer_amd.so"
OUT_OF_SCOPE = {"test_profiler_fixed.cpp"}   # includes turboinfer/util/profiler.hpp

pytestmark = pytest.mark.skipif(not (REF / "include").is_dir() or shutil.which("g++") is None,
                                reason="needs the reference sources and g++ (build container only)")


def _programs():
    progs = []
    for sub in ("tests", "benchmarks", "examples"):
        progs += sorted((REF / sub).glob("*.cpp"))
    return progs


def _syntax(path):
    r = subprocess.run(["g++", "-std=c++20", "-fsyntax-only", f"-I{REPO / 'include'}", str(path)],
                       capture_output=True, text=True, timeout=300)
    return path.name, r.returncode, r.stderr


def test_reference_programs_compile_against_our_headers():
    progs = _programs()
    assert len(progs) > 30
    with ThreadPoolExecutor(max_workers=min(8, os.cpu_count() or 1)) as ex:
        results = list(ex.map(_syntax, progs))
    failed = {name: err.splitlines()[:3] for name, rc, err in results if rc != 0}
    assert set(failed) == OUT_OF_SCOPE, failed


@pytest.mark.parametrize("rel", ["benchmarks/benchmark_inference.cpp", "tests/test_tensor_engine.cpp",
                                 "tests/test_inference_engine.cpp"])
def test_reference_programs_link_against_our_library(rel, tmp_path):
    if not LIB.exists():
        pytest.skip("libturboinfer_amd.so not built")
    out = tmp_path / "prog"
    r = subprocess.run(["g++", "-std=c++20", "-O0", f"-I{REPO / 'include'}", str(REF / rel), "-o", str(out),
                        f"-L{LIB.parent}", "-lturboinfer_amd"], capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]


def test_public_layouts_match_reference(tmp_path):
    outs = []
    for inc in (REF / "include", REPO / "include"):
        exe = tmp_path / f"layout_{len(outs)}"
        r = subprocess.run(["g++", "-std=c++20", "-Wno-invalid-offsetof", f"-I{inc}",
                            str(REPO / "tests" / "cpp" / "layout" / "layout_probe.cpp"), "-o", str(exe)],
                           capture_output=True, text=True, timeout=300)
        assert r.returncode == 0, r.stderr[-2000:]
        outs.append(subprocess.run([str(exe)], capture_output=True, text=True, timeout=60, check=True).stdout)
    assert "InferenceEngine" in outs[0] and outs[0] == outs[1], (outs[0], outs[1])


def test_reference_header_build_links_against_our_library():
    """test_inference_engine.cpp built against the reference's own headers, linked against
    libturboinfer_amd.so: the binary the GPU test runs (kept in tests/cpp/bin, git-ignored)."""
    if not LIB.exists():
        pytest.skip("libturboinfer_amd.so not built")
    out = REPO / "tests" / "cpp" / "bin" / "ref_test_inference_engine"
    out.parent.mkdir(parents=True, exist_ok=True)
    r = subprocess.run(["g++", "-std=c++20", "-O1", f"-I{REF / 'include'}", str(REF / "tests" / "test_inference_engine.cpp"),
                        "-o", str(out), f"-L{LIB.parent}", "-lturboinfer_amd",
                        "-Wl,-rpath,$ORIGIN/../../../turboinfer_amd/lib"], capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
