"""Build rules the GPU found the hard way, checked on the CPU by cross-compiling every kernel source to gfx950 assembly.

Rule 1: no packed fp32 operation (v_pk_fma_f32 / v_pk_mul_f32 / v_pk_add_f32) in any kernel.  hipcc -O3 forms them by itself from ordinary
float code, and the forms that read the high dword of a VGPR src1 pair in the low lane return wrong results while another wave of the same
SIMD issues MFMAs (profiles/r04_pkfma_probe.txt) -- parity-green and bit-stable alone, wrong beside a neighbour.  The libraries are built
with the feature off (build.FLAGS); this test compiles with the same flags and looks at what came out.

Rule 2: no scratch memory in the kernels of the language models' library.  A tile kernel whose epilogue outgrew the compiler's unrolling kept its
accumulators there -- right results, 25 us more per launch."""
import os
import re
import shutil
import subprocess
from concurrent.futures import ThreadPoolExecutor

import pytest

from ht_vllm_omni_amd import build as B

CSRC = B.CSRC
HIPCC = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"
PACKED = re.compile(r"^\s*(v_pk_(?:fma|mul|add)_f32)\b")


def _asm(name, tmp_path, defines=()):
    out = os.path.join(tmp_path, name + ".s")
    subprocess.run([HIPCC, *B.FLAGS, *B.EXTRA.get(name, []), *defines, "-S", "--cuda-device-only", os.path.join(CSRC, name), "-o", out],
                   check=True, capture_output=True, timeout=900)
    return open(out).read().split("\n")


def packed_fp32(lines):
    return [l.strip() for l in lines if PACKED.match(l)]


def scratch_bytes(lines):
    return [int(m.group(1)) for m in (re.match(r"^; ScratchSize: (\d+)", l) for l in lines) if m]


def test_the_scanner_sees_the_form():
    got = packed_fp32(["_Zk:", "\tv_pk_fma_f32 v[0:1], v[2:3], v[4:5], v[0:1] op_sel:[0,1,0]", "\tv_pk_mul_f32 v[0:1], v[2:3], v[4:5]",
                       "\tv_pk_add_f32 v[0:1], v[2:3], s[4:5]", "\tv_pk_fma_f16 v0, v1, v2, v3", "\tv_fma_f32 v0, v1, v2, v3"])
    assert len(got) == 3


def test_the_feature_is_off_in_the_flags():
    f = B.FLAGS
    i = f.index("-packed-fp32-ops")
    assert f[i - 3:i] == ["-Xclang", "-target-feature", "-Xclang"]


# both builds: the product, and the diagnostics build (-DOMNI_DEBUG_HOOKS turns the policy knobs into run-time variables: other code)
@pytest.mark.parametrize("defines", [(), ("-DOMNI_DEBUG_HOOKS",)], ids=["product", "debug-hooks"])
@pytest.mark.skipif(not os.path.exists(HIPCC), reason="no hipcc")
def test_no_kernel_holds_a_packed_fp32_op(tmp_path, defines):
    names = sorted(f for f in os.listdir(CSRC) if f.endswith(".hip"))
    with ThreadPoolExecutor(max_workers=min(8, os.cpu_count() or 1)) as pool:
        asms = list(pool.map(lambda n: _asm(n, str(tmp_path), defines), names))
    bad = [(n, x) for n, lines in zip(names, asms) for x in packed_fp32(lines)]
    assert sum(len(a) for a in asms) > 10000
    assert not bad, f"{len(bad)} packed fp32 ops, e.g. {bad[:4]}"
    if not defines:
        scratch = {n: scratch_bytes(lines) for n, lines in zip(names, asms) if n in B.DECODER_SOURCES}
        assert sum(map(len, scratch.values())) > 50
        assert not any(map(any, scratch.values())), {n: v for n, v in scratch.items() if any(v)}
