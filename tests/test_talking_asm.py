"""Kernels that keep their accumulators in named AGPRs through inline assembly: the
compiler must use no AGPR of its own there (it takes them for free between the asm
statements, and a value it parked in one would be overwritten), and every read of an
accumulator must stand behind the padding that covers the last MFMA. Checked in the
assembly built here."""
import re
import shutil
import subprocess
from pathlib import Path

import pytest

from kgs.utils import build

HIPCC = "/opt/rocm/bin/hipcc"

pytestmark = pytest.mark.skipif(not Path(HIPCC).exists() and shutil.which("hipcc") is None,
                                reason="hipcc not available")


def assembly(src: str, tmp_path) -> dict[str, list[str]]:
    """Function -> its lines, comments that mark inline assembly kept."""
    t = next(t for t in build.targets() if t.name == "kernels")
    out = tmp_path / (src + ".s")
    cmd = [t.compiler, *t.flags, *t.source_flags.get(src, []), "-S", "--offload-device-only",
           str(build.NATIVE / "kernels" / src), "-o", str(out)]
    r = subprocess.run(cmd, capture_output=True, text=True, timeout=500)
    assert r.returncode == 0, r.stderr[-2000:]
    res, name = {}, None
    for ln in out.read_text().splitlines():
        m = re.match(r"^(_Z\w+):", ln)
        if m:
            name = m.group(1)
            res[name] = []
        elif name:
            res[name].append(ln)
    return res


def faults(lines: list[str]) -> list[str]:
    asm, bad, since = False, [], 99
    for ln in lines:
        if "ASMSTART" in ln or "ASMEND" in ln:
            asm = "ASMSTART" in ln
            continue
        t = ln.split(";")[0].strip()
        if not t or t.startswith("."):
            continue
        if not asm and re.search(r"\ba\d+\b|\ba\[\d|accvgpr", t):
            bad.append("outside: " + t)
        if "scratch_" in t:
            bad.append(t)
        if t.startswith("v_mfma") and re.match(r"v_mfma\S+ a\[", t):
            since = 0
        elif t.startswith("s_nop"):
            since += int(t.split()[1], 0) + 1
        elif t.startswith("v_accvgpr_read") and since < 18:
            bad.append("unpadded: " + t)
        else:
            since += 1
    return bad


def test_scan_sees_faults():
    ok = [" ;;#ASMSTART", " v_mfma_f32_16x16x32_bf16 a[0:3], v[0:3], v[4:7], a[0:3]", " s_nop 7", " s_nop 7", " s_nop 3",
          " v_accvgpr_read_b32 v0, a0", " ;;#ASMEND", " v_add_f32_e32 v0, v0, v1"]
    assert not faults(ok)
    assert faults(ok[:2] + ok[3:]) and faults(ok + [" v_accvgpr_write_b32 a9, v3"]) and faults([" scratch_load_dword v1, off"])


@pytest.mark.parametrize("src,kernel,count", [("talking.hip", "attn_tiles", 12), ("moe.hip", "groupedILi", 5)])
def test_accumulators_are_left_alone(src, kernel, count, tmp_path):
    fns = {n: b for n, b in assembly(src, tmp_path).items() if kernel in n}
    assert len(fns) == count, sorted(fns)
    for name, body in fns.items():
        assert not faults(body), (name, faults(body)[:5])
