"""The latent-attention kernel issues its LDS reads in inline assembly, ahead of their
use, and waits for them by count. The compiler takes their registers for written
at the issue, so nothing may touch one between the read and the wait that covers
it (a copy there would move stale data). Checked in the assembly built here."""
import re
import shutil
import subprocess
from pathlib import Path

import pytest

ROOT = Path(__file__).resolve().parents[1]
HIPCC = "/opt/rocm/bin/hipcc"

pytestmark = pytest.mark.skipif(not Path(HIPCC).exists() and shutil.which("hipcc") is None,
                                reason="hipcc not available")


def _regs(text: str) -> set[int]:
    out = set()
    for lo, hi in re.findall(r"\bv\[(\d+):(\d+)\]", text):
        out |= set(range(int(lo), int(hi) + 1))
    return out | {int(r) for r in re.findall(r"\bv(\d+)\b", text)}


def outstanding_hazards(lines: list[str]) -> tuple[list[str], int]:
    """Instructions that touch a register of a hand-issued read still in flight, and
    the number of such reads. Straight-line order; a read is done once a wait allows
    fewer LDS operations than were issued after it."""
    pending: list[tuple[set, str]] = []
    bad, reads, asm = [], 0, False
    for ln in lines:
        t = ln.strip()
        if t.startswith(";#ASMSTART") or t.startswith(";;#ASMSTART"):
            asm = True
            continue
        if t.startswith(";#ASMEND") or t.startswith(";;#ASMEND"):
            asm = False
            continue
        t = t.split(";")[0].strip()
        if not t or t.startswith(".") or t.endswith(":"):
            continue
        m = re.search(r"lgkmcnt\((\d+)\)", t)
        if t.startswith("s_waitcnt"):
            if m:
                pending = pending[len(pending) - int(m.group(1)):] if int(m.group(1)) else []
            continue
        used = _regs(t)
        hit = [p for p in pending if p[0] & used]
        if hit and not (asm and t.startswith("ds_read")):
            bad.append(f"{t}   touches {hit[0][1]}")
        if asm and t.startswith("ds_read"):
            dest, rest = t.split(None, 1)[1].split(",", 1)
            if any(p[0] & (_regs(rest) | _regs(dest)) for p in pending):
                bad.append(f"{t}   reuses a register in flight")
            pending.append((_regs(dest), t))
            reads += 1
        elif t.startswith("ds_"):
            pending.append((set(), t))
    return bad, reads


def test_checker_sees_a_copy_in_flight():
    head = [";#ASMSTART", "ds_read_b128 v[4:7], v1", ";#ASMEND", ";#ASMSTART", "ds_read_b128 v[8:11], v1", ";#ASMEND"]
    ok = head + ["s_waitcnt lgkmcnt(1)", "v_mov_b32_e32 v0, v5", "s_waitcnt lgkmcnt(0)", "v_mov_b32_e32 v0, v9"]
    assert outstanding_hazards(ok) == ([], 2)
    assert outstanding_hazards(head + ["s_waitcnt lgkmcnt(1)", "v_accvgpr_write_b32 a0, v9"])[0]


def test_no_register_of_a_read_in_flight_is_touched(tmp_path):
    from kgs.utils.build import targets

    t = next(x for x in targets() if x.name == "kernels")
    r = subprocess.run([HIPCC, *t.flags, *t.source_flags["latent.hip"], "--offload-device-only", "-S",
                        str(ROOT / "native" / "kernels" / "latent.hip"), "-o", str(tmp_path / "l.s")],
                       capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    asm = (tmp_path / "l.s").read_text()
    seen = 0
    for m in re.finditer(r"^(_ZN3kgs6latent4attnILi(\d+)ELi(\d+)E\S+):[^\n]*$", asm, re.M):
        body = asm[m.end():asm.index(".Lfunc_end", m.end())].splitlines()
        bad, reads = outstanding_hazards(body)
        assert not bad, (m.group(1), bad[:5])
        rt, rk = int(m.group(2)), int(m.group(3))
        assert reads == 2 * (rt + rk) + 4 * rt, (rt, rk, reads)  # keys twice per step, four transposed reads per tile pair
        seen += 1
    assert seen == 3 * 8
