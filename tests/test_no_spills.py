"""Build-time guard: the kernels whose residency is tuned to a register budget must not spill (hipcc's allocator is
one refactor away from scratch traffic in the middle of a load burst).  Cross-compiles for gfx950; no GPU needed."""
import re
import shutil
import subprocess
from pathlib import Path

import pytest

from sglang_amd.build import HIPCC_FLAGS

ROOT = Path(__file__).resolve().parent.parent
HIPCC = shutil.which("hipcc") or "/opt/rocm/bin/hipcc"


def _resource_usage(src: str, tmp_path):
    out = tmp_path / "k.s"
    cmd = [HIPCC, *HIPCC_FLAGS, f"-I{ROOT / 'include'}", "--cuda-device-only", "-S",
           str(ROOT / "sglang_amd" / "csrc" / src), "-o", str(out)]
    res = subprocess.run(cmd, capture_output=True, text=True)
    assert res.returncode == 0, res.stderr[-2000:]
    usage = {}
    name = None
    for line in out.read_text().splitlines():
        m = re.match(r"\s+\.name:\s+(\S+)", line)
        if m:
            name = m.group(1)
        m = re.match(r"\s+\.(vgpr_count|vgpr_spill_count|sgpr_spill_count|group_segment_fixed_size):\s+(\d+)", line)
        if m:
            usage.setdefault("pending", {})[m.group(1)] = int(m.group(2))
        if name and "pending" in usage and line.strip().startswith(".wavefront_size"):
            usage[name] = usage.pop("pending")
            name = None
    usage.pop("pending", None)
    return usage


@pytest.mark.skipif(not Path(HIPCC).exists(), reason="hipcc not installed")
def test_cascade_chunk_kernel_fits_five_workgroups_per_cu(tmp_path):
    usage = _resource_usage("cascade_attention.hip", tmp_path)
    chunk = {k: v for k, v in usage.items() if "cascade_chunk_kernel" in k}
    assert len(chunk) == 8, sorted(usage)                       # head dim {64, 128} x {bf16, fp8} x {NHD, HND}
    for name, u in chunk.items():
        # Compiled with the library's own flags.  Without packed fp32 instructions (build.py) the D = 128 instances need more
        # registers than the 96 of five workgroups per CU: 5 values go to scratch in the bf16 ones (none with packed
        # instructions) and up to 12 in the e4m3 ones (3 before).  Known cost of that flag; anything more must fail here
        limit = 12 if "ILi128ELb1E" in name else 5 if "ILi128ELb0E" in name else 2
        assert u["vgpr_spill_count"] <= limit and u["sgpr_spill_count"] == 0, (name, u)
        assert u["vgpr_count"] <= 96, (name, u)                 # 512 / 5 waves per SIMD, 8-register granules
        # five workgroups per CU: LDS is handed out in 1280-byte granules -- the 16 KiB image + the token-split units' side buffer
        # (8 KiB at D = 128) + 256 B of (max, sum) = 20 granules, five of them 128 000 of the 163 840 bytes
        assert u["group_segment_fixed_size"] <= 25600, (name, u)
    # the looping form (large request tables: a bounded grid walks the item list) runs four workgroups per CU and must not spill at all
    # (a five-per-CU instance parks ~29 registers in scratch and measured 34 against 26.7 us per layer: profiles/r05_exp1b_cascade_forms.json)
    loop = {k: v for k, v in usage.items() if "cascade_chunk_loop_kernel" in k}
    assert len(loop) == 8, sorted(usage)
    for name, u in loop.items():
        limit = 8 if "ILi128ELb1ELb0E" in name else 0          # (the same cost in the token-major e4m3 instance)
        assert u["vgpr_spill_count"] <= limit and u["sgpr_spill_count"] == 0, (name, u)
        assert u["vgpr_count"] <= 128 and u["group_segment_fixed_size"] <= 25600, (name, u)


@pytest.mark.skipif(not Path(HIPCC).exists(), reason="hipcc not installed")
def test_extend_eight_wave_kernels_keep_their_registers_and_lds(tmp_path):
    """The 8-wave kernels run two waves per SIMD (256 registers each) in one workgroup per CU.  The 32x32 kernel holds
    O^T (64), two score sets (64), Q^T (32), P (16), the staging rows (16) and three K fragments at ~245: a spill would
    sit between the matrix instructions; LDS = two K and two V images."""
    usage = _resource_usage("extend_attention.hip", tmp_path)
    for kernel, lds, n in (("extend_attention_pipe_kernel", 72 * 1024, 4), ("extend_attention_dbuf_kernel", 80 * 1024, 2)):
        inst = {k: v for k, v in usage.items() if kernel in k}
        assert len(inst) == n, sorted(usage)                    # head dim {64, 128} (x {bf16, e4m3 rows} for the 32x32 kernel)
        for name, u in inst.items():
            assert u["vgpr_spill_count"] == 0 and u["sgpr_spill_count"] == 0, (name, u)
            assert u["vgpr_count"] <= 256, (name, u)
            assert u["group_segment_fixed_size"] <= lds, (name, u)


@pytest.mark.skipif(not Path(HIPCC).exists(), reason="hipcc not installed")
def test_general_extend_kernels_do_not_spill(tmp_path):
    """Every instance of the general extend kernel (fp8 / paged pools, sliding window, soft cap, custom mask; the 4-wave
    shapes of short extends): a spill would sit inside the KV-tile loop."""
    usage = _resource_usage("extend_attention.hip", tmp_path)
    gen = {k: v for k, v in usage.items() if "extend_attention_kernel" in k}
    assert len(gen) == 12, sorted(usage)                        # head dim {64, 128} x {41, 42, 82} x {bf16, fp8}
    for name, u in gen.items():
        assert u["vgpr_spill_count"] == 0 and u["sgpr_spill_count"] == 0, (name, u)


@pytest.mark.skipif(not Path(HIPCC).exists(), reason="hipcc not installed")
def test_moe_256_tile_kernel_keeps_its_registers_and_lds(tmp_path):
    """moe_gemm256_kernel runs two waves per SIMD in one workgroup per CU: 128 accumulator registers + two fragment sets
    (64) + the eight LDS-DMA row pointers at ~213; a spill would sit between the products.  LDS = two 64 KiB stages."""
    usage = _resource_usage("moe_tiled_gemm.hip", tmp_path)
    k256 = {k: v for k, v in usage.items() if "moe_gemm256_kernel" in k}
    assert len(k256) == 1, sorted(usage)
    for name, u in k256.items():
        assert u["vgpr_spill_count"] == 0 and u["sgpr_spill_count"] == 0, (name, u)
        assert u["vgpr_count"] <= 256, (name, u)
        assert u["group_segment_fixed_size"] == 128 * 1024, (name, u)
    k128 = {k: v for k, v in usage.items() if "moe_tiled_gemm_kernel" in k}
    assert len(k128) == 1
    for name, u in k128.items():
        assert u["vgpr_spill_count"] == 0 and u["sgpr_spill_count"] == 0 and u["vgpr_count"] <= 128, (name, u)   # two workgroups per CU


@pytest.mark.skipif(not Path(HIPCC).exists(), reason="hipcc not installed")
def test_hybrid_kernels_keep_their_state_in_registers(tmp_path):
    """The chunked recurrences hold the state tile in accumulators over a whole segment and the latent attention kernels hold
    queries and output sums: a spill would sit inside their loops.  (bf16 instances of the sizes real layers have.)"""
    usage = _resource_usage("recurrent_chunk.hip", tmp_path)
    for kernel in ("mamba2_chunk_kernelItLi8E", "delta_chunk_kernelItLi8E", "mamba2_chunk_kernelItLi4E", "delta_chunk_kernelItLi4E", "memory_chunk_kernelItLi8E",
                   "memory_chunk_kernelItLi4E"):
        inst = {k: v for k, v in usage.items() if kernel in k}
        assert len(inst) == 1, sorted(usage)
        for name, u in inst.items():
            assert u["vgpr_spill_count"] == 0 and u["vgpr_count"] <= 256, (name, u)
    usage = _resource_usage("latent_attention.hip", tmp_path)
    for kernel, n in (("latent_prefill_kernel", 3), ("latent_attention_mfma_kernelILi18E", 2)):
        inst = {k: v for k, v in usage.items() if kernel in k}
        assert len(inst) == n, sorted(usage)
        for name, u in inst.items():
            assert u["vgpr_spill_count"] == 0 and u["vgpr_count"] <= 256, (name, u)


@pytest.mark.skipif(not Path(HIPCC).exists(), reason="hipcc not installed")
def test_grouped_attention_kernels_keep_their_sums_in_registers(tmp_path):
    """Queries, sums and the next tile's rows live in registers through the key loop.  Only the widest decode instance (keys and values
    both above 128 elements) goes over, by 20 values.  Two prefill workgroups share a compute unit up to 128 / 128."""
    usage = _resource_usage("grouped_attention.hip", tmp_path)
    decode = {k: v for k, v in usage.items() if "grouped_attention_mfma_kernel" in k}
    prefill = {k: v for k, v in usage.items() if "grouped_prefill_kernel" in k}
    assert len(decode) == 18 and len(prefill) == 18, sorted(usage)      # softmax (with kept tokens or without) and sigmoid weights
    for name, u in decode.items():
        assert u["vgpr_spill_count"] <= (20 if "ILi8ELi16E" in name else 0) and u["vgpr_count"] <= 256, (name, u)
    for name, u in prefill.items():
        assert u["vgpr_spill_count"] == 0 and u["sgpr_spill_count"] == 0, (name, u)
        if "ILi8E" not in name:
            assert u["vgpr_count"] <= 256 and u["group_segment_fixed_size"] <= 80 * 1024, (name, u)
    for name, u in _resource_usage("moe_route.hip", tmp_path).items():
        assert u["vgpr_spill_count"] == 0, (name, u)
    for name, u in _resource_usage("residual_norm.hip", tmp_path).items():
        if "residual_rms_kernel" in name:
            assert u["vgpr_spill_count"] == 0, (name, u)


@pytest.mark.skipif(not Path(HIPCC).exists(), reason="hipcc not installed")
def test_projection_row_kernels_do_not_spill(tmp_path):
    """Rows, rotation partners and four partials in flight stay in registers; none of these launches asks for scratch."""
    usage = _resource_usage("projection_rows.hip", tmp_path)
    assert sum("head_prepare_kernel" in k for k in usage) == 8 and sum("latent_down_kernel" in k for k in usage) == 4, sorted(usage)
    for name, u in usage.items():
        assert u["vgpr_spill_count"] == 0 and u["sgpr_spill_count"] == 0 and u["vgpr_count"] <= 128, (name, u)
