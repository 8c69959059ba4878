"""Builds the shared libraries of the C ABI (include/evo_mi355x.h) from evo_amd/csrc/*.hip with hipcc for gfx950.

The sources are grouped into components, one library each, so that a process builds and loads only what its model calls:
  core          dense layers, norms, embedding, scoring tail -- every model
  stripedhyena  the Hyena operator and the causal attention of the StripedHyena models
  mixers        what every model described by a config.json shares: the token-local kernels around the mixers, softmax attention of prompts
  lightning, latent, heads, rglru
                one mechanism each: decayed linear attention, latent attention, attention with cached keys and values, gated linear
                recurrence

In-tree build: the .so files land in evo_amd/_lib/ so they travel with the repo snapshot to the GPU box
(they are git-ignored).  hipcc cross-compiles without a GPU.
"""
from __future__ import annotations

import os
import shutil
import subprocess
from concurrent.futures import ThreadPoolExecutor
from pathlib import Path

ROOT = Path(__file__).resolve().parent
CSRC = ROOT / "csrc"
LIBDIR = ROOT / "_lib"
# A/B builds: EVO_AMD_LIBNAME picks another base name in _lib/, EVO_AMD_HIPCC_FLAGS appends compiler flags
LIBNAME = os.environ.get("EVO_AMD_LIBNAME", "libevo_mi355x.so")
ARCH = "gfx950"

# component -> (suffix of the library's name, sources, headers beside common.h, the symbols of include/evo_mi355x.h it exports)
COMPONENTS = {
    "core": ("", ["elementwise", "gemm", "gemv", "score_tail", "probe"], [], [
        "evo_abi_version", "evo_embed_bf16", "evo_rmsnorm_bf16", "evo_rmsnorm_rows_bf16", "evo_rms_finalize_f32", "evo_rope_qk_bf16",
        "evo_rope_append_decode_bf16", "evo_gelu_gate_bf16", "evo_logprob_entropy", "evo_unembed_logprob_bf16",
        "evo_linear_small_m_bf16", "evo_norm_linear_small_m_bf16", "evo_mlp_gate_small_m_bf16", "evo_norm_mlp_gate_small_m_bf16",
        "evo_hyena_decode_fused_small_m", "evo_linear_mfma_bf16", "evo_linear_mfma_nf_bf16", "evo_mlp_gate_mfma_bf16",
        "evo_mlp_gate_mfma_nf_bf16", "evo_linear_xblk_mfma_bf16", "evo_linear_xblk_mfma_nf_bf16", "evo_linear_t_mfma_bf16",
        "evo_linear_t_mfma_nf_bf16", "evo_linear_act_mfma_bf16", "evo_postnorm_linear_small_m_bf16",
        "evo_postnorm_mlp_gate_small_m_bf16", "evo_probe_copy_f4", "evo_probe_mfma_bf16",
    ]),
    "stripedhyena": ("_stripedhyena", ["attn", "attn_w64", "hyena", "hyena_ct"], ["attn_common.h"], [
        "evo_hyena_seg_state", "evo_hyena_carry_scan", "evo_hyena_carry_add", "evo_hyena_apply", "evo_hyena_step", "evo_hyena_ct",
        "evo_attn_fwd_causal_bf16", "evo_attn_decode_bf16",
    ]),
    "mixers": ("_mixers", ["stream", "window_attn"], ["mixers_common.h"], [
        "evo_embed_stream", "evo_postnorm_residual", "evo_sum_norm", "evo_rmsnorm_stream", "evo_gated_norm", "evo_silu_gate", "evo_act_cols",
        "evo_window_attn",
    ]),
    "lightning": ("_lightning", ["lightning"], ["mixers_common.h"], ["evo_lightning_chunk_bf16", "evo_lightning_recurrent"]),
    "latent": ("_latent", ["latent"], ["mixers_common.h"], ["evo_latent_prep", "evo_latent_absorb", "evo_latent_decode", "evo_latent_up"]),
    "heads": ("_heads", ["heads"], ["mixers_common.h"], ["evo_heads_prep", "evo_heads_decode", "evo_heads_merge"]),
    "rglru": ("_rglru", ["rglru"], ["mixers_common.h"], ["evo_rglru_chunk_bf16", "evo_rglru_step_bf16", "evo_rglru_any"]),
}

# every symbol include/evo_mi355x.h declares
EXPORTS = [name for _, _, _, names in COMPONENTS.values() for name in names]
COMPONENT_OF = {name: comp for comp, (_, _, _, names) in COMPONENTS.items() for name in names}

# packed fp32 instructions stay off in every file: some of their forms are not reliable on this part
BASE_FLAGS = [f"--offload-arch={ARCH}", "-O3", "-std=c++17", "-fPIC", "-fno-gpu-rdc", "-Wno-inline-asm", "-Wno-unused-command-line-argument",
              "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]
# per-file compiler flags.  attn_w64.hip: its softmax streams are scalar fp32 on purpose, so the SLP vectoriser stays off for that file
FILE_FLAGS = {"attn_w64.hip": ["-fno-slp-vectorize", "-Wno-unused-value"]}


def lib_path(component: str = "core") -> Path:
    name = Path(LIBNAME)
    return LIBDIR / (name.stem + COMPONENTS[component][0] + name.suffix)


def sources(component: str = None):
    comps = COMPONENTS if component is None else [component]
    return [CSRC / (s + ".hip") for c in comps for s in COMPONENTS[c][1]]


def _hipcc() -> str:
    for cand in (os.environ.get("HIPCC"), shutil.which("hipcc"), "/opt/rocm/bin/hipcc"):
        if cand and os.path.exists(cand):
            return cand
    raise RuntimeError("hipcc not found: cannot build the evo_mi355x libraries")


def is_stale(component: str = "core") -> bool:
    out = lib_path(component)
    if not out.exists():
        return True
    deps = sources(component) + [CSRC / h for h in ["common.h"] + COMPONENTS[component][2]] + [ROOT.parent / "include" / "evo_mi355x.h"]
    return max(p.stat().st_mtime for p in deps if p.exists()) > out.stat().st_mtime


def _run(cmd, what: str, verbose: bool) -> None:
    if verbose:
        print(" ".join(cmd))
    proc = subprocess.run(cmd, capture_output=True, text=True)
    if proc.returncode != 0:
        raise RuntimeError(f"hipcc failed on {what}:\n" + proc.stdout + proc.stderr)


def build(components=None, force: bool = False, verbose: bool = False) -> dict:
    """Compile the HIP sources of the given components (all by default; one object per file, in parallel) and link one shared library
    per component.  Libraries newer than their sources are kept unless `force`.  Returns {component: library path}."""
    wanted = list(COMPONENTS) if components is None else list(components)
    todo = [c for c in wanted if force or is_stale(c)]
    if todo:
        LIBDIR.mkdir(exist_ok=True)
        objdir = LIBDIR / ("obj%d" % os.getpid())
        objdir.mkdir(exist_ok=True)
        try:
            def compile_one(src):
                _run([_hipcc()] + BASE_FLAGS + os.environ.get("EVO_AMD_HIPCC_FLAGS", "").split() + FILE_FLAGS.get(src.name, [])
                     + ["-c", str(src), "-o", str(objdir / (src.stem + ".o"))], src.name, verbose)
            with ThreadPoolExecutor(max_workers=8) as ex:
                list(ex.map(compile_one, [s for c in todo for s in sources(c)]))
            for c in todo:
                tmp = lib_path(c).with_suffix(".so.tmp%d" % os.getpid())
                _run([_hipcc(), f"--offload-arch={ARCH}", "-shared", "-fPIC", "-fno-gpu-rdc", "-o", str(tmp)]
                     + [str(objdir / (s.stem + ".o")) for s in sources(c)], f"link of {lib_path(c).name}", verbose)
                os.replace(tmp, lib_path(c))
        finally:
            shutil.rmtree(objdir, ignore_errors=True)
    return {c: lib_path(c) for c in wanted}


if __name__ == "__main__":
    print(build(force=True, verbose=True))
