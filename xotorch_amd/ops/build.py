"""In-tree build of the CDNA4 HIP extensions (no network, no JIT cache).

Invoked by __graft_entry__.build(). Every hip/*.hip translation unit becomes
one extension next to this file, compiled with hipcc --offload-arch=gfx950,
so the built artifacts travel with the repo snapshot to the GPU box. The
compiler runs are independent and go in parallel.
"""
from __future__ import annotations

import os
import subprocess
import sys
import sysconfig
from pathlib import Path
from typing import List, Optional, Sequence

PKG_DIR = Path(__file__).resolve().parent
# extension module -> its source
EXTENSIONS = {
  "_hip_ops": PKG_DIR / "hip" / "hip_ops.hip",
  "_hip_mixers": PKG_DIR / "hip" / "mixer_ops.hip",
  "_hip_attn": PKG_DIR / "hip" / "attn_rows.hip",
  "_hip_rotary": PKG_DIR / "hip" / "rotary_attn.hip",
  "_hip_lru": PKG_DIR / "hip" / "lru_ops.hip",
  "_hip_experts": PKG_DIR / "hip" / "expert_ops.hip",
  "_hip_scan": PKG_DIR / "hip" / "scan_ops.hip",
  "_hip_latent": PKG_DIR / "hip" / "latent_ops.hip",
  "_hip_stream": PKG_DIR / "hip" / "stream_ops.hip",
  "_hip_mlstm": PKG_DIR / "hip" / "mlstm_ops.hip",
}


def out_path(name: str) -> Path:
  return PKG_DIR / f"{name}.so"


def needs_build(name: str) -> bool:
  out = out_path(name)
  sources = [EXTENSIONS[name], *(PKG_DIR / "hip").glob("*.h")]
  return not out.exists() or max(s.stat().st_mtime for s in sources) > out.stat().st_mtime


def _command(name: str, out: Path) -> List[str]:
  import torch
  from torch.utils import cpp_extension
  abi = 1 if torch._C._GLIBCXX_USE_CXX11_ABI else 0
  cmd = [
    "hipcc", "--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-shared",
    # packed fp32 instructions stay off: plain fp32 code must not turn into them
    "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
    f"-DTORCH_EXTENSION_NAME={name}", "-DTORCH_API_INCLUDE_EXTENSION_H",
    f"-D_GLIBCXX_USE_CXX11_ABI={abi}", "-DUSE_ROCM", "-D__HIP_PLATFORM_AMD__",
  ]
  for inc in [*cpp_extension.include_paths(), sysconfig.get_paths()["include"]]:
    cmd += ["-I", inc]
  cmd += [str(EXTENSIONS[name]), "-o", str(out)]
  for lp in cpp_extension.library_paths():
    cmd += ["-L", lp]
  return cmd + ["-ltorch", "-ltorch_hip", "-lc10", "-lc10_hip", "-ltorch_python"]


def build(force: bool = False, verbose: bool = True, missing_only: bool = False,
          only: Optional[Sequence[str]] = None) -> List[Path]:
  """Compile the extensions (`only`: of these) that are missing or older than their
  source; `force` compiles all, `missing_only` trusts what is built already."""
  names = [n for n in (EXTENSIONS if only is None else only) if force or (not out_path(n).exists() if missing_only else needs_build(n))]
  jobs = []
  for n in names:
    # compile beside the target and move into place: a concurrent reader sees
    # the old library or the new one, never half of one
    tmp = out_path(n).with_suffix(f".so.tmp{os.getpid()}")
    cmd = _command(n, tmp)
    if verbose:
      print(f"[xotorch_amd] building {n}:", " ".join(cmd), file=sys.stderr)
    jobs.append((n, tmp, cmd, subprocess.Popen(cmd)))
  for n, tmp, cmd, proc in jobs:
    proc.wait()
  for n, tmp, cmd, proc in jobs:
    if proc.returncode:
      tmp.unlink(missing_ok=True)
      raise subprocess.CalledProcessError(proc.returncode, cmd)
    os.replace(tmp, out_path(n))
  return [out_path(n) for n in names]


if __name__ == "__main__":
  build(force="--force" in sys.argv)
