"""Packaging + in-tree HIP extension build for mlx_sharding_amd.

Entry points mirror the reference CLI surface
(/root/reference/setup.py:27-32): `mlx-sharding-server` and
`mlx-sharding-api`, plus our `mlx-sharding-generate` CLI.

Build the gfx950 extension in-tree with:
    PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext --inplace
(`__graft_entry__.build()` drives this.)
"""

import os
from pathlib import Path

from setuptools import find_packages, setup

ROOT = Path(__file__).parent
HIP_DIR = ROOT / "mlx_sharding_amd" / "ops" / "hip"

# scalar fp32 math only: the packed v_pk_*_f32 forms the optimizer makes out
# of ordinary float code are kept out of every kernel
NO_PACKED_FP32 = ["-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops"]

# extension -> its sources; MLXS_AMD_EXT=name[,name] builds only those
# (bin/trace_run builds just what its model loads)
SOURCES = {
    "_hip_ragged": lambda name: name.startswith("ragged_") or name == "elementwise.hip",
    "_hip_ops": lambda name: not name.startswith("ragged_"),
}

ext_modules = []
cmdclass = {}
hip_sources = sorted(p for p in HIP_DIR.glob("*.hip") if not p.name.endswith("_hip.hip"))
if hip_sources and os.environ.get("MLXS_AMD_SKIP_EXT", "0") != "1":
    try:
        from torch.utils.cpp_extension import BuildExtension, CUDAExtension

        os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")
        wanted = [n for n in os.environ.get("MLXS_AMD_EXT", "").split(",") if n]
        for ext_name in wanted or sorted(SOURCES):
            ext_modules.append(CUDAExtension(
                name=f"mlx_sharding_amd.{ext_name}",
                sources=[str(p) for p in hip_sources if SOURCES[ext_name](p.name)],
                extra_compile_args={
                    "cxx": ["-O3", "-std=c++17"],
                    "nvcc": ["-O3", "-std=c++17", "--offload-arch=gfx950",
                             *NO_PACKED_FP32],
                },
            ))
        cmdclass = {"build_ext": BuildExtension}
    except ImportError:  # torch missing at sdist time
        pass

setup(
    name="mlx_sharding_amd",
    version="0.1.0",
    description="MI355X-native pipeline-parallel LLM inference engine",
    packages=find_packages(include=["mlx_sharding_amd", "mlx_sharding_amd.*"]),
    package_data={
        # web UI served by the API server (reference shard/static/*)
        "mlx_sharding_amd.server": ["static/*"],
        # kernel sources ship so build_ext works from an sdist
        "mlx_sharding_amd.ops": ["hip/*.hip", "hip/*.h"],
    },
    include_package_data=True,
    python_requires=">=3.10",
    ext_modules=ext_modules,
    cmdclass=cmdclass,
    entry_points={
        "console_scripts": [
            "mlx-sharding-server=mlx_sharding_amd.cli.server_main:main",
            "mlx-sharding-api=mlx_sharding_amd.server.openai_api:main",
            "mlx-sharding-generate=mlx_sharding_amd.cli.generate:main",
            "mlx-sharding-split=mlx_sharding_amd.cli.shard_weights:main",
            "mlx-sharding-rccl-serve=mlx_sharding_amd.cli.rccl_serve:main",
        ]
    },
)
