"""Build the CDNA4 HIP extension in-tree:

    PYTORCH_ROCM_ARCH=gfx950 python setup.py build_ext --inplace

The libraries land at substratus_amd/_C*.so and substratus_amd/_hybrid*.so
(git-ignored). SUB_EXT names the extensions to build, with commas between them;
default all.
"""

import glob
import os

from setuptools import find_packages, setup

os.environ.setdefault("PYTORCH_ROCM_ARCH", "gfx950")

from torch.utils.cpp_extension import BuildExtension, CUDAExtension  # noqa: E402

ROOT = os.path.dirname(os.path.abspath(__file__))
HIP_DIR = os.path.join(ROOT, "substratus_amd", "ops", "hip")
HYBRID_DIR = os.path.join(HIP_DIR, "hybrid")

# Hand-written kernel sources only. torch's CUDAExtension hipify pass emits
# *_hip.hip/*_hip.cpp siblings into the build dir; exclude any that leak
# in-tree so the generated copies can never shadow the originals.
def hip_sources(folder):
    return [os.path.join(folder, f) for f in sorted(os.listdir(folder))
            if f.endswith(".hip") and not f.endswith("_hip.hip")]


def drop_stale_objects():
    """Objects older than a header: the build itself only looks at sources."""
    headers = glob.glob(os.path.join(HIP_DIR, "**", "*.h"), recursive=True)
    newest = max(os.path.getmtime(h) for h in headers)
    for obj in glob.glob(os.path.join(ROOT, "build", "temp*", "**", "*.o"),
                         recursive=True):
        if os.path.getmtime(obj) < newest:
            os.remove(obj)


def extension(name, sources):
    return CUDAExtension(
        name=f"substratus_amd.{name}", sources=sources,
        extra_compile_args={
            "cxx": ["-O3", "-std=c++17"],
            # packed-FP32 VALU forms stay off: some of them have given
            # wrong results on this hardware
            "nvcc": ["-O3", "-std=c++17", "-Xclang", "-target-feature",
                     "-Xclang", "-packed-fp32-ops"],
        })


# _C: the kernels of the uniform transformer families, sampling, training.
# _hybrid: the kernels of models whose layers differ (models/hybrid.py).
extensions = {
    "_C": hip_sources(HIP_DIR),
    "_hybrid": hip_sources(HYBRID_DIR) + [
        os.path.join(HIP_DIR, "activation.hip")],
}
drop_stale_objects()
wanted = os.environ.get("SUB_EXT", ",".join(extensions)).split(",")

setup(
    name="substratus_amd",
    version="0.1.0",
    packages=find_packages(include=["substratus_amd", "substratus_amd.*"]),
    # wheels carry the built _C.so + the GEMM tables; kernel SOURCES ride
    # the sdist via MANIFEST.in (which can exclude the *_hip.hip siblings
    # torch's hipify regenerates in-tree on every build)
    package_data={"substratus_amd": ["data/tunables/*.csv"]},

    entry_points={"console_scripts": [
        "sub = substratus_amd.cli.main:main",
        "nbwatch = substratus_amd.containertools.nbwatch:watch",
    ]},
    ext_modules=[extension(n, extensions[n]) for n in wanted],
    cmdclass={"build_ext": BuildExtension},
)
