"""Builds libnvmai_hip.so in-tree with hipcc for gfx950."""
import glob
import os
import subprocess
import sys

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
LIB = os.path.join(HERE, "libnvmai_hip.so")

FLAGS = ["--offload-arch=gfx950", "-O3", "-std=c++17", "-fPIC", "-ffp-contract=off",
         "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops",
         "-Wall", "-Wno-unused-function",
         # "#pragma unroll" on loops whose trip count is a template parameter: the instantiations that take
         # the count at run time cannot unroll, and say so once per loop
         "-Wno-pass-failed"]


# Part libraries: the sources that one family of models needs, for a run that must not wait for the rest.
_DENSE = ["ctx_api", "dense_api", "dense_erf_api", "dense_bias_api", "dense_pairs_api", "dense_full_api", "norm_api", "sample_api"]
PARTS = {"dense": _DENSE + ["gla_api", "latent_api"], "scan": _DENSE + ["window_api", "scan_api"]}


def part_path(part):
    return LIB[:-3] + "." + part + ".so"


def _compile(srcs, out, verbose, jobs):
    objs, procs = [], []
    for src in srcs:
        obj = src[:-4] + ".o"
        objs.append(obj)
        cmd = ["hipcc", *FLAGS, "-c", src, "-o", obj]
        if verbose:
            print(" ".join(cmd), flush=True)
        procs.append((src, subprocess.Popen(cmd, stdout=subprocess.PIPE, stderr=subprocess.STDOUT)))
        if len(procs) >= jobs:
            _wait(procs)
    _wait(procs)
    tmp = "%s.%d.tmp" % (out, os.getpid())
    subprocess.run(["hipcc", "--offload-arch=gfx950", "-shared", "-fPIC", "-o", tmp, *objs], check=True)
    os.replace(tmp, out)                 # a library is there whole or not at all
    return out


def build(verbose=False, jobs=8):
    """Compile every .hip file under csrc/ and link them into one shared library."""
    return _compile(sorted(glob.glob(os.path.join(CSRC, "*.hip"))), LIB, verbose, jobs)


def ensure(part, verbose=False, jobs=8):
    """The library if it is built, else the part library, built now if it is not there either."""
    if os.path.exists(LIB):
        return LIB
    os.environ["NVMAI_HIP_PART"] = part              # which of several parts the package loads
    if os.path.exists(part_path(part)):
        return part_path(part)
    return _compile([os.path.join(CSRC, n + ".hip") for n in PARTS[part]], part_path(part), verbose, jobs)


def _wait(procs):
    while procs:
        src, proc = procs.pop(0)
        out = proc.communicate()[0].decode()
        # the host pass does not know the packed-fp32 feature flag and says so
        out = "\n".join(l for l in out.splitlines() if "packed-fp32-ops" not in l)
        if proc.returncode != 0:
            raise RuntimeError("hipcc failed on %s:\n%s" % (src, out))
        if out.strip():
            print(out, file=sys.stderr)


if __name__ == "__main__":
    print(build(verbose=True))
