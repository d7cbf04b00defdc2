"""Builds the two in-tree shared libraries of koifish_amd:

  libkf_hip.so   hipcc --offload-arch=gfx950: the kernels + the C ABI of include/kf_abi.h
  libkf_host.so  g++: the C++ host mirror of the reference's neuron interface, above the ABI

Both are written next to this file so they travel with the source tree.  No JIT cache.
"""
import os
import re
import subprocess
import sys

HERE = os.path.dirname(os.path.abspath(__file__))
CSRC = os.path.join(HERE, "csrc")
HOST = os.path.join(HERE, "host")
HIP_SOURCES = ["kf_gemv.hip", "kf_gemv_canon.hip", "kf_gemm.hip", "kf_gemm2.hip", "kf_gemm3.hip", "kf_attn.hip", "kf_engine.hip", "kf_xengine.hip", "kf_xengine_q1.hip", "kf_attn_prefill.hip", "kf_ops.hip", "kf_lut.hip", "kf_loss.hip", "kf_norm_bwd.hip", "kf_linear_bwd.hip", "kf_embed_bwd.hip", "kf_attn_bwd_mfma.hip", "kf_awq.hip", "kf_tp.hip", "kf_rb_ops.hip", "kf_rb_linear.hip", "kf_rb_gemm.hip", "kf_rb_attn.hip", "kf_rb_recur.hip", "kf_abi.hip"]
LIB_HIP = os.path.join(HERE, "libkf_hip.so")
LIB_HOST = os.path.join(HERE, "libkf_host.so")
HIPCC = os.environ.get("HIPCC", "/opt/rocm/bin/hipcc")
# -ffp-contract=off: the kernels spell every fma they want; an implicit contraction would change the rounding
# points that the oracle pins (RoPE, kf_expf, RMSNorm).
# -fno-slp-vectorize: keeps the dequant chain in plain v_fma/v_sub (the packed-f32 forms the SLP pass picks cost more issue
# slots, need s_nop hazard padding and 40 % more registers on this kernel)
# -packed-fp32-ops: no v_pk_add_f32 / v_pk_mul_f32 / v_pk_fma_f32 (some of their forms have given wrong results on this part); the two halves of an f32x2 fma are two v_fma_f32, same bits
HIP_FLAGS = ["--offload-arch=gfx950", "-Xclang", "-target-feature", "-Xclang", "-packed-fp32-ops", "-O3", "-std=c++17", "-fPIC", "-ffp-contract=off", "-fno-slp-vectorize", "-Wall", "-Wno-unused-function"]
# MFMA results that the VALU works on next (attention scores, the epilogues of the token-batch GEMMs): with the default AGPR form of the MFMA destination the
# compiler moves every such value AGPR -> VGPR (v_accvgpr_read) and zero-fills accumulators through v_accvgpr_write -- 160 of the ~330 vector instructions of a
# key tile in the attention backward.  The VGPR form has none of them (and the files below stay inside 256 VGPRs where it matters).
HIP_FILE_FLAGS = {f: ["-mllvm", "-amdgpu-mfma-vgpr-form=1"] for f in os.environ.get("KF_VGPR_FORM", "kf_attn_prefill.hip,kf_attn_bwd_mfma.hip,kf_gemm.hip").split(",") if f}


def _stale(target, deps):
    if not os.path.exists(target):
        return True
    t = os.path.getmtime(target)
    return any(os.path.getmtime(d) > t for d in deps)


def _includes(path, seen=None):
    """path and every in-tree file it #includes, directly or not"""
    seen = set() if seen is None else seen
    path = os.path.normpath(path)
    if path in seen or not os.path.exists(path):
        return seen
    seen.add(path)
    with open(path) as f:
        for m in re.finditer(r'^\s*#include "([^"]+)"', f.read(), re.M):
            _includes(os.path.join(os.path.dirname(path), m.group(1)), seen)
    return seen


def _compile(sources, force, verbose):
    """objects of the named csrc/ files, compiled where stale"""
    objs, cmds = [], []
    for s in [os.path.join(CSRC, s) for s in sources]:
        o = s[:-4] + ".o"
        objs.append(o)
        if force or _stale(o, _includes(s)):
            cmds.append([HIPCC] + HIP_FLAGS + HIP_FILE_FLAGS.get(os.path.basename(s), []) + ["-c", s, "-o", o])
    if cmds:   # independent translation units: a few at a time (the container has 8 CPUs; one hipcc peaks near 2 GB)
        from concurrent.futures import ThreadPoolExecutor

        def run(cmd):
            if verbose:
                print(" ".join(cmd), flush=True)
            subprocess.check_call(cmd)
        with ThreadPoolExecutor(max_workers=int(os.environ.get("KF_BUILD_JOBS", "6"))) as ex:
            list(ex.map(run, cmds))
    return objs


def build_hip(force=False, verbose=False):
    objs = _compile(HIP_SOURCES, force, verbose)
    if force or _stale(LIB_HIP, objs):
        cmd = [HIPCC, "--offload-arch=gfx950", "-shared", "-fPIC", "-o", LIB_HIP] + objs
        if verbose:
            print(" ".join(cmd))
        subprocess.check_call(cmd)
    return LIB_HIP


HOST_SOURCES = ["kf_host.cpp", "kf_safetensors.cpp", "kf_train.cpp", "kf_seq.cpp", "kf_tizusun.cpp", "kf_bolopel.cpp"]


def _host_cmd(out, libdir, opt):
    return ["g++"] + opt + ["-std=c++17", "-fPIC", "-shared", "-Wall", "-o", out] + [os.path.join(HOST, s) for s in HOST_SOURCES] + ["-L" + libdir, "-lkf_hip", "-Wl,-rpath,$ORIGIN"]


def _host_deps(libhip):
    deps = set()
    for s in HOST_SOURCES:
        _includes(os.path.join(HOST, s), deps)
    return sorted(deps) + [libhip]


def build_host(force=False, verbose=False):
    if force or _stale(LIB_HOST, _host_deps(LIB_HIP)):
        cmd = _host_cmd(LIB_HOST, HERE, ["-O2"])
        if verbose:
            print(" ".join(cmd))
        subprocess.check_call(cmd)
    return LIB_HOST


# What one family of models launches.  A fresh checkout that only serves such a model (bin/trace_run) compiles these files and no others: seconds instead of minutes.
PARTS = {"rows": ["kf_rb_ops.hip", "kf_rb_linear.hip", "kf_rb_gemm.hip", "kf_rb_attn.hip", "kf_rb_recur.hip", "kf_ops.hip", "kf_abi.hip"]}


def build_part(part, verbose=False):
    """The two libraries with the device code of one part, in a directory of their own (koifish_amd/part_<part>/): the launchers of every other kernel are bound to a stub
    that reports KF_UNSUPPORTED_DATATYPE.  Returns the directory (what KF_LIB_DIR takes)."""
    out = os.path.join(HERE, "part_" + part)
    os.makedirs(out, exist_ok=True)
    hip, host = os.path.join(out, "libkf_hip.so"), os.path.join(out, "libkf_host.so")
    objs = _compile(PARTS[part], False, verbose)
    if _stale(hip, objs):
        def symbols(flag):
            return {l.split()[-1] for o in objs for l in subprocess.check_output(["nm", flag, o]).decode().splitlines() if l.split()}
        absent = sorted(s for s in symbols("--undefined-only") - symbols("--defined-only") if s.startswith("_ZN2kf"))
        stub = os.path.join(out, "absent.c")
        with open(stub, "w") as f:
            f.write("/* launchers of kernels this build leaves out */\nint kf_part_absent(void) { return -1000; }\n")
        subprocess.check_call(["gcc", "-O1", "-fPIC", "-fvisibility=hidden", "-c", stub, "-o", stub[:-2] + ".o"])
        cmd = [HIPCC, "--offload-arch=gfx950", "-shared", "-fPIC", "-o", hip] + objs + [stub[:-2] + ".o"] + ["-Wl,--defsym=%s=kf_part_absent" % s for s in absent]
        if verbose:
            print(" ".join(cmd[:12]), "...", flush=True)
        subprocess.check_call(cmd)
    if _stale(host, _host_deps(hip)):
        subprocess.check_call(_host_cmd(host, out, ["-O2"]))
    return out


def build_host_asan(verbose=False):
    """CPU-only sanitizer build of the host library (AddressSanitizer + UBSan): the JSON / msgpack / mmap parsers of kf_safetensors.cpp read untrusted
    files.  Written to libkf_host_asan.so; tests/test_host_asan_cpu.py runs the checkpoint tests under it (LD_PRELOAD of libasan, KF_HOST_LIB).
    Never for the GPU box: sanitizers run on the CPU build only."""
    out = os.path.join(HERE, "libkf_host_asan.so")
    if _stale(out, _host_deps(LIB_HIP)):
        cmd = _host_cmd(out, HERE, ["-O1", "-g", "-fno-omit-frame-pointer", "-fsanitize=address,undefined", "-fno-sanitize-recover=undefined"])
        if verbose:
            print(" ".join(cmd))
        subprocess.check_call(cmd)
    return out


def build_all(force=False, verbose=False):
    return build_hip(force, verbose), build_host(force, verbose)


if __name__ == "__main__":
    if "asan" in sys.argv:   # python -m koifish_amd.build asan
        print(build_host_asan(verbose=True))
    else:
        print(build_all(force="--force" in sys.argv, verbose=True))
