"""The model registry: config.json -> the class that serves it.

A checkpoint directory is recognised by its config.json: `architecture` (designs described layer by layer) or Hugging Face's `model_type` / `architectures`.
"""
import json
import os

from . import lib as L
from .build import PARTS
from .runtime import Bolopel, Qwen3, Tizusun


def _tizusun(path, dtype, max_seq, device):
    return Tizusun.from_dir(path, dtype=dtype, max_seq=max_seq, device=device)


def _bolopel(path, dtype, max_seq, device):
    return Bolopel.from_dir(path, dtype=dtype, max_seq=max_seq, device=device)


def _qwen3(path, dtype, max_seq, device):
    if dtype != "bfloat16":
        raise L.KFError("Qwen3 runs in bfloat16 (dtype %r)" % dtype)
    return Qwen3.from_hf(path, layer_type=L.BF16, head_type=L.BF16, device=device, max_seq=max_seq)


# name -> (loader, the part of the device code it needs: build.PARTS, None = all of it)
ARCHITECTURES = {"Tizusun": (_tizusun, "rows"), "Bolopel": (_bolopel, "rows"), "Qwen3ForCausalLM": (_qwen3, None), "qwen3": (_qwen3, None)}
assert all(p is None or p in PARTS for _, p in ARCHITECTURES.values())


def architecture(path):
    """the registered name a checkpoint directory asks for"""
    with open(os.path.join(str(path), "config.json")) as f:
        cfg = json.load(f)
    names = [cfg.get("architecture"), cfg.get("model_type")] + list(cfg.get("architectures") or [])
    for n in names:
        if n in ARCHITECTURES:
            return n
    raise L.KFError("%s/config.json: architecture %s is not registered (registered: %s)" % (path, [n for n in names if n], ", ".join(sorted(ARCHITECTURES))))


def load_model(path, dtype="bfloat16", max_seq=0, device=0):
    return ARCHITECTURES[architecture(path)][0](path, dtype, max_seq, device)
