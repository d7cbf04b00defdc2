"""What the tests of the decoders described layer by layer share: requests in slots against a plain statement of the design (a module with forward(cfg, weights, tokens))."""
import json
import os
import struct

import numpy as np


def rel(got, ref):
    """row-wise rms difference of the centred logits against the rms of the reference"""
    d = got - ref
    d = d - d.mean(-1, keepdims=True)
    return np.sqrt((d ** 2).mean(-1)) / np.sqrt(((ref - ref.mean(-1, keepdims=True)) ** 2).mean())


def bf16_view(u):
    return (u.astype(np.uint32) << 16).view(np.float32)


class Seqs:
    """requests in slots, fed in any cut; every fed row's logits against the plain model over the whole history"""

    def __init__(self, plain, m, w, cfg, tol, n=4):
        from koifish_amd.runtime import XcdReplicas
        self.plain, self.m, self.w, self.cfg, self.tol, self.x, self.tok, self.slot, self.ref = plain, m, w, cfg, tol, XcdReplicas(m, n), {}, {}, {}

    def open(self, name, tokens, ref=None):
        self.slot[name], self.tok[name] = self.x.acquire(), [[], list(tokens)]
        self.ref[name] = self.plain.forward(self.cfg, self.w, tokens) if ref is None else ref

    def feed(self, cut):
        spans, want, rows = [], [], []
        for k, (name, n) in enumerate(cut.items()):
            done, left = self.tok[name]
            spans.append((self.slot[name], len(done), left[:n]))
            want += [(k, t) for t in range(n)]
            rows += [self.ref[name][len(done) + t] for t in range(n)]
            self.tok[name] = [done + left[:n], left[n:]]
        got = self.x.run(spans, want)
        e = rel(got, np.array(rows))
        i = int(e.argmax())
        assert e[i] < self.tol[self.m.dtype], (cut, want[i], e[i])

    def close(self, name):
        self.x.release(self.slot.pop(name))


def arrays(w):
    return {k: v.float().numpy() for k, v in w.items()}


def tokens(cfg, n, seed=3):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], size=n).astype(np.int32)


def write_dir(path, cfg, w):
    """a checkpoint directory: config.json and model.safetensors of bf16 tensors"""
    import torch
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    hdr, data, at = {}, [], 0
    for name, t in w.items():
        b = t.contiguous().view(torch.int16).numpy().tobytes()
        hdr[name] = {"dtype": "BF16", "shape": list(t.shape), "data_offsets": [at, at + len(b)]}
        data.append(b)
        at += len(b)
    h = json.dumps(hdr).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(h)) + h + b"".join(data))
