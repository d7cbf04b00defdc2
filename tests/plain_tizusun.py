"""A plain, slow statement of the Tizusun decoder in numpy float64: one function per mechanism, whole sequences, no cache.

Test infrastructure only.  It shares no code with koifish_amd: the product's kernels, its loader and its state manager are compared with what this file computes.
A model is (config dict, {tensor name: numpy array}); config has the layout of a Tizusun config.json.
"""
import math

import numpy as np


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def relu(z):
    return np.maximum(z, 0.0)


def softmax(s):
    e = np.exp(s - np.max(s, axis=-1, keepdims=True))
    return e / np.sum(e, axis=-1, keepdims=True)


def rope_frequencies(base, dims, scaling):
    """the dims / 2 angular frequencies: fast ones kept, slow ones divided by `factor`, a blend between (piecewise in the number of turns over `original` positions)"""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling:
            factor, low, high, original = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
            turns = original / (2.0 * math.pi / f)
            if turns < low:
                f = f / factor
            elif turns <= high:
                kept = (turns - low) / (high - low)
                f = kept * f + (1.0 - kept) * (f / factor)
        out.append(f)
    return np.array(out)


def rope(x, positions, freqs):
    """x [T, heads, dim]: the first 2 len(freqs) dimensions rotated in pairs (i, i + len(freqs)), the rest passed through"""
    n = len(freqs)
    a = positions[:, None, None] * freqs[None, None, :]
    u, v = x[..., :n], x[..., n:2 * n]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a), x[..., 2 * n:]], axis=-1)


def chunk_mask(T, size):
    """visible[i, j]: j is not after i and lies in i's chunk of `size` positions counted from 0 (size 0: no chunks)"""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & ((i // size == j // size) if size else True)


def attend(q, v, gate, qn, kn, mx, eps):
    """one sequence's heads: q [T, H, D], v [T, G, D] (the key projection: value as it is, key after norm and rotation), gate [T, H * D] before the sigmoid -> [T, H * D]"""
    T, H, D = q.shape
    G = v.shape[1]
    q, k = rms_norm(q, qn, eps), rms_norm(v, kn, eps)
    freqs = rope_frequencies(mx["rot"]["base"], mx["rot"]["dims"], mx["rot"].get("scaling"))
    pos = np.arange(T, dtype=np.float64)
    q, k = rope(q, pos, freqs), rope(k, pos, freqs)
    seen = chunk_mask(T, mx["mask"]["size"] if mx.get("mask") else 0)
    out = np.zeros((T, H, D))
    for n in range(H):
        g = n // (H // G)
        s = np.where(seen, (q[:, n] @ k[:, g].T) * mx["scale"], -np.inf)
        out[:, n] = softmax(s) @ v[:, g]
    return out.reshape(T, H * D) * sigmoid(gate)


def attention(h, W, mx, eps):
    """h [T, width] -> [T, width]; W(name) gives the mixer's tensors"""
    T, H, G, D = h.shape[0], mx["heads"], mx["kv_heads"], mx["dim"]
    heads = attend((h @ W("q").T).reshape(T, H, D), (h @ W("k").T).reshape(T, G, D), h @ W("g").T, W("q.norm"), W("k.norm"), mx, eps)
    return heads @ W("o").T


def gated_ff(h, gate, up, down, act):
    return (act(h @ gate.T) * (h @ up.T)) @ down.T


def route(h, router, bias, top):
    """[T, experts] weights: softmax over the `top` largest logits, zero elsewhere"""
    z = h @ router.T + bias
    out = np.zeros_like(z)
    for t in range(z.shape[0]):
        chosen = np.argsort(-z[t], kind="stable")[:top]
        out[t, chosen] = softmax(z[t, chosen])
    return out


def mixture(h, W, mlp):
    w = route(h, W("router"), W("router.b"), mlp["router"]["top"])
    out = np.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows = np.nonzero(w[:, e])[0]
        if len(rows):
            out[rows] += w[rows, e:e + 1] * gated_ff(h[rows], W("e%d.gate" % e), W("e%d.up" % e), W("e%d.down" % e), silu)
    return out


def layer(x, i, cfg, P):
    lay, eps, alpha = cfg["layers"][i], cfg["norm"]["eps"], cfg["postln_alpha"]
    x = rms_norm(alpha * x + attention(x, lambda n: P["l%d.mix.%s" % (i, n)], lay["mixer"], eps), P["l%d.norm1" % i], eps)
    mlp = lay.get("mlp")
    if mlp is None:
        return x
    W = lambda n: P["l%d.mlp.%s" % (i, n)]
    y = gated_ff(x, W("gate"), W("up"), W("down"), relu) if mlp["kind"] == "dense" else mixture(x, W, mlp)
    return rms_norm(alpha * x + y, P["l%d.norm2" % i], eps)


def forward(cfg, P, tokens, want_layers=False):
    """logits [T, vocab] (and the residual stream after every layer)"""
    P = {k: np.asarray(v, dtype=np.float64) for k, v in P.items()}
    x = P["embed"][np.asarray(tokens)]
    streams = []
    for i in range(len(cfg["layers"])):
        x = layer(x, i, cfg, P)
        streams.append(x)
    logits = rms_norm(x, P["final.norm"], cfg["norm"]["eps"]) @ P["head"].T
    return (logits, np.stack(streams)) if want_layers else logits


def greedy(cfg, P, prompt, n_new):
    seq = list(prompt)
    for _ in range(n_new):
        seq.append(int(np.argmax(forward(cfg, P, seq)[-1])))
    return seq[len(prompt):]
