"""A plain, slow statement of the Bolopel decoder in numpy float64: one function per mechanism, whole sequences token by token, no cache.

Test infrastructure only.  It shares no code with koifish_amd: the product's kernels, its loader and its state manager are compared with what this file computes.
A model is (config dict, {tensor name: numpy array}); config has the layout of a Bolopel config.json.
"""
import numpy as np


def sigmoid(z):
    e = np.exp(-np.abs(z))
    return np.where(z >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def by_rms(x, eps):
    """the last axis divided by its root mean square"""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x, w, eps):
    d = x - np.mean(x, axis=-1, keepdims=True)
    return d / np.sqrt(np.mean(d * d, axis=-1, keepdims=True) + eps) * w


def sinusoid(positions, width):
    """row p: sin and cos of p / 10000^(2 i / width) side by side"""
    c = np.arange(width)
    a = np.asarray(positions, dtype=np.float64)[:, None] * 10000.0 ** (-2.0 * (c // 2) / width)
    return np.where(c % 2 == 0, np.sin(a), np.cos(a))


def short_conv(x, taps):
    """x [T, channels], taps [channels, n]: y_t = sum over j of taps[:, n - 1 - j] x_(t - j), zeros before the start"""
    y, n = np.zeros_like(x), taps.shape[1]
    for j in range(min(n, len(x))):
        y[j:] += taps[:, n - 1 - j] * x[:len(x) - j]
    return y


def unit(x):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + 1e-6)


def delta_rule(q, k, v, g, beta, S=None):
    """one head: q, k, g [T, dim], v [T, vdim], beta [T] -> ([T, vdim], last state [dim, vdim]).  Decay by rows, then the write of what k does not recall yet, then the read"""
    T, V = v.shape
    S = np.zeros((k.shape[1], V)) if S is None else S.copy()
    o = np.zeros((T, V))
    for t in range(T):
        S = g[t][:, None] * S
        S = S + np.outer(k[t], beta[t] * (v[t] - k[t] @ S))
        o[t] = q[t] @ S
    return o, S


def decays(h, W, heads, dim):
    """[T, heads, dim] factors in (0, 1)"""
    z = (h @ W("a1").T) @ W("a2").T + W("dt_bias")
    return np.exp(-np.exp(W("A_log"))[None, :, None] * softplus(z).reshape(len(h), heads, dim))


def channel_delta(h, W, mx, eps):
    T, H, G, D, V = len(h), mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (silu(short_conv(h @ W(n).T, W(n + ".conv"))) for n in ("q", "k", "v"))
    q, k, v = unit(q.reshape(T, G, D)) * D ** -0.5, unit(k.reshape(T, G, D)), v.reshape(T, H, V)
    g, beta = decays(h, W, H, D), sigmoid(h @ W("b").T)
    o = np.stack([delta_rule(q[:, n // (H // G)], k[:, n // (H // G)], v[:, n], g[:, n], beta[:, n])[0] for n in range(H)], axis=1)
    gate = sigmoid((h @ W("g1").T) @ W("g2").T)
    return ((by_rms(o, eps) * W("norm")).reshape(T, H * V) * gate) @ W("o").T


def window_mask(T, size):
    """visible[i, j]: j is i or one of the size - 1 positions before it"""
    d = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (d >= 0) & (d < size)


def softmax_with_sink(s):
    """rows of scores (-inf: not visible): exp(s) / (1 + sum exp(s))"""
    m = np.maximum(np.max(s, axis=-1, keepdims=True), 0.0)
    e = np.exp(s - m)
    return e / (np.exp(-m) + np.sum(e, axis=-1, keepdims=True))


def attend(q, k, v, scale, window, eps):
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H * vdim]"""
    T, H, _ = q.shape
    G = k.shape[1]
    q, k, seen = by_rms(q, eps), by_rms(k, eps), window_mask(T, window)
    out = np.stack([softmax_with_sink(np.where(seen, q[:, n] @ k[:, n // (H // G)].T * scale, -np.inf)) @ v[:, n // (H // G)] for n in range(H)], axis=1)
    return out.reshape(T, -1)


def window_attention(h, W, mx, eps):
    T, H, G = len(h), mx["heads"], mx["kv_heads"]
    return attend((h @ W("q").T).reshape(T, H, -1), (h @ W("k").T).reshape(T, G, -1), (h @ W("v").T).reshape(T, G, -1), mx["scale"], mx["mask"]["size"], eps) @ W("o").T


def decayed_sum(q, k, v, decay, S=None):
    """one head: S <- decay S + k v^T, o = S^T q; ([T, vdim], last state)"""
    S = np.zeros((k.shape[1], v.shape[1])) if S is None else S.copy()
    o = np.zeros_like(v)
    for t in range(len(v)):
        S = decay * S + np.outer(k[t], v[t])
        o[t] = q[t] @ S
    return o, S


def lightning(h, W, mx, eps):
    T, H = len(h), mx["heads"]
    q, k, v = (silu(h @ W(n).T).reshape(T, H, -1) for n in ("q", "k", "v"))
    o = np.concatenate([decayed_sum(q[:, n], k[:, n], v[:, n], mx["decay"][n])[0] for n in range(H)], axis=1)
    return (by_rms(o, eps) * W("norm") * sigmoid(h @ W("g").T)) @ W("o").T


def parallel(h, W, mx, eps):
    return mx["left_scale"] * window_attention(h, lambda n: W("left." + n), mx["left"], eps) + mx["right_scale"] * lightning(h, lambda n: W("right." + n), mx["right"], eps)


def dense(h, W):
    return (silu(h @ W("gate").T) * (h @ W("up").T)) @ W("down").T


MIXERS = {"channel_delta": channel_delta, "parallel": parallel}


def layer(x, i, cfg, P):
    lay, eps = cfg["layers"][i], cfg["norm"]["eps"]
    x = x + layer_norm(MIXERS[lay["type"]](x, lambda n: P["l%d.mix.%s" % (i, n)], lay["mixer"], eps), P["l%d.norm1" % i], eps)
    if lay.get("mlp") is None:
        return x
    return x + layer_norm(dense(x, lambda n: P["l%d.mlp.%s" % (i, n)]), P["l%d.norm2" % i], eps)


def embed(cfg, P, tokens):
    return layer_norm(P["embed"][np.asarray(tokens)] + sinusoid(np.arange(len(tokens)), cfg["width"]), P["embed.norm"], cfg["norm"]["eps"])


def forward(cfg, P, tokens, want_layers=False):
    """logits [T, vocab] (and the residual stream after every layer)"""
    P = {k: np.asarray(v, dtype=np.float64) for k, v in P.items()}
    x = embed(cfg, P, tokens)
    streams = []
    for i in range(len(cfg["layers"])):
        x = layer(x, i, cfg, P)
        streams.append(x)
    logits = layer_norm(x, P["final.norm"], cfg["norm"]["eps"]) @ P["head"].T
    return (logits, np.stack(streams)) if want_layers else logits


def greedy(cfg, P, prompt, n_new):
    seq = list(prompt)
    for _ in range(n_new):
        seq.append(int(np.argmax(forward(cfg, P, seq)[-1])))
    return seq[len(prompt):]
