"""Small Bolopel models for the tests: configurations of their own and random bf16 weights."""
import math

import torch

from layered_helpers import arrays, tokens, write_dir  # noqa: F401


def delta(heads, kv, dim, vdim, conv, rank_a, rank_g, ff=None):
    """(config.json's layer, the ranks that only the tensors tell)"""
    return {"type": "channel_delta", "mixer": dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, conv=conv), "mlp": ff and dict(kind="dense", ff=ff)}, (rank_a, rank_g)


def parallel(left, window, scale, right, decay, ls, rs, ff=None):
    """left: heads, kv heads, dim, vdim; right: heads, dim, vdim"""
    l = dict(zip(("heads", "kv_heads", "dim", "vdim"), left), mask=dict(size=window), scale=scale)
    return {"type": "parallel", "mixer": dict(left=l, right=dict(zip(("heads", "dim", "vdim"), right), decay=list(decay)), left_scale=ls, right_scale=rs), "mlp": ff and dict(kind="dense", ff=ff)}, None


def model(width, vocab, eps, layers):
    return dict(architecture="Bolopel", width=width, vocab=vocab, norm=dict(eps=eps), layers=[l for l, _ in layers]), [r for _, r in layers]


# every branch, every layer with sizes of its own
MODELS = {
    "mixed": model(96, 151, 1e-5, [delta(4, 2, 24, 40, 3, 10, 18, 72), parallel((6, 2, 32, 16), 24, 0.3, (3, 20, 36), (0.5, 0.9, 0.999), 0.7, 1.3),
                                   parallel((4, 4, 16, 48), 7, 0.9, (2, 32, 16), (0.8, 0.97), 1.0, 0.4, 40), delta(3, 3, 64, 32, 4, 70, 9)]),
    # sizes no vector width divides (the plain attention form in bf16 too), one tap: no history
    "odd": model(75, 97, 1e-6, [delta(3, 1, 18, 21, 1, 5, 7, 51), parallel((3, 3, 18, 11), 13, 0.5, (2, 9, 14), (0.3, 0.95), 1.4, 0.8, 33), delta(2, 2, 33, 70, 6, 3, 65, 20)]),
    # sizes of one, a window of one position, no decay at all, equal scales
    "ones": model(64, 80, 1e-6, [parallel((1, 1, 8, 8), 1, 1.0, (1, 128, 24), (1.0,), 1.0, 1.0), delta(1, 1, 32, 32, 2, 1, 1, 64), delta(2, 1, 16, 24, 1, 1, 1)]),
    # query groups past one block of columns, larger heads, windows past a tile
    "wide": model(160, 300, 1e-6, [delta(2, 1, 128, 256, 4, 40, 64, 128), parallel((40, 1, 16, 32), 300, 0.4, (2, 256, 128), (0.9, 0.99), 1.1, 0.6, 64),
                                   parallel((4, 2, 192, 64), 90, 0.1, (4, 64, 64), (0.1, 0.6, 0.98, 0.9995), 0.9, 1.0), delta(6, 2, 256, 64, 4, 128, 12, 48)]),
    # the sizes the chunked prompt forms are made for
    "heads": model(128, 120, 1e-5, [delta(2, 2, 128, 128, 4, 128, 128, 96), parallel((4, 2, 64, 64), 128, 0.15, (2, 128, 128), (0.95, 0.998), 1.0, 0.7, 96), delta(4, 2, 64, 64, 4, 16, 16, 96)]),
}


def shapes(name_or_model):
    cfg, ranks = MODELS[name_or_model] if isinstance(name_or_model, str) else name_or_model
    C = cfg["width"]
    out = {"embed": (cfg["vocab"], C), "embed.norm": (C,), "final.norm": (C,), "head": (cfg["vocab"], C)}
    for i, (L, r) in enumerate(zip(cfg["layers"], ranks)):
        p, m = "l%d." % i, L["mixer"]
        out[p + "norm1"] = (C,)
        if L["type"] == "channel_delta":
            qd, vd, hd = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"], m["heads"] * m["dim"]
            q = p + "mix."
            out.update({q + "q": (qd, C), q + "k": (qd, C), q + "v": (vd, C), q + "q.conv": (qd, m["conv"]), q + "k.conv": (qd, m["conv"]), q + "v.conv": (vd, m["conv"]), q + "b": (m["heads"], C),
                        q + "A_log": (m["heads"],), q + "norm": (m["vdim"],), q + "a1": (r[0], C), q + "a2": (hd, r[0]), q + "dt_bias": (hd,), q + "g1": (r[1], C), q + "g2": (vd, r[1]), q + "o": (C, vd)})
        else:
            a, b = m["left"], m["right"]
            out.update({p + "mix.left." + n: s for n, s in dict(q=(a["heads"] * a["dim"], C), k=(a["kv_heads"] * a["dim"], C), v=(a["kv_heads"] * a["vdim"], C), o=(C, a["heads"] * a["vdim"])).items()})
            sq, sv = b["heads"] * b["dim"], b["heads"] * b["vdim"]
            out.update({p + "mix.right." + n: s for n, s in dict(q=(sq, C), k=(sq, C), v=(sv, C), g=(sv, C), o=(C, sv), norm=(sv,)).items()})
        if L["mlp"]:
            f = L["mlp"]["ff"]
            out.update({p + "norm2": (C,), p + "mlp.gate": (f, C), p + "mlp.up": (f, C), p + "mlp.down": (C, f)})
    return out


def weights(name_or_model, seed=0):
    """{name: torch.bfloat16}: unit-gain matrices, norm weights around 1; decays of a channel from nearly none to nearly all per token"""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, s in shapes(name_or_model).items():
        w = torch.randn(s, generator=g)
        leaf = name.split(".")[-1]
        if leaf.startswith("norm"):
            w = 1.0 + 0.2 * w
        elif leaf == "A_log":
            w = w - 0.5
        elif leaf == "dt_bias":
            w = 2.5 * w - 3.0
        elif leaf == "conv":
            w = w / math.sqrt(s[1])
        elif leaf == "embed":
            w = 1.5 * w
        elif len(s) == 2:
            w = w * (1.5 if leaf in ("q", "k") else 1.0) / math.sqrt(s[1])
        out[name] = w.to(torch.bfloat16)
    return out
