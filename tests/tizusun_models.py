"""Small Tizusun models for the tests: configurations of their own, random bf16 weights, and a writer for checkpoint directories."""
import torch

from layered_helpers import arrays, tokens, write_dir  # noqa: F401


def mixer(heads, kv, dim, chunk, rot, base=1000.0, scale=None, scaling=(8.0, 1.0, 4.0, 32)):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "mask": {"size": chunk}, "scale": dim ** -0.5 if scale is None else scale,
            "rot": {"base": base, "dims": rot, "scaling": dict(zip(("factor", "low", "high", "original"), scaling))}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def layer(mx, mlp):
    return {"type": "attention", "mixer": mx, "mlp": mlp}


# every branch, every layer with sizes of its own
CONFIGS = {
    "mixed": dict(width=96, vocab=151, postln_alpha=1.75, norm={"eps": 1e-5}, layers=[
        layer(mixer(6, 2, 32, 24, 16), moe(40, 6, 2)), layer(mixer(4, 4, 16, 7, 16, base=300.0), None), layer(mixer(5, 1, 48, 50, 32, scale=0.3), dense(72)),
        layer(mixer(8, 2, 24, 33, 4), moe(24, 5, 5))]),
    # sizes no vector width divides (the plain attention form in bf16 too), one query head per kv-head
    "odd": dict(width=75, vocab=97, postln_alpha=0.8, norm={"eps": 1e-6}, layers=[
        layer(mixer(3, 3, 18, 13, 10), dense(51)), layer(mixer(2, 1, 20, 40, 20, scaling=(2.0, 1.0, 2.0, 16)), moe(19, 3, 1))]),
    # a chunk of one position, a lone expert, a head wider than the stream
    "ones": dict(width=64, vocab=80, postln_alpha=1.0, norm={"eps": 1e-6}, layers=[
        layer(mixer(1, 1, 128, 1, 64), moe(32, 1, 1)), layer(mixer(2, 2, 32, 64, 2, scaling=(1.0, 1.0, 4.0, 64)), dense(64))]),
    # query groups past one block of columns, larger heads
    "wide": dict(width=160, vocab=300, postln_alpha=2.0, norm={"eps": 1e-6}, layers=[
        layer(mixer(40, 1, 16, 300, 8), dense(128)), layer(mixer(4, 2, 192, 90, 96), moe(64, 9, 3)), layer(mixer(2, 1, 256, 128, 256), moe(48, 4, 2))]),
}
CONFIGS = {k: dict(v, architecture="Tizusun") for k, v in CONFIGS.items()}


def shapes(cfg):
    C, out = cfg["width"], {"embed": (cfg["vocab"], cfg["width"]), "head": (cfg["vocab"], cfg["width"]), "final.norm": (cfg["width"],)}
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], "l%d." % i
        qd, kd = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
        out.update({p + "norm1": (C,), p + "mix.q": (qd, C), p + "mix.k": (kd, C), p + "mix.g": (qd, C), p + "mix.o": (C, qd), p + "mix.q.norm": (m["dim"],), p + "mix.k.norm": (m["dim"],)})
        f = L["mlp"]
        if f is None:
            continue
        out[p + "norm2"] = (C,)
        ff = f["ff"] if f["kind"] == "dense" else f["expert"]["ff"]
        for e in ([""] if f["kind"] == "dense" else ["e%d." % e for e in range(f["router"]["experts"])]):
            out.update({p + "mlp." + e + "gate": (ff, C), p + "mlp." + e + "up": (ff, C), p + "mlp." + e + "down": (C, ff)})
        if f["kind"] == "moe":
            out.update({p + "mlp.router": (f["router"]["experts"], C), p + "mlp.router.b": (f["router"]["experts"],)})
    return out


def weights(cfg, seed=0, qk=1.5, settled=False):
    """{name: torch.bfloat16}: unit-gain matrices, norm weights around 1 (`qk` for the q / k norms: how peaked the attention is).  settled: routers whose biases keep the chosen
    experts apart from the rest (a bf16 run and the float64 one must choose alike; which expert is chosen by a close call is not what a model-level test is about)"""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, s in shapes(cfg).items():
        w = torch.randn(s, generator=g)
        if name.endswith("norm") or name.endswith("norm1") or name.endswith("norm2"):
            w = (qk if ".mix." in name else 1.0) * (1.0 + 0.2 * w)
        elif name.endswith("router"):
            w = w * (0.2 if settled else 2.0) / s[1] ** 0.5
        elif settled and name.endswith("router.b"):
            w = torch.randperm(s[0], generator=g).float()
        elif name == "embed":
            pass
        elif len(s) == 2:
            w = w * (2.0 if name.endswith((".k", ".o", ".down")) else 1.0) / s[1] ** 0.5
        out[name] = w.to(torch.bfloat16)
    return out
