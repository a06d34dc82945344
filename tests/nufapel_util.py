"""Small Nufapel models for the tests: configurations as a config.json states them and random weights that give every
mechanism something to get wrong (files, loading and running: hybrid_util)."""
import numpy as np

from lumen_amd import synth


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, groups=None, scale=1.5, limit=1.5):
    r = {"experts": experts, "top": top, "scale": scale}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": r}


def general(heads, dim, mlp=None):
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim}, "mlp": mlp}


def parallel(left, right, mlp=None, bias_max=40, scale=None, cap=6.0):
    """left: (heads, kv_heads, dim, vdim), right: (heads, dim, vdim)."""
    h, g, d, v = left
    return {"type": "parallel", "mlp": mlp,
            "mixer": {"left": {"heads": h, "kv_heads": g, "dim": d, "vdim": v, "bias_max": bias_max, "scale": scale or d ** -0.5},
                      "right": {"heads": right[0], "dim": right[1], "vdim": right[2], "gate_cap": cap}}}


def config(width, vocab, layers, loop=None, eps=1e-5, softcap=9.0, positions=900):
    cfg = {"architecture": "Nufapel", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "max_positions": positions}
    if softcap:
        cfg["logit_softcap"] = softcap
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def shapes(cfg, rank=5, bias_rows=12):
    """Tensor shapes of the design, written down from its equations (not taken from the library)."""
    W, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, W), "pos": (cfg["max_positions"], W), "head": (V, W)}

    def norm(name):
        s.update({name: (W,), name + ".b": (W,), name + ".alpha": ()})
    norm("final.norm")
    if cfg.get("loop"):
        s["loop.step"] = (cfg["loop"]["times"], W)
    for i, e in enumerate(cfg["layers"]):
        p, m = "l%d." % i, e["mixer"]
        norm(p + "norm1")
        s.update({p + "rg1": (W, W), p + "rg1.b": (W,)})
        if e["type"] == "general_delta":
            n = m["heads"] * m["dim"]
            s.update({p + "mix." + x: (n, W) for x in "rkvga"})
            s.update({p + "mix.a.b": (n,), p + "mix.w1": (rank, W), p + "mix.w2": (n, rank), p + "mix.w0": (n,), p + "mix.norm": (n,), p + "mix.o": (W, n)})
        else:
            a, r = m["left"], m["right"]
            x, H, G = p + "mix.left.", a["heads"], a["kv_heads"]
            s.update({x + "q": (H * a["dim"], W), x + "k": (G * a["dim"], W), x + "v": (G * a["vdim"], W), x + "rel": (bias_rows, H), x + "temp": (H,),
                      x + "sink": (H,), x + "g": (H, W), x + "o": (W, H * a["vdim"]), x + "out": (W,)})
            x, H, n = p + "mix.right.", r["heads"], r["heads"] * r["vdim"]
            s.update({x + "q": (H * r["dim"], W), x + "k": (H * r["dim"], W), x + "v": (n, W), x + "g": (n, W), x + "o": (W, n), x + "norm": (n,),
                      x + "i": (H, W), x + "i.b": (H,), x + "f": (H, W), x + "f.b": (H,), x + "out": (W,)})
        if e["mlp"]:
            norm(p + "norm2")
            s.update({p + "rg2": (W, W), p + "rg2.b": (W,)})
            if e["mlp"]["kind"] == "dense":
                s.update({p + "mlp.up": (e["mlp"]["ff"], W), p + "mlp.down": (W, e["mlp"]["ff"])})
            else:
                F, E = e["mlp"]["expert"]["ff"], e["mlp"]["router"]["experts"]
                s[p + "mlp.router"] = (E, W)
                for k in range(E):
                    x = p + "mlp.e%d." % k
                    s.update({x + "gate": (F, W), x + "up": (F, W), x + "down": (W, F)})
    return s


def make_params(cfg, seed=0, rank=5, bias_rows=12):
    """Values bf16 represents exactly, so both storages hold the same model."""
    return {n: synth.bf16_widen(synth.bf16_round(synth.nufapel_param(n, sh, seed))).reshape(sh) for n, sh in shapes(cfg, rank, bias_rows).items()}


def sharpen(params, factor=3.0):
    """Larger queries: attention scores that stand out among hundreds."""
    for n in params:
        if n.endswith("left.q"):
            params[n] = synth.bf16_widen(synth.bf16_round(params[n] * np.float32(factor)))
    return params
