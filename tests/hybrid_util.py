"""Small models of the layered hybrid decoder for the tests: configurations as a config.json states them, random weights
that give every mechanism something to get wrong, and the files a model folder holds."""
import json
import os

import numpy as np

from lumen_amd import synth


def attention(heads, kv_heads, dim, vdim, window, scale=None, softcap=20.0, ff=0):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window},
                                           "scale": scale or dim ** -0.5, "softcap": softcap},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def wkv(heads, dim, ff=0):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def delta(heads, kv_heads, dim, vdim, conv=3, ff=0):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(width, vocab, layers, loop=None, eps=1e-5, residual_mult=0.9, scale=3.0):
    cfg = {"architecture": "Pinavik", "width": width, "vocab": vocab, "layers": layers, "embedding": {"scale": scale},
           "norm": {"eps": eps}, "residual_mult": residual_mult}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return cfg


def shapes(cfg, ranks=(5, 11)):
    """Tensor shapes of the design, written down from its equations (not taken from the library)."""
    W, V = cfg["width"], cfg["vocab"]
    s = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    if cfg.get("loop"):
        s["loop.in"], s["loop.step"] = (W, 2 * W), (cfg["loop"]["times"], W)
    for i, e in enumerate(cfg["layers"]):
        p, m = "l%d." % i, e["mixer"]
        H, D = m["heads"], m["dim"]
        G, Dv = m.get("kv_heads", H), m.get("vdim", D)
        lo, hi = ranks
        x = {"o": (W, H * Dv)}
        if e["type"] == "attention":
            x.update({"q": (H * D, W), "k": (G * D, W), "v": (G * Dv, W), "g": (H * Dv, W), "q.norm": (H * D,), "k.norm": (G * D,),
                      "r1": (H,), "r2": (H,)})
        elif e["type"] == "wkv":
            x.update({n: (H * D, W) for n in "rkvg"})
            x.update({"mu." + n: (W,) for n in "rkvgw"})
            x.update({"w1": (lo, W), "w2": (H * D, lo), "w0": (H * D,), "u": (H, D), "norm": (H * D,)})
        else:
            c = m["conv"]
            x.update({"q": (G * D, W), "k": (G * D, W), "v": (H * Dv, W), "q.conv": (G * D, c), "k.conv": (G * D, c), "v.conv": (H * Dv, c),
                      "b": (H, W), "A_log": (H,), "norm": (Dv,), "a1": (lo, W), "a2": (H * D, lo), "dt_bias": (H * D,), "g1": (hi, W),
                      "g2": (H * Dv, hi)})
        s.update({p + "mix." + n: v for n, v in x.items()})
        s[p + "norm1"] = (W,)
        if e["mlp"]:
            s[p + "norm2"] = (W,)
            s.update({p + "mlp.up": (e["mlp"]["ff"], W), p + "mlp.down": (W, e["mlp"]["ff"]), p + "mlp.act": (4,)})
    return s


def make_params(cfg, seed=0, ranks=(5, 11)):
    """Random weights whose values bf16 represents exactly (both storages then hold the same model)."""
    out = {}
    for n, sh in shapes(cfg, ranks).items():
        a = synth.hybrid_param(n, sh, seed)
        out[n] = synth.bf16_widen(synth.bf16_round(a))
    return out


def write_model(folder, cfg, params):
    """config.json and a bf16 safetensors file."""
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    head, blobs, at = {}, [], 0
    for n, a in params.items():
        b = synth.bf16_round(a).tobytes()
        head[n] = {"dtype": "BF16", "shape": list(a.shape), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    h = json.dumps(head).encode()
    with open(os.path.join(folder, "model.safetensors"), "wb") as f:
        f.write(len(h).to_bytes(8, "little") + h + b"".join(blobs))
    return str(folder)


def load(tmp_path, cfg, params, dtype="float32", max_seq_len=512):
    from lumen_amd.registry import load_model
    return load_model(write_model(tmp_path, cfg, params), dtype, max_seq_len)


def run(model, tokens, cuts, residual=False):
    """All tokens' logits with the sequence cut into portions of the given sizes (the last size repeats)."""
    model.reset()
    rows, taps, at, i = [], [], 0, 0
    while at < len(tokens):
        n = min(cuts[min(i, len(cuts) - 1)], len(tokens) - at)
        r = model.step(tokens[at:at + n], np.arange(n), **({"residual": True} if residual else {}))
        if residual:
            taps.append(r[1])
            r = r[0]
        rows.append(r)
        at += n
        i += 1
    logits = np.concatenate(rows)
    return (logits, np.concatenate(taps, 1)) if residual else logits
