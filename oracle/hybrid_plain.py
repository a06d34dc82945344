"""Plain numpy restatement of the layered hybrid decoder (Pinavik and its mechanisms), one function per mechanism,
token by token and head by head, in float64.  Test infrastructure: it shares no code with the library, is slow, and
keeps whole histories where the library keeps rolling state.

Layouts: activations [tokens, channels]; weights [out, in].
"""
import numpy as np


def rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def zero_centred_norm(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def polynorm(z, abce, eps):
    a, b, c, e = abce
    return a * rms(z, eps) + b * rms(z ** 2, eps) + c * rms(z ** 3, eps) + e


def causal_conv_silu(x, taps):
    """Depthwise causal convolution over time, [T, C] with taps [C, n] (last column: the current token), then SiLU."""
    T, n = x.shape[0], taps.shape[1]
    out = np.zeros_like(x)
    for t in range(T):
        for j in range(n):
            src = t - (n - 1) + j
            if src >= 0:
                out[t] += taps[:, j] * x[src]
    return silu(out)


def unit(x, eps=1e-6):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + eps)


def window_attention(q, k, v, scale, softcap, r1, r2, window):
    """q [T, H, D], k [T, G, D], v [T, G, Dv]; head h reads key/value head h // (H/G); scores squashed by
    softcap * tanh(. / softcap), less r1[h] ln(1 + r2[h] distance), over the last `window` tokens.  [T, H, Dv]."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        lo = max(0, t - window + 1) if window else 0
        dist = t - np.arange(lo, t + 1)
        for h in range(H):
            s = k[lo:t + 1, h // rep] @ q[t, h] * scale
            if softcap:
                s = softcap * np.tanh(s / softcap)
            s = s - r1[h] * np.log1p(r2[h] * dist)
            p = np.exp(s - s.max())
            out[t, h] = (p / p.sum()) @ v[lo:t + 1, h // rep]
    return out


def attention_mixer(h, p, L, eps):
    H, G, D, Dv = L["heads"], L["kv_heads"], L["dim"], L["vdim"]
    T = h.shape[0]
    q = rms(h @ p["q"].T, eps) * p["q.norm"]
    k = rms(h @ p["k"].T, eps) * p["k.norm"]
    v = h @ p["v"].T
    o = window_attention(q.reshape(T, H, D), k.reshape(T, G, D), v.reshape(T, G, Dv), L["scale"], L["softcap"],
                         p["r1"], p["r2"], L["window"]).reshape(T, H * Dv)
    return (o * sigmoid(h @ p["g"].T)) @ p["o"].T


def wkv_recurrence(r, k, v, w, u, S):
    """r, k, w [T, H, D], v [T, H, Dv], u [H, D], S [H, D, Dv] (changed in place); o [T, H, Dv]."""
    out = np.zeros(v.shape)
    for t in range(r.shape[0]):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hd,hdv->hv", r[t], S + u[:, :, None] * kv)
        S *= w[t][:, :, None]
        S += kv
    return out


def wkv_mixer(h, p, L, eps):
    H, D, T = L["heads"], L["dim"], h.shape[0]
    prev = np.concatenate([np.zeros((1, h.shape[1])), h[:-1]])
    mix = {s: h + (prev - h) * p["mu." + s] for s in "rkvgw"}
    r, k, v = ((mix[s] @ p[s].T).reshape(T, H, D) for s in "rkv")
    gate = silu(mix["g"] @ p["g"].T)
    w = np.exp(-np.exp(np.tanh(mix["w"] @ p["w1"].T) @ p["w2"].T + p["w0"])).reshape(T, H, D)
    o = wkv_recurrence(r, k, v, w, p["u"], np.zeros((H, D, D)))
    return (rms(o, eps).reshape(T, H * D) * p["norm"] * gate) @ p["o"].T


def delta_recurrence(q, k, v, g, beta, S):
    """q, k, g [T, H, D], v [T, H, Dv], beta [T, H], S [H, D, Dv] (changed in place); o [T, H, Dv]."""
    out = np.zeros(v.shape)
    for t in range(q.shape[0]):
        S *= g[t][:, :, None]
        u = beta[t][:, None] * (v[t] - np.einsum("hdv,hd->hv", S, k[t]))
        S += k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t])
    return out


def channel_delta_mixer(h, p, L, eps):
    H, G, D, Dv, T = L["heads"], L["kv_heads"], L["dim"], L["vdim"], h.shape[0]
    q = unit(causal_conv_silu(h @ p["q"].T, p["q.conv"]).reshape(T, G, D)) * D ** -0.5
    k = unit(causal_conv_silu(h @ p["k"].T, p["k.conv"]).reshape(T, G, D))
    v = causal_conv_silu(h @ p["v"].T, p["v.conv"]).reshape(T, H, Dv)
    q, k = np.repeat(q, H // G, axis=1), np.repeat(k, H // G, axis=1)
    beta = sigmoid(h @ p["b"].T)
    z = softplus((h @ p["a1"].T) @ p["a2"].T + p["dt_bias"]).reshape(T, H, D)
    g = np.exp(-np.exp(p["A_log"])[None, :, None] * z)
    o = delta_recurrence(q, k, v, g, beta, np.zeros((H, D, Dv)))
    gate = sigmoid((h @ p["g1"].T) @ p["g2"].T)
    return ((rms(o, eps) * p["norm"]).reshape(T, H * Dv) * gate) @ p["o"].T


MIXERS = {"attention": attention_mixer, "wkv": wkv_mixer, "channel_delta": channel_delta_mixer}


def layer_runs(cfg):
    """[(layer index, pass number or None at all but the first layer of a pass)] in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop["times"]
    runs = [(i, None) for i in range(a)]
    for t in range(times):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


def flat_layer(entry):
    m = dict(entry["mixer"])
    m["window"] = (m.get("mask") or {}).get("size", 0)
    return m


def forward(cfg, params, tokens, taps=None):
    """Logits [T, vocab] of a whole sequence from its start; `taps`: list that receives the residual stream after
    every layer run."""
    P = {k: np.asarray(v, np.float64) for k, v in params.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x0 = P["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
    x = x0
    for i, t in layer_runs(cfg):
        if t is not None:
            x = np.concatenate([x, x0], axis=1) @ P["loop.in"].T + P["loop.step"][t]
        entry, pre = cfg["layers"][i], "l%d." % i
        mp = {k[len(pre) + 4:]: v for k, v in P.items() if k.startswith(pre + "mix.")}
        x = x + m * MIXERS[entry["type"]](zero_centred_norm(x, P[pre + "norm1"], eps), mp, flat_layer(entry), eps)
        if entry.get("mlp"):
            z = zero_centred_norm(x, P[pre + "norm2"], eps) @ P[pre + "mlp.up"].T
            x = x + m * (polynorm(z, P[pre + "mlp.act"], eps) @ P[pre + "mlp.down"].T)
        if taps is not None:
            taps.append(x)
    return zero_centred_norm(x, P["final.norm"], eps) @ P["head"].T
