"""Plain numpy restatement of the Nufapel design and its mechanisms, one function per mechanism, token by token and head
by head, in float64.  Test infrastructure: it shares no code with the library, is slow, and keeps whole histories
where the library keeps state.

Layouts: activations [tokens, channels]; weights [out, in].
"""
import math

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def logsigmoid(z):
    return -np.logaddexp(0.0, -z)


def rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def dynamic_tanh(x, alpha, w, b):
    return np.tanh(alpha * x) * w + b


def gelu(z):
    """z Phi(z), Phi the normal distribution function."""
    return 0.5 * z * (1.0 + np.vectorize(math.erf, otypes=[float])(z / math.sqrt(2.0)))


def soft_cap(z, cap):
    return cap * np.tanh(z / cap) if cap else z


# ------------------------------------------------------------------ attention with a learned distance bias and a sink
def bucket(n, count, bias_max):
    """Row of the bias table for distance n: one row per distance in the lower half, a logarithmic scale up to bias_max above."""
    half = count // 2
    if n < half:
        return n
    return min(count - 1, half + int(math.floor(math.log(n / half) / math.log(bias_max / half) * (count - half) + 1e-9)))


def biased_sink_attention(q, k, v, scale, temp, rel, bias_max, sink):
    """q [T, H, D], k [T, G, D], v [T, G, Dv], temp [H], rel [B, H], sink [H] -> [T, H, Dv]."""
    T, H, _ = q.shape
    rep = H // k.shape[1]
    rows = np.array([bucket(n, rel.shape[0], bias_max) for n in range(T)])
    out = np.zeros((T, H, v.shape[2]))
    for t in range(T):
        for h in range(H):
            s = (k[:t + 1, h // rep] @ q[t, h]) * scale * temp[h] + rel[rows[t::-1], h]
            top = max(s.max(), sink[h])
            p = np.exp(s - top)
            out[t, h] = p @ v[:t + 1, h // rep] / (p.sum() + np.exp(sink[h] - top))
    return out


def left_mixer(h, p, m):
    T, H, G, D, Dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (h @ p["q"].T).reshape(T, H, D), (h @ p["k"].T).reshape(T, G, D), (h @ p["v"].T).reshape(T, G, Dv)
    o = biased_sink_attention(q, k, v, m["scale"], p["temp"], p["rel"], m["bias_max"], p["sink"])
    return (o * sigmoid(h @ p["g"].T)[:, :, None]).reshape(T, H * Dv) @ p["o"].T


# ------------------------------------------------------------------ matrix memory with exponential gates
def mlstm_recurrence(q, k, v, i, f, S, n, m):
    """q, k [T, H, D], v [T, H, Dv], log gates i, f [T, H]; S [H, D, Dv], n [H, D], m [H] changed in place; [T, H, Dv]."""
    out = np.zeros(v.shape)
    for t in range(q.shape[0]):
        new = np.maximum(f[t] + m, i[t])
        keep, add = np.exp(f[t] + m - new), np.exp(i[t] - new)
        S *= keep[:, None, None]
        S += add[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n *= keep[:, None]
        n += add[:, None] * k[t]
        m[:] = new
        den = np.maximum(np.abs(np.sum(n * q[t], axis=1)), np.exp(-m)) + 1e-6
        out[t] = np.einsum("hdv,hd->hv", S, q[t]) / den[:, None]
    return out


def log_gates(h, p, cap):
    i = cap * np.tanh((h @ p["i"].T + p["i.b"]) / cap)
    return i, logsigmoid(cap * np.tanh((h @ p["f"].T + p["f.b"]) / cap))


def right_mixer(h, p, m, eps):
    T, H, D, Dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ p["q"].T).reshape(T, H, D) * D ** -0.5
    k, v = (h @ p["k"].T).reshape(T, H, D), (h @ p["v"].T).reshape(T, H, Dv)
    i, f = log_gates(h, p, m["gate_cap"])
    o = mlstm_recurrence(q, k, v, i, f, np.zeros((H, D, Dv)), np.zeros((H, D)), np.zeros(H))
    return (rms(o, eps).reshape(T, H * Dv) * p["norm"] * sigmoid(h @ p["g"].T)) @ p["o"].T


def sub(p, name):
    return {k[len(name) + 1:]: v for k, v in p.items() if k.startswith(name + ".")}


def parallel_mixer(h, p, m, eps):
    left, right = left_mixer(h, sub(p, "left"), m["left"]), right_mixer(h, sub(p, "right"), m["right"], eps)
    return 0.5 * (rms(left, eps) * p["left.out"] + rms(right, eps) * p["right.out"])


# ------------------------------------------------------------------ generalised delta rule
def general_delta_recurrence(r, k, v, w, a, S):
    """r, k, w, a [T, H, D], v [T, H, Dv]; S [H, D, Dv] changed in place; [T, H, Dv]."""
    out = np.zeros(v.shape)
    for t in range(r.shape[0]):
        u = k[t] / np.sqrt(np.sum(k[t] * k[t], axis=1, keepdims=True) + 1e-6)
        seen = np.einsum("hd,hdv->hv", u, S)
        S[:] = w[t][:, :, None] * S - (a[t] * u)[:, :, None] * seen[:, None, :] + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, r[t])
    return out


def general_delta_mixer(h, p, m, eps):
    T, H, D = h.shape[0], m["heads"], m["dim"]
    r, k, v = ((h @ p[n].T).reshape(T, H, D) for n in "rkv")
    w = np.exp(-math.exp(-0.5) * sigmoid(np.tanh(h @ p["w1"].T) @ p["w2"].T + p["w0"])).reshape(T, H, D)
    a = sigmoid(h @ p["a"].T + p["a.b"]).reshape(T, H, D)
    o = general_delta_recurrence(r, k, v, w, a, np.zeros((H, D, D)))
    return (rms(o, eps).reshape(T, H * D) * p["norm"] * sigmoid(h @ p["g"].T)) @ p["o"].T


# ------------------------------------------------------------------ feed-forwards
def route(z, router):
    """z [experts]: (indices, weights) of the experts a token uses."""
    s = sigmoid(z)
    groups = router.get("groups") or {"count": 1, "keep": 1}
    size = len(s) // groups["count"]
    score = [sum(sorted(s[g * size:(g + 1) * size])[-2:]) for g in range(groups["count"])]
    kept = sorted(range(groups["count"]), key=lambda g: -score[g])[:groups["keep"]]
    allowed = [e for g in kept for e in range(g * size, (g + 1) * size)]
    chosen = sorted(allowed, key=lambda e: (-s[e], e))[:router["top"]]
    total = sum(s[e] for e in chosen) + 1e-20
    return chosen, [s[e] / total * router.get("scale", 1.0) for e in chosen]


def clamped_expert(x, p, limit):
    g = np.minimum(p["gate"] @ x, limit)
    u = np.clip(p["up"] @ x, -limit, limit)
    return p["down"] @ (g * sigmoid(1.702 * g) * (u + 1.0))


def feed_forward(h, p, mlp):
    if mlp["kind"] == "dense":
        return gelu(h @ p["up"].T) @ p["down"].T
    experts = [sub(p, "e%d" % e) for e in range(mlp["router"]["experts"])]
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in zip(*route(p["router"] @ h[t], mlp["router"])):
            out[t] += w * clamped_expert(h[t], experts[e], mlp["expert"]["limit"])
    return out


# ------------------------------------------------------------------ the model
def layer_runs(cfg):
    """[(layer index, pass number at the first layer of a pass, else None)] in the order they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    return ([(i, None) for i in range(a)] + [(i, t if i == a else None) for t in range(loop["times"]) for i in range(a, b)] +
            [(i, None) for i in range(b, n)])


def forward(cfg, params, tokens, taps=None):
    """Logits [T, vocab] of a whole sequence from its start; `taps`: list that receives the residual stream after every
    layer run."""
    P = {k: np.asarray(v, np.float64) for k, v in params.items()}
    eps = cfg["norm"]["eps"]
    norm = lambda x, n: dynamic_tanh(x, P[n + ".alpha"], P[n], P[n + ".b"])  # noqa: E731
    x = P["embed"][np.asarray(tokens)] + P["pos"][:len(tokens)]
    for i, t in layer_runs(cfg):
        if t is not None:
            x = x + P["loop.step"][t]
        entry, p = cfg["layers"][i], sub(P, "l%d" % i)
        h = norm(x, "l%d.norm1" % i)
        if entry["type"] == "parallel":
            y = parallel_mixer(h, sub(p, "mix"), entry["mixer"], eps)
        else:
            y = general_delta_mixer(h, sub(p, "mix"), entry["mixer"], eps)
        x = x + y * sigmoid(h @ p["rg1"].T + p["rg1.b"])
        if entry.get("mlp"):
            h = norm(x, "l%d.norm2" % i)
            x = x + feed_forward(h, sub(p, "mlp"), entry["mlp"]) * sigmoid(h @ p["rg2"].T + p["rg2.b"])
        if taps is not None:
            taps.append(x)
    return soft_cap(norm(x, "final.norm") @ P["head"].T, cfg.get("logit_softcap"))
