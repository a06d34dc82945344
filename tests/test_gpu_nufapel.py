"""Nufapel on the GPU against its plain restatement (oracle/nufapel_plain.py): every mechanism alone through the C ABI, then
whole models -- prompts, decoding, portions, reuse, generation."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from gpu_util import max_rel
import hybrid_util as hu
import nufapel_util as nu
from oracle import nufapel_plain as npn
from test_gpu_hybrid import CUTS, L, rng, tokens_of  # noqa: F401  (L: the fixture)

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
LOG2E = 1.4426950408889634


def f32(r, *shape):
    return r.standard_normal(shape).astype(np.float32)


def d(x):
    return np.asarray(x, np.float64)


# ------------------------------------------------------------------ mechanisms
@pytest.mark.parametrize("rows,dim", [(1, 1), (3, 7), (2, 64), (3, 1000), (1, 4097)])
def test_dynamic_tanh(L, rows, dim):  # noqa: F811
    r = rng(rows, dim)
    x, w, b = f32(r, rows, dim) * 3, f32(r, dim), f32(r, dim)
    out = L.out(rows, dim)
    L.call("lumen_dynamic_tanh_f32", L.dev(x), L.dev([0.7]), L.dev(w), L.dev(b), out, rows, dim)
    assert max_rel(out.data(), npn.dynamic_tanh(d(x), np.float32(0.7), d(w), d(b))) < 1e-6


@pytest.mark.parametrize("rows,dim,width", [(1, 4, 3), (3, 40, 37), (20, 64, 64), (2, 2048, 2048), (17, 4104, 4099), (1, 16384, 16384)])
def test_gated_residual_of_one_and_of_a_pair(L, rows, dim, width):  # noqa: F811
    r = rng(rows, dim)
    x, y, y2, w1, w2, gate, gb = f32(r, rows, dim), f32(r, rows, dim), f32(r, rows, dim) * 5, f32(r, dim), f32(r, dim), f32(r, rows, dim), f32(r, dim)
    for a in (y, y2):
        a[:, width:] = 0
    out = L.out(rows, dim)
    L.call("lumen_gated_residual_f32", L.dev(x), L.dev(y), None, None, None, L.dev(gate), L.dev(gb), out, rows, dim, width, 1.0, 0.0)
    g = npn.sigmoid(d(gate) + d(gb))
    assert max_rel(out.data(), d(x) + g * d(y)) < 1e-6
    L.call("lumen_gated_residual_f32", L.dev(x), L.dev(y), L.dev(y2), L.dev(w1), L.dev(w2), L.dev(gate), L.dev(gb), out, rows, dim, width, 0.5, 1e-2)
    v = 0.5 * (npn.rms(d(y)[:, :width], 1e-2) * w1[:width] + npn.rms(d(y2)[:, :width], 1e-2) * w2[:width])
    assert max_rel(out.data()[:, :width], d(x)[:, :width] + g[:, :width] * v) < 2e-6


@pytest.mark.parametrize("heads,dim,vdim", [(1, 3, 4), (2, 16, 16), (3, 48, 20), (2, 64, 64), (1, 100, 70), (2, 128, 128), (1, 200, 33)])
def test_general_delta_recurrence(L, heads, dim, vdim):  # noqa: F811
    """Whole, token by token and in portions: same outputs, same state; keys with much in common, rates near 0 and near 1."""
    T = 100
    r = rng(heads, dim, vdim)
    R, K, V, z, a = f32(r, T, heads, dim), f32(r, T, heads, dim) + 1, f32(r, T, heads, vdim), f32(r, T, heads, dim) * 2, f32(r, T, heads, dim)
    zb = np.linspace(-9, 9, heads * dim).astype(np.float32).reshape(heads, dim)
    ab = np.linspace(6, -6, heads * dim).astype(np.float32).reshape(heads, dim)
    S = np.zeros((heads, dim, vdim))
    w = np.exp(-np.exp(-0.5) * npn.sigmoid(d(z) + zb))
    want = npn.general_delta_recurrence(d(R), d(K), d(V), w, npn.sigmoid(d(a) + ab), S)
    rows = L.state_rows(dim)
    for cuts in CUTS:
        state, got, at, i = L.out(heads, vdim, rows), [], 0, 0
        while at < T:
            n = min(cuts[min(i, len(cuts) - 1)], T - at)
            o, sl = L.out(n, heads, vdim), slice(at, at + n)
            L.call("lumen_general_delta_f32", L.dev(R[sl]), L.dev(K[sl]), L.dev(V[sl]), L.dev(z[sl]), L.dev(a[sl]), L.dev(zb), L.dev(ab), state, o, n,
                   heads, dim, vdim, 1e-6)
            got.append(o.data())
            at += n
            i += 1
        assert max_rel(np.concatenate(got), want) < 2e-5, cuts
        st = state.data()
        assert max_rel(st[:, :, :dim].transpose(0, 2, 1), S) < 2e-5, cuts
        assert not st[:, :, dim:].any()


@pytest.mark.parametrize("heads,dim,vdim,T", [(1, 3, 4, 100), (2, 16, 15, 100), (3, 48, 20, 100), (2, 64, 64, 300), (1, 100, 130, 100), (1, 256, 256, 60)])
def test_matrix_memory(L, heads, dim, vdim, T):  # noqa: F811
    """Heads whose gates sit at either cap, whose inputs come and go, and whose running maximum moves both ways; whole, token
    by token and in portions."""
    r = rng(heads, dim, vdim)
    q, k, v, i, f = f32(r, T, heads, dim), f32(r, T, heads, dim), f32(r, T, heads, vdim), f32(r, T, heads) * 8, f32(r, T, heads) * 4
    ib, fb, gain = np.linspace(-4, 4, heads).astype(np.float32), np.linspace(5, 0, heads).astype(np.float32), 1 + 0.2 * f32(r, heads, vdim)
    i[30:50] -= 30
    cap, eps = 5.0, 1e-4
    S, n, m = np.zeros((heads, dim, vdim)), np.zeros((heads, dim)), np.zeros(heads)
    li, lf = cap * np.tanh((d(i) + ib) / cap), npn.logsigmoid(cap * np.tanh((d(f) + fb) / cap))
    want = npn.rms(npn.mlstm_recurrence(d(q) * dim ** -0.5, d(k), d(v), li, lf, S, n, m), eps) * gain
    rows = L.state_rows(dim)
    for cuts in CUTS + ([[299, 1]] if T > 256 else []):
        state, mx, got, at, j = L.out(heads, vdim + 1, rows), L.out(heads), [], 0, 0
        while at < T:
            c = min(cuts[min(j, len(cuts) - 1)], T - at)
            o, sl = L.out(c, heads, vdim), slice(at, at + c)
            L.call("lumen_matrix_memory_f32", L.dev(q[sl]), L.dev(k[sl]), L.dev(v[sl]), L.dev(i[sl]), L.dev(f[sl]), L.dev(ib), L.dev(fb), L.dev(gain),
                   state, mx, o, c, heads, dim, vdim, cap, eps)
            got.append(o.data())
            at += c
            j += 1
        assert max_rel(np.concatenate(got), want) < 3e-5, cuts
        st = state.data()
        assert max_rel(st[:, :vdim, :dim].transpose(0, 2, 1), S) < 2e-5, cuts
        assert max_rel(st[:, vdim, :dim], n) < 2e-5, cuts
        assert max_rel(mx.data(), m) < 1e-5


def bias_table(rel, bias_max, n):
    """[heads][n] times log2 e, as the attention kernels read it."""
    return np.stack([rel[npn.bucket(x, len(rel), bias_max)] for x in range(n)], 1) * LOG2E


class Biased:
    """A sequence's attention through lumen_biased_attn_f32, store and position carried."""

    def __init__(self, L, heads, kv_heads, dim, vdim, cap, scale, temp=None, tab=None, sink=None):  # noqa: F811
        self.L, self.a, self.cap, self.scale, self.pos = L, (heads, kv_heads, dim, vdim), cap, scale, 0
        self.temp, self.sink = (L.dev(x) if x is not None else None for x in (temp, sink))
        self.tab, self.n = (L.dev(tab), tab.shape[1]) if tab is not None else (None, 0)
        self.kr, self.vr = L.out(kv_heads, cap, (dim + 3) // 4 * 4), L.out(kv_heads, cap, (vdim + 3) // 4 * 4)

    def step(self, q, k, v, gate=None):
        heads, kv_heads, dim, vdim = self.a
        out, dev = self.L.out(len(q), heads, vdim), self.L.dev
        self.L.call("lumen_biased_attn_f32", dev(q), dev(k), dev(v), dev(gate) if gate is not None else None, self.temp, self.tab, self.n, self.sink,
                    self.kr, self.vr, self.cap, out, len(q), self.pos, heads, kv_heads, dim, vdim, self.window,
                    self.scale)
        self.pos += len(q)
        return out.data()


def biased(L, T, big, *shape, **kw):  # noqa: F811
    """window T over a store of T - 1 + big positions: every key is seen."""
    b = Biased(L, *shape, cap=T - 1 + big, **kw)
    b.window = T
    return b


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,T", [(2, 2, 16, 16, 40), (4, 1, 10, 7, 90), (4, 2, 48, 20, 150), (1, 1, 100, 130, 70), (2, 1, 12, 16, 600)])
def test_attention_with_distance_bias_sink_and_temperature(L, heads, kv_heads, dim, vdim, T):  # noqa: F811
    r = rng(heads, dim, T)
    q, k, v, gate = f32(r, T, heads, dim) * 2, f32(r, T, kv_heads, dim), f32(r, T, kv_heads, vdim), f32(r, T, heads)
    temp, sink, rel = 1 + 0.4 * f32(r, heads), f32(r, heads) * 2, f32(r, 14, heads) * 2
    bias_max, scale = 33, 0.4
    tab = bias_table(rel, bias_max, bias_max + 1)
    want = npn.biased_sink_attention(d(q), d(k), d(v), scale, d(temp), d(rel), bias_max, d(sink)) * npn.sigmoid(d(gate))[:, :, None]
    for c in [[T], [2, 3, 64, 1, 1, 17, 65, 1, 128], [T - 30, 1]] + ([[1]] if T <= 150 else []):
        b = biased(L, T, max(c), heads, kv_heads, dim, vdim, scale=scale, temp=temp, tab=tab, sink=sink)
        got, at, i = [], 0, 0
        while at < T:
            n = min(c[min(i, len(c) - 1)], T - at)
            sl = slice(at, at + n)
            got.append(b.step(q[sl], k[sl], v[sl], gate[sl]))
            at += n
            i += 1
        assert max_rel(np.concatenate(got), want) < 1e-5, c


@pytest.mark.parametrize("rows,bias_max", [(6, 8), (12, 40), (7, 30), (32, 500)])
@pytest.mark.parametrize("decode", [False, True])
def test_every_distance_reads_its_own_row_of_the_bias(L, rows, bias_max, decode):  # noqa: F811
    """Equal scores, one row of the table raised at a time: the weight of the keys at its distances says which they are."""
    T = min(2 * bias_max, 300)
    own = np.array([npn.bucket(n, rows, bias_max) for n in range(T)])
    assert own[0] == 0 and (np.diff(own) >= 0).all() and (T < bias_max or own[-1] == rows - 1)
    z = np.zeros((T, 1, 4), np.float32)
    v = np.zeros((T, 1, T), np.float32)
    v[np.arange(T), 0, np.arange(T)] = 1
    for row in sorted({0, 1, rows // 2 - 1, rows // 2, rows - 2, rows - 1}):
        rel = np.zeros((rows, 1))
        rel[row] = 3
        want = np.exp(rel[own[T - 1 - np.arange(T)], 0])
        want /= want.sum()
        for v0 in range(0, T, 256):  # (value rows are at most 256 wide)
            vv = v[:, :, v0:v0 + 256]
            b = biased(L, T, T, 1, 1, 4, vv.shape[2], scale=1.0, tab=bias_table(rel, bias_max, bias_max + 1))
            if decode:
                b.step(z[:-1], z[:-1], vv[:-1])
                got = b.step(z[-1:], z[-1:], vv[-1:])[-1, 0]
            else:
                got = b.step(z, z, vv)[-1, 0]
            assert np.abs(got - want[v0:v0 + 256]).max() < 1e-6, row


def test_the_sink_takes_its_weight_once(L):  # noqa: F811
    """A dominant sink silences the head, a tiny one changes nothing, and one of the size of a key counts as one key -- over one
    slice of a step's keys and over several."""
    for T in (1, 5, 40, 700):
        z, one = np.zeros((T, 3, 4), np.float32), np.ones((T, 3, 4), np.float32)
        for cuts in ([T], [max(T - 3, 1), 1]):
            b = biased(L, T, T, 3, 3, 4, 4, scale=1.0, sink=np.array([30.0, -30.0, 0.0]))
            got, at, i = [], 0, 0
            while at < T:
                n = min(cuts[min(i, len(cuts) - 1)], T - at)
                got.append(b.step(z[at:at + n], z[at:at + n], one[at:at + n]))
                at += n
                i += 1
            got = np.concatenate(got)
            n = np.arange(1, T + 1)
            assert got[:, 0].max() < 1e-9 and np.abs(got[:, 1] - 1).max() < 1e-6
            assert np.abs(got[:, 2, 0] - n / (n + 1)).max() < 1e-6


@pytest.mark.parametrize("at", [0, 1, 31, 32, 255, 256, 511])
def test_a_far_key_among_hundreds(L, at):  # noqa: F811
    """One key stands out for one query direction; every later query finds it, in a prompt and in decoding, at tile and slice edges."""
    T, dim = 560, 8
    k, v, q = (np.zeros((T, 1, dim), np.float32) for _ in range(3))
    k[:, 0, 0] = -1
    k[at, 0, 0] = 1
    v[:, 0, 1] = 1
    v[at, 0, 1], v[at, 0, 2] = 0, 1
    q[:, 0, 0] = 12
    sink = np.array([-4.0])
    whole = biased(L, T, T, 1, 1, dim, dim, scale=1.0, sink=sink).step(q, k, v)
    b = biased(L, T, T, 1, 1, dim, dim, scale=1.0, sink=sink)
    b.step(q[:-12], k[:-12], v[:-12])
    tail = np.concatenate([b.step(q[t:t + 1], k[t:t + 1], v[t:t + 1]) for t in range(T - 12, T)])
    assert (whole[at:, 0, 2] > 0.99).all() and (whole[:at, 0, 2] == 0).all()
    assert (tail[:, 0, 2] > 0.99).all()


@pytest.mark.parametrize("experts,groups,keep,top", [(1, 1, 1, 1), (12, 4, 3, 3), (12, 4, 1, 3), (8, 8, 3, 2), (64, 8, 2, 6), (100, 1, 1, 7), (384, 6, 3, 9)])
def test_router(L, experts, groups, keep, top):  # noqa: F811
    r = rng(experts, groups, top)
    z = f32(r, 50, experts) * 2
    z[0] = 0.25  # ties everywhere: the lower index first
    z[1] = -200  # scores of zero
    sel, w = L.out(50, top), L.out(50, top)
    L.call("lumen_route_f32", L.dev(z), sel, w, 50, experts, groups, keep, top, 1.75)
    got = sel.data().view(np.int32)
    for t in range(50):
        e, want = npn.route(d(z[t]), {"top": top, "scale": 1.75, "groups": {"count": groups, "keep": keep}})
        if t != 1:
            assert got[t].tolist() == e, t
            assert np.abs(w.data()[t] - want).max() < 2e-6
        assert len(set(got[t].tolist())) == top and got[t].min() >= 0 and got[t].max() < experts


@pytest.mark.parametrize("s,dim,ff,experts,top", [(1, 8, 8, 3, 2), (5, 40, 24, 7, 3), (70, 64, 48, 4, 2), (300, 32, 16, 2, 2), (33, 136, 200, 40, 5),
                                                    (20, 72, 40, 3, 1), (30, 64, 24, 5, 2), (200, 40, 48, 20, 2)])
def test_experts_of_a_prompt(L, s, dim, ff, experts, top):  # noqa: F811
    """More tokens than a tile, experts nobody chose, experts everybody chose; the clamps bite."""
    r = rng(s, dim, experts)
    h, z = f32(r, s, dim), f32(r, s, experts)
    z[:, 0] += 2
    up, down = f32(r, experts, 2 * ff, dim) * 0.5, f32(r, experts, dim, ff) * 0.3
    out, w = L.out(s, top, dim), L.out(s, top)
    L.call("lumen_experts_f32", L.dev(h), L.dev(z), L.dev(up), L.dev(down), 0, out, w, s, dim, ff, experts, 1, 1, top, 2.0, 1.1)
    got = out.data()
    for t in range(s):
        chosen, weights = npn.route(d(z[t]), {"top": top, "scale": 2.0})
        want = np.stack([npn.clamped_expert(d(h[t]), {"gate": d(up[e, ::2]), "up": d(up[e, 1::2]), "down": d(down[e])}, 1.1) for e in chosen])
        assert max_rel(got[t], want) < 5e-6, t
        assert np.abs(w.data()[t] - weights).max() < 2e-6


def test_operators_refuse_what_they_cannot_do(L):  # noqa: F811
    o = L.out(4, 4)
    for args in ((12, 5, 1, 1), (12, 4, 5, 1), (12, 4, 1, 4), (12, 4, 1, 0)):
        with pytest.raises(L.error):
            L.call("lumen_route_f32", o, o, o, 1, *args, 1.0)
    with pytest.raises(L.error):
        L.call("lumen_gated_residual_f32", o, o, None, None, None, o, o, o, 1, 6, 6, 1.0, 0.0)
    with pytest.raises(L.error):
        L.call("lumen_general_delta_f32", o, o, o, o, o, o, o, o, o, 1, 1, 257, 4, 1e-6)
    with pytest.raises(L.error):
        L.call("lumen_matrix_memory_f32", o, o, o, o, o, o, o, o, o, o, o, 1, 1, 4, 4, 0.0, 1e-6)


# ------------------------------------------------------------------ models
MODELS = {
    # every mechanism, sizes that are multiples of nothing, a loop over the middle
    "odd": nu.config(37, 61, [nu.general(3, 7, nu.dense(45)), nu.parallel((6, 3, 10, 7), (3, 5, 9), nu.moe(11, 6, 2, (3, 2))),
                              nu.general(2, 20, nu.moe(19, 5, 3)), nu.parallel((2, 1, 12, 5), (1, 70, 3), nu.dense(29), bias_max=17)],
                     loop=(1, 3, 3), eps=1e-4),
    # no loop, no cap, no feed-forward in places, wide heads, one group kept of several
    "plain": nu.config(64, 128, [nu.parallel((2, 2, 80, 72), (1, 130, 140)), nu.general(1, 130), nu.parallel((1, 1, 16, 16), (2, 16, 64), nu.moe(40, 16, 4, (4, 1))),
                                 nu.general(4, 16, nu.moe(8, 9, 9, scale=0.5, limit=7.0))], softcap=0),
    # the loop over everything, and passes of a single layer
    "whole_loop": nu.config(48, 96, [nu.parallel((4, 1, 16, 16), (2, 24, 16), nu.dense(80), bias_max=9), nu.general(2, 32, nu.moe(24, 8, 2, (2, 1)))],
                            loop=(0, 2, 2), softcap=3.0),
    "one_layer_loop": nu.config(40, 50, [nu.general(2, 20, nu.dense(30)), nu.parallel((3, 3, 8, 8), (2, 20, 20), nu.moe(16, 4, 1)), nu.general(1, 8)],
                                loop=(1, 2, 4)),
    "once": nu.config(32, 33, [nu.parallel((2, 2, 16, 8), (1, 8, 8), nu.dense(48)), nu.general(1, 16, nu.moe(8, 2, 1))], loop=(0, 1, 1)),
}


@pytest.mark.parametrize("name", sorted(MODELS))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_model_against_the_plain_one(tmp_path, name, dtype):
    """Prompt, decoding and portions down to two tokens: the same logits and the same residual stream."""
    cfg = MODELS[name]
    params = nu.make_params(cfg, seed=3)
    model = hu.load(tmp_path, cfg, params, dtype)
    toks = tokens_of(cfg, 60)
    taps = []
    want = npn.forward(cfg, params, toks, taps)
    got, got_taps = hu.run(model, toks, [60], residual=True)
    for i, (a, b) in enumerate(zip(got_taps, taps)):
        assert max_rel(a, b) < 3e-5, i
    assert max_rel(got, want) < 5e-5
    _, dec_taps = hu.run(model, toks[:12], [3, 1], residual=True)
    assert max_rel(dec_taps, np.stack(taps)[:, :12]) < 3e-5
    for cuts in ([1], [2], [3, 1, 2, 5, 16, 1, 17, 8], [47, 1]):
        assert max_rel(hu.run(model, toks, cuts), want) < 5e-5, cuts


def test_a_sequence_does_not_see_the_one_before(tmp_path):
    cfg = MODELS["odd"]
    params = nu.make_params(cfg, seed=4)
    model = hu.load(tmp_path, cfg, params)
    a, b = tokens_of(cfg, 45, 1), tokens_of(cfg, 50, 2)
    first = hu.run(model, b, [20, 1])
    hu.run(model, a, [45])
    hu.run(model, a, [1])
    again = hu.run(model, b, [20, 1])
    assert np.array_equal(first, again)
    assert max_rel(first, npn.forward(cfg, params, b)) < 5e-5
    model.reset()
    assert model.length == 0
    assert max_rel(model.step(b[:1], [0]), first[:1]) < 5e-5  # the first token, decoded


def test_long_sequences_with_sharp_attention(tmp_path):
    """Hundreds of keys whose scores stand out, several slices per step, prompts the model cuts itself, positions to the last one."""
    from lumen_amd.hybrid import HybridModel, nufapel_config
    cfg = nu.config(32, 40, [nu.parallel((2, 1, 8, 16), (1, 8, 8), nu.dense(40), bias_max=300), nu.general(1, 16),
                             nu.parallel((4, 2, 8, 6), (2, 8, 12), nu.moe(8, 4, 2))], positions=640)
    params = nu.sharpen(nu.make_params(cfg, seed=6, bias_rows=20))
    toks = tokens_of(cfg, 640)
    want = npn.forward(cfg, params, toks)
    hc = nufapel_config(cfg, lambda n: params[n].shape, 100000, "f32")
    assert hc.max_seq_len == 640
    hc.max_chunk = 100
    model = HybridModel(hc)
    model.load_params(params)
    for cuts in ([640], [250, 1, 1, 1, 1, 1, 40, 2, 200, 1], [256, 256, 100, 1]):
        assert max_rel(hu.run(model, toks, cuts), want) < 1e-4, cuts


def test_long_decoding_graph_and_eager(tmp_path):
    cfg = MODELS["odd"]
    params = nu.make_params(cfg, seed=7)
    model = hu.load(tmp_path, cfg, params, "bfloat16")
    prompt = tokens_of(cfg, 10)
    picks = {}
    for mode in ("graph", "eager"):
        model.set_decode_mode(mode)
        model.reset()
        first = int(np.argmax(model.step(prompt, [9])[0]))
        picks[mode] = model.decode_greedy(first, 300, want_logits=True)
    assert np.array_equal(picks["graph"][0], picks["eager"][0])
    assert np.array_equal(picks["graph"][1], picks["eager"][1])
    ids, logits = picks["graph"]
    seq = np.concatenate([prompt, [first], ids[:-1]])
    assert max_rel(logits, npn.forward(cfg, params, seq)[len(prompt):]) < 1e-4
    prof = model.decode_profile(int(ids[-1]), 2)
    assert prof["general"][1] == 8 and prof["memory"][1] == 8 and prof["experts_up"][1] == 12  # (two steps; the loop's layers three times each)


def plain_greedy(cfg, params, prompt, n):
    seq, out, gaps = list(prompt), [], []
    for _ in range(n):
        row = npn.forward(cfg, params, seq)[-1]
        top = np.sort(row)[-2:]
        gaps.append((top[1] - top[0]) / np.abs(row).max())
        out.append(int(np.argmax(row)))
        seq.append(out[-1])
    return out, gaps


def test_greedy_generation_through_the_turn_loop_and_the_command_line(tmp_path, capsys):
    cfg = MODELS["whole_loop"]
    params = nu.make_params(cfg, seed=8)
    prompt = [int(t) for t in tokens_of(cfg, 21)]
    want, gaps = plain_greedy(cfg, params, prompt, 12)
    assert min(gaps) > 1e-4  # no pick that rounding could turn
    model = hu.load(tmp_path, cfg, params)
    assert model.generate_turn(prompt, top_p=0.0, repetition_penalty=1.0, max_gen=12).tolist() == want
    more, _ = plain_greedy(cfg, params, prompt + want + [7, 3], 4)
    assert model.generate_turn([7, 3], history=prompt + want, top_p=0.0, repetition_penalty=1.0, max_gen=4).tolist() == more
    del model
    from lumen_amd.__main__ import main
    assert main(["generate", "--model", str(tmp_path), "--prompt", ",".join(map(str, prompt)), "--max-new", "12", "--greedy", "--max-seq", "100"]) == 0
    assert [int(t) for t in capsys.readouterr().out.split()] == want


def test_model_errors(tmp_path):
    from lumen_amd import _lib
    from lumen_amd.hybrid import HybridModel, nufapel_config
    cfg = MODELS["once"]
    params = nu.make_params(cfg, seed=9)
    model = hu.load(tmp_path, cfg, params, max_seq_len=20)
    with pytest.raises(_lib.LumenError) as e:
        model.step(np.zeros(21, int), [0])
    assert e.value.status == _lib.ERR_KV_OVERFLOW
    with pytest.raises(_lib.LumenError) as e:
        model.set_param("l0.norm1.alpha", np.zeros(1, np.float32))
    assert e.value.status == _lib.ERR_SHAPE
    for change in (dict(experts=0), dict(top=3), dict(groups=2, keep=3)):
        hc = nufapel_config(cfg, lambda n: params[n].shape, 20, "f32")
        for k, v in change.items():
            setattr(hc.layers[1], k, v)
        with pytest.raises(_lib.LumenError):
            HybridModel(hc)
    hc = nufapel_config(cfg, lambda n: params[n].shape, 20, "f32")
    hc.max_seq_len = cfg["max_positions"] + 1
    with pytest.raises(_lib.LumenError):
        HybridModel(hc)
    del params["l1.mlp.e1.up"]
    with pytest.raises(_lib.LumenError, match="lacks 1"):
        hu.load(tmp_path / "short", cfg, params)


def test_trace_runner(tmp_path):
    """bin/trace_run over two requests, one after the other, cut differently."""
    cfg = MODELS["odd"]
    params = nu.make_params(cfg, seed=10)
    folder = hu.write_model(tmp_path / "model", cfg, params)
    out = tmp_path / "out"
    out.mkdir()
    a, b = tokens_of(cfg, 30, 1).tolist(), tokens_of(cfg, 17, 2).tolist()
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:25], "want": [24, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[25:26], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "a", "tokens": a[26:], "want": [0, 3]}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "b", "tokens": b, "want": [16]}], "end": ["b"]}]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "30"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    la, lb = npn.forward(cfg, params, a), npn.forward(cfg, params, b)
    read = lambda i: np.fromfile(out / ("%d.f32" % i), "<f4").reshape(-1, cfg["vocab"])  # noqa: E731
    assert max_rel(read(0), la[[24, 3]]) < 5e-5
    assert max_rel(read(2), la[[26, 29]]) < 5e-5
    assert max_rel(read(3), lb[[16]]) < 5e-5


def test_tiny_model(tmp_path):
    """Every mechanism once at the smallest sizes: a prompt, a portion of two, decoding."""
    cfg = nu.config(8, 11, [nu.parallel((2, 1, 4, 4), (1, 4, 3), nu.moe(8, 4, 2, (2, 1)), bias_max=20), nu.general(1, 4, nu.dense(8))], loop=(0, 1, 2),
                    positions=16)
    params = nu.make_params(cfg, seed=11, rank=2, bias_rows=4)
    model = hu.load(tmp_path, cfg, params, max_seq_len=16)
    toks = tokens_of(cfg, 6)
    assert max_rel(hu.run(model, toks, [3, 2, 1]), npn.forward(cfg, params, toks)) < 5e-5
