"""The layered hybrid decoder on the GPU against its plain restatement (oracle/hybrid_plain.py): every mechanism alone
through the C ABI, then whole models -- prompts, decoding, portions, reuse, generation."""
import ctypes as C
import json
import os
import subprocess
import sys

import numpy as np
import pytest

from gpu_util import max_rel
import hybrid_util as hu
from oracle import hybrid_plain as hp

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


@pytest.fixture(scope="module")
def L():
    from lumen_amd import _lib
    from lumen_amd.autograd import Tensor, default_ctx

    class Lib:
        ctx = default_ctx()

        @staticmethod
        def dev(a):
            return Tensor.from_array_no_grad(np.ascontiguousarray(a, np.float32))

        @staticmethod
        def out(*shape):
            return Tensor.from_array_no_grad(np.zeros(shape, np.float32))

        @staticmethod
        def call(name, *args):
            _lib.check(getattr(_lib.lib, name)(Lib.ctx.handle, *[a.ptr if isinstance(a, Tensor) else a for a in args]))

        @staticmethod
        def state_rows(dim):
            n = C.c_int()
            _lib.check(_lib.lib.lumen_recurrence_state_rows(dim, C.byref(n)))
            return n.value

        error = _lib.LumenError
    return Lib


def rng(*key):
    return np.random.default_rng(list(key))


# ------------------------------------------------------------------ mechanisms
@pytest.mark.parametrize("rows,dim", [(1, 1), (3, 7), (5, 64), (2, 1000), (4, 1026), (2, 5000), (1, 16384), (1, 20001)])
def test_polynorm(L, rows, dim):
    r = rng(rows, dim)
    z = r.standard_normal((rows, dim)) * 2
    coef = np.array([0.7, -0.4, 0.3, 0.2])
    out = L.out(rows, dim)
    L.call("lumen_polynorm_f32", L.dev(z), L.dev(coef), out, rows, dim, 1e-3)
    assert max_rel(out.data(), hp.polynorm(z.astype(np.float32).astype(np.float64), coef, 1e-3)) < 3e-6


@pytest.mark.parametrize("dim", [8, 33, 1028])
def test_token_shift_carries_the_last_token(L, dim):
    r = rng(dim)
    h, mu = r.standard_normal((7, dim)), r.standard_normal((3, dim))
    prev = np.zeros(dim)
    for a, b in ((0, 1), (1, 3), (3, 7)):
        mixes, nxt = L.out(3, b - a, dim), L.out(dim)
        L.call("lumen_token_shift_f32", L.dev(h[a:b]), L.dev(mu), L.dev(prev), nxt, mixes, 3, b - a, dim)
        before = np.concatenate([prev[None], h[a:b - 1]])
        want = np.stack([h[a:b] + (before - h[a:b]) * m for m in mu])
        assert max_rel(mixes.data(), want) < 1e-6
        assert np.array_equal(nxt.data(), h[b - 1].astype(np.float32))
        prev = h[b - 1]


@pytest.mark.parametrize("taps,heads,kv_heads,dim,vdim", [(1, 2, 2, 8, 8), (2, 3, 1, 5, 9), (3, 4, 2, 64, 70), (5, 2, 2, 130, 16), (9, 1, 1, 256, 200)])
def test_convolution_and_unit_vectors(L, taps, heads, kv_heads, dim, vdim):
    r = rng(taps, dim)
    n = 2 * kv_heads * dim + heads * vdim
    x, w = r.standard_normal((13, n)), r.standard_normal((n, taps))
    x, w = x.astype(np.float32), w.astype(np.float32)
    y = hp.causal_conv_silu(x.astype(np.float64), w.astype(np.float64))
    nq = kv_heads * dim
    want_q = hp.unit(y[:, :nq].reshape(13, kv_heads, dim)).reshape(13, nq) * 0.3
    want_k = hp.unit(y[:, nq:2 * nq].reshape(13, kv_heads, dim)).reshape(13, nq)
    prev = np.zeros((max(taps - 1, 1), n))
    for a, b in ((0, 2), (2, 3), (3, 13)):
        s = b - a
        q, k, v, nxt = L.out(s, nq), L.out(s, nq), L.out(s, heads * vdim), L.out(max(taps - 1, 1), n)
        L.call("lumen_conv_unit_f32", L.dev(x[a:b]), L.dev(w), L.dev(prev), nxt, q, k, v, s, taps, heads, kv_heads, dim, vdim, 1e-6, 0.3)
        assert max_rel(q.data(), want_q[a:b]) < 1e-5
        assert max_rel(k.data(), want_k[a:b]) < 1e-5
        assert max_rel(v.data(), y[a:b, 2 * nq:]) < 1e-5
        prev = nxt.data()
        if taps > 1:
            held = np.concatenate([np.zeros((taps, n)), x[:b]])[-(taps - 1):]
            assert np.array_equal(prev, held.astype(np.float32))


@pytest.mark.parametrize("shared", [0, 1])
@pytest.mark.parametrize("act", [0, 1, 2])
def test_head_norm_and_gate(L, shared, act):
    r = rng(shared, act)
    o, gate = r.standard_normal((3, 4, 37)), r.standard_normal((3, 4, 37))
    gain = r.standard_normal(37 if shared else 4 * 37)
    d = L.dev(o)
    L.call("lumen_head_norm_gate_f32", d, L.dev(gain), shared, L.dev(gate) if act else None, act, 3, 4, 37, 1e-4)
    g = 1.0 if act == 0 else hp.sigmoid(gate) if act == 1 else hp.silu(gate)
    assert max_rel(d.data(), hp.rms(o, 1e-4) * (gain if shared else gain.reshape(4, 37)) * g) < 3e-6


CUTS = [[100], [1], [2, 3, 1, 9, 16, 17, 8, 33, 7], [15, 16, 1, 32, 36]]


@pytest.mark.parametrize("heads,dim", [(1, 3), (2, 16), (3, 48), (2, 64), (1, 80), (2, 128), (1, 200)])
def test_wkv_recurrence(L, heads, dim):
    """Whole, token by token and in portions (16 tokens are taken at a time inside): same outputs, same state; channels
    that forget within a token beside channels that forget nothing."""
    T = 100
    r = rng(heads, dim)
    f = lambda *s: r.standard_normal(s).astype(np.float32)  # noqa: E731
    R, K, V = f(T, heads, dim), f(T, heads, dim), f(T, heads, dim)
    z = f(T, heads, dim) * 2
    bias = np.linspace(-9, 3, heads * dim).astype(np.float32).reshape(heads, dim)
    u = f(heads, dim)
    S = np.zeros((heads, dim, dim))
    w = np.exp(-np.exp(z.astype(np.float64) + bias))
    want = hp.wkv_recurrence(*(x.astype(np.float64) for x in (R, K, V)), w, u.astype(np.float64), S)
    rows = L.state_rows(dim)
    for cuts in CUTS:
        state, got, at, i = L.out(heads, dim, rows), [], 0, 0
        while at < T:
            n = min(cuts[min(i, len(cuts) - 1)], T - at)
            o, sl = L.out(n, heads, dim), slice(at, at + n)
            L.call("lumen_wkv_f32", L.dev(R[sl]), L.dev(K[sl]), L.dev(V[sl]), L.dev(z[sl]), L.dev(bias), L.dev(u), state, o, n, heads, dim)
            got.append(o.data())
            at += n
            i += 1
        assert max_rel(np.concatenate(got), want) < 1e-5, cuts
        st = state.data()
        assert max_rel(st[:, :, :dim].transpose(0, 2, 1), S) < 1e-5, cuts
        assert not st[:, :, dim:].any()


@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [(1, 1, 4, 3), (4, 2, 16, 20), (2, 1, 48, 64), (2, 2, 64, 33), (3, 3, 100, 128), (2, 1, 144, 16), (1, 1, 256, 40)])
def test_channel_delta_recurrence(L, heads, kv_heads, dim, vdim):
    T, rep = 100, heads // kv_heads
    r = rng(heads, dim, vdim)
    f = lambda *s: r.standard_normal(s).astype(np.float32)  # noqa: E731
    q = hp.unit(f(T, kv_heads, dim).astype(np.float64)).astype(np.float32)
    k = hp.unit((f(T, kv_heads, dim) + 1.0).astype(np.float64)).astype(np.float32)  # (keys with much in common)
    V, z, b = f(T, heads, vdim), f(T, heads, dim) * 2, f(T, heads) + 1
    bias = np.linspace(-9, 3, heads * dim).astype(np.float32).reshape(heads, dim)
    a_log = np.linspace(-1, 2, heads).astype(np.float32)
    S = np.zeros((heads, dim, vdim))
    g = np.exp(-np.exp(a_log.astype(np.float64))[None, :, None] * hp.softplus(z.astype(np.float64) + bias))
    want = hp.delta_recurrence(np.repeat(q, rep, 1).astype(np.float64), np.repeat(k, rep, 1).astype(np.float64), V.astype(np.float64), g,
                               hp.sigmoid(b.astype(np.float64)), S)
    rows = L.state_rows(dim)
    for cuts in CUTS:
        state, got, at, i = L.out(heads, vdim, rows), [], 0, 0
        while at < T:
            n = min(cuts[min(i, len(cuts) - 1)], T - at)
            o, sl = L.out(n, heads, vdim), slice(at, at + n)
            L.call("lumen_channel_delta_f32", L.dev(q[sl]), L.dev(k[sl]), L.dev(V[sl]), L.dev(z[sl]), L.dev(b[sl]), L.dev(bias), L.dev(a_log),
                   state, o, n, heads, kv_heads, dim, vdim)
            got.append(o.data())
            at += n
            i += 1
        assert max_rel(np.concatenate(got), want) < 2e-5, cuts
        st = state.data()
        assert max_rel(st[:, :, :dim].transpose(0, 2, 1), S) < 2e-5, cuts
        assert not st[:, :, dim:].any()


class Window:
    """A sequence's attention through lumen_window_attn_f32, ring and position carried."""

    def __init__(self, L, heads, kv_heads, dim, vdim, window, cap, scale, softcap, eps=1e-5, bias=None, norms=None, gate=False):
        self.L, self.a = L, (heads, kv_heads, dim, vdim, window)
        self.cap, self.scale, self.softcap, self.eps, self.gate = cap, scale, softcap, eps, gate
        self.bias = [L.dev(x) for x in bias] if bias else [None, None]
        self.norms = [L.dev(x) for x in norms] if norms else [None, None]
        self.kr = L.out(kv_heads, cap, (dim + 3) // 4 * 4)
        self.vr = L.out(kv_heads, cap, (vdim + 3) // 4 * 4)
        self.pos = 0

    def step(self, q, k, v, gate=None):
        heads, kv_heads, dim, vdim, window = self.a
        s = len(q)
        out = self.L.out(s, heads, vdim)
        self.L.call("lumen_window_attn_f32", self.L.dev(q), self.L.dev(k), self.L.dev(v), self.L.dev(gate) if gate is not None else None,
                    *self.norms, *self.bias, self.kr, self.vr, self.cap, out, s, self.pos, heads, kv_heads, dim, vdim, window, self.scale,
                    self.softcap, self.eps)
        self.pos += s
        return out.data()


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,window,T", [
    (2, 2, 16, 16, 1, 40), (2, 1, 10, 7, 2, 40), (4, 2, 48, 20, 33, 150), (1, 1, 64, 64, 31, 90), (2, 1, 100, 130, 64, 140),
    (1, 1, 200, 256, 20, 70), (2, 1, 12, 16, 257, 700), (1, 1, 8, 12, 600, 640)])
def test_window_attention_in_prompts_portions_and_decoding(L, heads, kv_heads, dim, vdim, window, T):
    r = rng(heads, dim, window)
    f = lambda *s: r.standard_normal(s).astype(np.float32)  # noqa: E731
    q, k, v, gate = f(T, heads, dim) * 3, f(T, kv_heads, dim), f(T, kv_heads, vdim), f(T, heads, vdim)
    r1, r2 = np.abs(f(heads)), np.abs(f(heads))
    gq, gk = 1 + 0.3 * f(heads * dim), 1 + 0.3 * f(kv_heads * dim)
    d = lambda x: x.astype(np.float64)  # noqa: E731
    qn = (hp.rms(d(q).reshape(T, -1), 1e-5) * gq).reshape(q.shape)
    kn = (hp.rms(d(k).reshape(T, -1), 1e-5) * gk).reshape(k.shape)
    want = hp.window_attention(qn * 3, kn, d(v), 0.5, 6.0, d(r1), d(r2), window) * hp.sigmoid(d(gate))
    cuts = [[T], [2, 3, 64, 1, 1, 17, 65, 1, 128], [T - 30, 1]] + ([[1]] if T <= 150 else [])
    for c in cuts:
        big = max(c)
        w = Window(L, heads, kv_heads, dim, vdim, window, window - 1 + big, 1.5, 6.0, bias=(r1, r2), norms=(gq, gk), gate=True)
        got, at, i = [], 0, 0
        while at < T:
            n = min(c[min(i, len(c) - 1)], T - at)
            sl = slice(at, at + n)
            got.append(w.step(q[sl], k[sl], v[sl], gate[sl]))
            at += n
            i += 1
        assert max_rel(np.concatenate(got), want) < 1e-5, c


@pytest.mark.parametrize("window", [1, 2, 15, 16, 17, 31, 32, 33, 70, 256, 257, 300])
@pytest.mark.parametrize("decode", [False, True])
def test_a_key_shows_up_to_the_window_and_not_one_token_further(L, window, decode):
    """One key stands out for one query direction: inside the window it takes the whole weight, just outside none."""
    T = window + 70
    dim = 8
    at = 5  # the standing-out key
    k = np.zeros((T, 1, dim), np.float32)
    k[:, 0, 0] = -1
    k[at, 0, 0] = 1
    v = np.zeros((T, 1, dim), np.float32)
    v[:, 0, 1] = 1
    v[at, 0, 1], v[at, 0, 2] = 0, 1
    q = np.zeros((T, 1, dim), np.float32)
    q[:, 0, 0] = 12
    w = Window(L, 1, 1, dim, dim, window, window - 1 + T, 1.0, 30.0)
    if decode:
        got = np.concatenate([w.step(q[:at + 2], k[:at + 2], v[:at + 2])] +
                             [w.step(q[t:t + 1], k[t:t + 1], v[t:t + 1]) for t in range(at + 2, T)])
    else:
        got = w.step(q, k, v)
    seen = got[:, 0, 2] > 0.99
    assert np.array_equal(np.nonzero(seen)[0], np.arange(at, min(at + window, T)))
    assert (got[~seen, 0, 2] == 0).all()


def test_soft_cap_and_distance_bias_bound_the_scores(L):
    """Scores far beyond the cap, no cap at all, and a bias that outweighs the score of a far key."""
    r = rng(9)
    T, dim = 60, 16
    q, k, v = (r.standard_normal((T, 2, dim)).astype(np.float32) for _ in range(3))
    d = lambda x: x.astype(np.float64)  # noqa: E731
    for scale, cap, r1, r2 in ((40.0, 5.0, 0.0, 1.0), (0.7, 0.0, 2.0, 0.5), (1e-3, 50.0, 0.0, 0.0), (0.3, 1.0, 3.0, 100.0)):
        b = (np.array([r1, r1 * 0.5], np.float32), np.array([r2, r2 * 3], np.float32))
        want = hp.window_attention(d(q), d(k), d(v), scale, cap, d(b[0]), d(b[1]), 40)
        for cuts in (60, 1):
            w = Window(L, 2, 2, dim, dim, 40, 39 + cuts, scale, cap, bias=b)
            got = np.concatenate([w.step(q[t:t + cuts], k[t:t + cuts], v[t:t + cuts]) for t in range(0, T, cuts)])
            assert max_rel(got, want) < 2e-5, (scale, cap, cuts)


def test_operators_refuse_what_they_cannot_do(L):
    o = L.out(4, 4)
    with pytest.raises(L.error):
        L.call("lumen_window_attn_f32", o, o, o, None, None, None, None, None, o, o, 4, o, 2, 0, 1, 1, 4, 4, 4, 1.0, 0.0, 1e-5)  # ring too small
    with pytest.raises(L.error):
        L.call("lumen_token_shift_f32", o, o, o, o, o, 1, 1, 4)  # prev is next
    with pytest.raises(L.error):
        L.state_rows(257)


# ------------------------------------------------------------------ models
MODELS = {
    # every mechanism, sizes that are multiples of nothing, shared key / value heads, a loop over the middle
    "odd": hu.config(37, 61, [hu.delta(4, 2, 6, 10, conv=5, ff=45), hu.attention(6, 3, 10, 7, 9, ff=50), hu.wkv(3, 11, ff=29),
                              hu.attention(2, 1, 12, 5, 30)], loop=(1, 3, 3), eps=1e-4, residual_mult=0.8),
    # no loop, no feed-forward in places, other orders, wide heads
    "plain": hu.config(64, 128, [hu.wkv(2, 72), hu.wkv(1, 40, ff=96), hu.delta(1, 1, 130, 70, conv=2), hu.attention(2, 2, 80, 72, 17, ff=64)]),
    # the loop over everything, and passes of a single layer
    "whole_loop": hu.config(48, 96, [hu.attention(4, 1, 16, 16, 40, ff=80), hu.delta(2, 1, 32, 64, conv=3, ff=100)], loop=(0, 2, 2), residual_mult=1.0),
    "one_layer_loop": hu.config(40, 50, [hu.wkv(2, 20, ff=30), hu.delta(2, 2, 20, 20, conv=1, ff=64), hu.attention(3, 3, 8, 8, 5)], loop=(1, 2, 4), scale=1.0),
    "once": hu.config(32, 33, [hu.attention(2, 2, 16, 8, 1, ff=48), hu.wkv(1, 16, ff=32)], loop=(0, 1, 1)),
}


def tokens_of(cfg, n, seed=0):
    return rng(seed, n).integers(0, cfg["vocab"], n)


@pytest.mark.parametrize("name", sorted(MODELS))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_model_against_the_plain_one(tmp_path, name, dtype):
    """Prompt, decoding and portions down to two tokens: the same logits and, in one run, the same residual stream."""
    cfg = MODELS[name]
    params = hu.make_params(cfg, seed=3)
    model = hu.load(tmp_path, cfg, params, dtype)
    toks = tokens_of(cfg, 60)
    taps = []
    want = hp.forward(cfg, params, toks, taps)
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
    params = hu.make_params(cfg, seed=4)
    model = hu.load(tmp_path, cfg, params)
    a, b = tokens_of(cfg, 45, 1), tokens_of(cfg, 50, 2)
    first = hu.run(model, b, [20, 1])
    hu.run(model, a, [45])
    hu.run(model, a, [1])
    again = hu.run(model, b, [20, 1])
    assert np.array_equal(first, again)
    assert max_rel(first, hp.forward(cfg, params, b)) < 5e-5
    model.reset()
    assert model.length == 0
    one = model.step(b[:1], [0])  # the first token, decoded
    assert max_rel(one, first[:1]) < 5e-5


def test_prompts_longer_than_a_chunk_and_rings_that_wrap(tmp_path):
    """max_chunk below the prompt's length: the model cuts it itself; the rings hold a window and a chunk and wrap."""
    from lumen_amd.hybrid import HybridModel, pinavik_config
    cfg = MODELS["whole_loop"]
    params = hu.make_params(cfg, seed=5)
    hc = pinavik_config(cfg, lambda n: params[n].shape, 400, "f32")
    hc.max_chunk = 24
    model = HybridModel(hc)
    model.load_params(params)
    toks = tokens_of(cfg, 230)
    want = hp.forward(cfg, params, toks)
    for cuts in ([230], [100, 1, 30, 2], [25], [1]):
        assert max_rel(hu.run(model, toks, cuts), want) < 5e-5, cuts


def test_windows_over_several_slices_of_a_decode_step(tmp_path):
    """Windows beyond 256 keys: a step's keys are cut into slices, folded by the output projection where its size
    allows that and by a launch of their own where not (head widths that are no multiple of 4)."""
    for vdim in (16, 6):
        cfg = hu.config(32, 40, [hu.attention(2, 1, 8, vdim, 300, ff=40), hu.attention(4, 2, 8, vdim, 700)])
        params = hu.make_params(cfg, seed=6)
        model = hu.load(tmp_path / str(vdim), cfg, params, max_seq_len=800)
        toks = tokens_of(cfg, 780)
        want = hp.forward(cfg, params, toks)
        got = hu.run(model, toks, [250, 1, 1, 1, 1, 1, 1, 1, 1, 1, 40, 1, 1, 1, 1, 200] + [1])
        assert max_rel(got, want) < 5e-5, vdim


def test_long_decoding_graph_and_eager(tmp_path):
    cfg = MODELS["odd"]
    params = hu.make_params(cfg, seed=7)
    model = hu.load(tmp_path, cfg, params, "bfloat16")
    prompt = tokens_of(cfg, 10)
    picks = {}
    for mode in ("graph", "eager"):
        model.set_decode_mode(mode)
        model.reset()
        first = int(np.argmax(model.step(prompt, [9])[0]))
        ids, logits = model.decode_greedy(first, 300, want_logits=True)
        picks[mode] = (ids, logits)
    assert np.array_equal(picks["graph"][0], picks["eager"][0])
    assert np.array_equal(picks["graph"][1], picks["eager"][1])
    ids, logits = picks["graph"]
    seq = np.concatenate([prompt, [first], ids[:-1]])
    assert max_rel(logits, hp.forward(cfg, params, seq)[len(prompt):]) < 1e-4
    prof = model.decode_profile(int(ids[-1]), 2)
    assert prof["wkv"][1] == 6 and prof["delta"][1] == 2 and prof["attn"][1] == 8  # (two steps; the loop's layers three times each)


def plain_greedy(cfg, params, prompt, n):
    seq, out, gaps = list(prompt), [], []
    for _ in range(n):
        row = hp.forward(cfg, params, seq)[-1]
        top = np.sort(row)[-2:]
        gaps.append((top[1] - top[0]) / np.abs(row).max())
        out.append(int(np.argmax(row)))
        seq.append(out[-1])
    return out, gaps


def test_greedy_generation_through_the_turn_loop_and_the_command_line(tmp_path, capsys):
    cfg = MODELS["whole_loop"]
    params = hu.make_params(cfg, seed=8)
    prompt = [int(t) for t in tokens_of(cfg, 21)]
    want, gaps = plain_greedy(cfg, params, prompt, 12)
    assert min(gaps) > 1e-3  # no pick that rounding could turn
    model = hu.load(tmp_path, cfg, params)
    got = model.generate_turn(prompt, top_p=0.0, repetition_penalty=1.0, max_gen=12)
    assert got.tolist() == want
    # a second turn goes on where the first ended
    more, _ = plain_greedy(cfg, params, prompt + want + [7, 3], 4)
    assert model.generate_turn([7, 3], history=prompt + want, top_p=0.0, repetition_penalty=1.0, max_gen=4).tolist() == more
    model.reset()
    assert model.generate_turn(prompt, top_p=0.0, repetition_penalty=1.0, max_gen=12, stop_ids=[want[4]]).tolist() == want[:want.index(want[4])]
    del model
    from lumen_amd.__main__ import main
    assert main(["generate", "--model", str(tmp_path), "--prompt", ",".join(map(str, prompt)), "--max-new", "12", "--greedy", "--max-seq", "100"]) == 0
    assert [int(t) for t in capsys.readouterr().out.split()] == want


def test_model_errors(tmp_path):
    from lumen_amd import _lib
    cfg = MODELS["once"]
    params = hu.make_params(cfg, seed=9)
    model = hu.load(tmp_path, cfg, params, max_seq_len=20)
    with pytest.raises(_lib.LumenError) as e:
        model.step(np.zeros(21, int), [0])
    assert e.value.status == _lib.ERR_KV_OVERFLOW
    for bad in (-1, cfg["vocab"]):
        with pytest.raises(_lib.LumenError) as e:
            model.step([0, bad], [0])
        assert e.value.status == _lib.ERR_EMBED_OOB
    with pytest.raises(_lib.LumenError):
        model.step([0, 1], [1, 0])  # places must ascend
    with pytest.raises(_lib.LumenError) as e:
        model.set_param("l0.norm1", np.zeros(31, np.float32))
    assert e.value.status == _lib.ERR_SHAPE
    with pytest.raises(_lib.LumenError):
        model.set_param("l9.norm1", np.zeros(32, np.float32))
    assert model.length == 0
    del params["l1.mix.w0"]
    with pytest.raises(_lib.LumenError, match="lacks 1"):
        hu.load(tmp_path / "short", cfg, params)


def test_trace_runner(tmp_path):
    """bin/trace_run over two requests, one after the other, cut differently; wanted places in any order."""
    cfg = MODELS["odd"]
    params = hu.make_params(cfg, seed=10)
    folder = hu.write_model(tmp_path / "model", cfg, params)
    out = tmp_path / "out"
    out.mkdir()
    a, b = tokens_of(cfg, 30, 1).tolist(), tokens_of(cfg, 17, 2).tolist()
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:25], "want": [24, 3]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[25:26], "want": []}], "end": []},
        {"step": 2, "entries": [{"id": "a", "tokens": a[26:], "want": [0, 3]}], "end": ["a"]},
        {"step": 3, "entries": [{"id": "b", "tokens": b, "want": [16]}], "end": ["b"]},
    ]
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "30"], input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == ["done %d" % i for i in range(4)]
    la, lb = hp.forward(cfg, params, a), hp.forward(cfg, params, b)
    read = lambda i: np.fromfile(out / ("%d.f32" % i), "<f4").reshape(-1, cfg["vocab"])  # noqa: E731
    assert max_rel(read(0), la[[24, 3]]) < 5e-5
    assert not (out / "1.f32").exists()
    assert max_rel(read(2), la[[26, 29]]) < 5e-5
    assert max_rel(read(3), lb[[16]]) < 5e-5
