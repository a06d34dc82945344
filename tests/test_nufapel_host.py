"""Nufapel without a GPU: the plain restatement in closed form, config.json and the registry, and the device code on the CPU
under sanitizers (tests/cpu_emu)."""
import math
import os
import subprocess
import sys

import numpy as np
import pytest

import hybrid_util as hu
import nufapel_util as nu
from oracle import nufapel_plain as npn
from test_hybrid_host import ROOT, emulation  # noqa: F401  (the fixture)


# ------------------------------------------------------------------ the plain restatement
def test_plain_attention_in_closed_form():
    z = np.zeros((5, 1, 1))
    v = np.arange(5.0).reshape(5, 1, 1)
    none = np.array([-1e9])
    flat = np.zeros((4, 1))
    assert np.allclose(npn.biased_sink_attention(z, z, v, 1.0, [1.0], flat, 8, none)[:, 0, 0], [0, 0.5, 1, 1.5, 2])
    assert np.allclose(npn.biased_sink_attention(z, z, v + 1, 1.0, [1.0], flat, 8, np.zeros(1))[:, 0, 0], [0.5, 1, 1.5, 2, 2.5])
    rel = np.array([[0.0], [math.log(3.0)], [-1e9], [-1e9]])  # distance 1 counts three times, 2 and beyond nothing
    assert np.allclose(npn.biased_sink_attention(z, z, v, 1.0, [1.0], rel, 8, none)[:, 0, 0], [0, 0.25, 1.25, 2.25, 3.25])
    q, k = np.ones((2, 1, 1)), np.array([0.0, math.log(2.0)]).reshape(2, 1, 1)
    v = np.array([0.0, 1.0]).reshape(2, 1, 1)  # scale 2 and temperature 1/2: weights 1 and 2
    assert np.isclose(npn.biased_sink_attention(q, k, v, 2.0, [0.5], flat, 8, none)[1, 0, 0], 2 / 3)


def test_buckets_of_the_distance_bias():
    assert [npn.bucket(n, 8, 64) for n in (0, 1, 3, 4, 7, 8, 15, 16, 31, 32, 63, 64, 1000)] == [0, 1, 3, 4, 4, 5, 5, 6, 6, 7, 7, 7, 7]
    rows = [npn.bucket(n, 24, 100) for n in range(200)]
    assert rows[:12] == list(range(12)) and rows == sorted(rows) and rows[100] == rows[199] == 23 and rows[99] == 23


def test_plain_recurrences_in_closed_form():
    # one key channel, no removal: a geometric sum of the values
    one, T = np.ones((6, 1, 1)), 6
    S = np.zeros((1, 1, 1))
    o = npn.general_delta_recurrence(one, one, one, one * 0.5, one * 0, S)
    assert np.allclose(o[:, 0, 0], [sum(0.5 ** i for i in range(t + 1)) for t in range(T)])
    # full removal along the unit key, no decay: the last value of a key alone; both terms read the state before the token
    k = np.zeros((3, 1, 2))
    k[[0, 2], 0, 0] = 2
    k[1, 0, 1] = 2
    v = np.array([5.0, 7.0, 9.0]).reshape(3, 1, 1)
    S = np.zeros((1, 2, 1))
    o = npn.general_delta_recurrence(k / 2, k, v, np.ones((3, 1, 2)), np.ones((3, 1, 2)), S)
    assert np.allclose(o[:, 0, 0], [10, 14, 18], atol=1e-4) and np.allclose(S[0, :, 0], [18, 14], atol=1e-4)
    # the matrix memory: a huge input gate forgets what came before; the normaliser divides it out again
    q, v, i = np.ones((3, 1, 1)), np.array([1.0, 2.0, 5.0]).reshape(3, 1, 1), np.array([0.0, 50.0, 0.0]).reshape(3, 1)
    m, n = np.zeros(1), np.zeros((1, 1))
    o = npn.mlstm_recurrence(q, q, v, i, np.zeros((3, 1)), np.zeros((1, 1, 1)), n, m)
    assert np.allclose(o[:, 0, 0], [1, 2, 2], atol=1e-4) and m[0] == 50
    # ... and a small |n.q| is replaced by exp(-m)
    o = npn.mlstm_recurrence(q[:1] * 0.1, q[:1], v[:1], i[:1], np.zeros((1, 1)), np.zeros((1, 1, 1)), np.zeros((1, 1)), np.zeros(1))
    assert np.isclose(o[0, 0, 0], 0.1, atol=1e-5)


def test_plain_router_and_experts():
    z = np.array([9.0, -9, 1, 1, 2, 0.9, -9, -9])
    router = {"top": 2, "scale": 3.0, "groups": {"count": 4, "keep": 1}}
    e, w = npn.route(z, router)  # expert 0 scores best, but its neighbour drags its group below {4, 5}
    s = npn.sigmoid(z)
    assert e == [4, 5] and np.allclose(w, 3.0 * s[[4, 5]] / (s[4] + s[5]))
    assert npn.route(z, {"top": 1, "scale": 1.0})[0] == [0]
    one = {"gate": np.array([[1.0]]), "up": np.array([[1.0]]), "down": np.array([[1.0]])}
    assert np.isclose(npn.clamped_expert(np.array([10.0]), one, 2.0)[0], 2 * npn.sigmoid(3.404) * 3)
    assert np.isclose(npn.clamped_expert(np.array([-10.0]), one, 2.0)[0], -10 * npn.sigmoid(-17.02) * -1)
    assert np.allclose(npn.gelu(np.array([0.0, 1.0, -1.0])), [0, 0.8413447, -0.1586553])


def test_plain_model_is_causal_and_loops_with_its_own_states():
    cfg = nu.config(12, 30, [nu.general(2, 6, nu.dense(20)), nu.parallel((2, 1, 6, 8), (1, 5, 4), nu.moe(6, 4, 2))], loop=(0, 2, 2))
    P = nu.make_params(cfg, seed=1)
    toks = np.arange(14) % 30
    a = npn.forward(cfg, P, toks)
    b = npn.forward(cfg, P, np.concatenate([toks[:9], [3, 3, 3]]))
    assert np.allclose(a[:9], b[:9]) and not np.allclose(a[9], b[9])
    assert npn.layer_runs(cfg) == [(0, 0), (1, None), (0, 1), (1, None)]


# ------------------------------------------------------------------ configuration, registry
def test_config_reader(tmp_path):
    from lumen_amd._lib import LumenError
    from lumen_amd.hybrid import nufapel_config
    from lumen_amd.registry import ARCHITECTURES, architecture, tensor_shape
    assert "Nufapel" in ARCHITECTURES and architecture({"architecture": "Nufapel"}) == "Nufapel"
    cfg = nu.config(24, 30, [nu.parallel((4, 2, 6, 10), (3, 5, 7), nu.moe(9, 8, 3, (4, 2), scale=2.5, limit=0.7), bias_max=70, scale=0.3, cap=11.0),
                             nu.general(2, 8, nu.dense(20)), nu.general(3, 4)], loop=(1, 3, 4), eps=1e-4, softcap=12.0, positions=77)
    P = nu.make_params(cfg, rank=6, bias_rows=14)
    path = os.path.join(hu.write_model(tmp_path, cfg, P), "model.safetensors")
    shape_of = lambda n: tensor_shape(path, n)  # noqa: E731
    assert shape_of("l0.norm1.alpha") == ()
    hc = nufapel_config(cfg, shape_of, 1000, "bf16")
    p, g, last = hc.layers
    assert (p.mixer, p.heads, p.kv_heads, p.dim, p.vdim, p.scale, p.bias_rows, p.bias_max) == ("parallel", 4, 2, 6, 10, 0.3, 14, 70)
    assert (p.mem_heads, p.mem_dim, p.mem_vdim, p.gate_cap) == (3, 5, 7, 11.0)
    assert (p.ff_kind, p.ff, p.experts, p.top, p.groups, p.keep, p.router_scale, p.limit) == ("experts", 9, 8, 3, 4, 2, 2.5, 0.7)
    assert (g.mixer, g.heads, g.kv_heads, g.dim, g.vdim, g.rank_lo, g.ff, g.ff_kind) == ("general_delta", 2, 2, 8, 8, 6, 20, "gelu")
    assert last.ff == 0
    assert (hc.loop_start, hc.loop_stop, hc.loop_times, hc.loop_kind) == (1, 3, 4, "add")
    assert (hc.vocab_size, hc.width, hc.norm_kind, hc.norm_eps, hc.residual_gate, hc.logit_softcap) == (30, 24, "dyt", 1e-4, True, 12.0)
    assert (hc.max_positions, hc.max_seq_len, hc.weight_dtype) == (77, 77, "bf16")
    del cfg["logit_softcap"], cfg["loop"], cfg["layers"][0]["mlp"]["router"]["groups"]
    hc = nufapel_config(cfg, shape_of, 50, "f32")
    assert (hc.logit_softcap, hc.loop_times, hc.max_seq_len, hc.layers[0].groups, hc.layers[0].keep) == (0.0, 0, 50, 1, 1)
    for key, what, match in (("type", "other", "unknown mixer"), ("mlp", {"kind": "other"}, "unknown feed-forward")):
        bad = nu.config(8, 8, [nu.general(1, 4, nu.dense(8))])
        bad["layers"][0][key] = what
        with pytest.raises(LumenError, match=match):
            nufapel_config(bad, lambda n: (1, 1), 8, "f32")


# ------------------------------------------------------------------ the device code on the CPU
# (single cases of the GPU suite: both recurrences over portions, attention in its prompt, portion and decode forms, the
# router, the experts, the row operations, and one model end to end)
@pytest.mark.parametrize("cases", [
    "test_general_delta_recurrence[1-3-4] or test_matrix_memory[1-3-4-100] or test_dynamic_tanh[3-7] or test_router[12-4-3-3]",
    "test_attention_with_distance_bias_sink_and_temperature[2-2-16-16-40] or test_gated_residual_of_one_and_of_a_pair[3-40-37]",
    "test_experts_of_a_prompt[1-8-8-3-2] or test_tiny_model",
])
def test_nufapel_kernels_on_the_cpu_under_sanitizers(emulation, cases):  # noqa: F811
    ids = ["tests/test_gpu_nufapel.py::" + c for c in cases.split(" or ")]
    r = subprocess.run([sys.executable, "-m", "pytest", "-q", "-m", "gpu", "-p", "no:cacheprovider", *ids], cwd=ROOT, env=emulation,
                       capture_output=True, text=True, timeout=900)
    assert r.returncode == 0, (r.stdout[-3000:], r.stderr[-3000:])
    assert "%d passed" % len(ids) in r.stdout
    assert "AddressSanitizer" not in r.stderr and "runtime error" not in r.stderr, r.stderr[-3000:]
