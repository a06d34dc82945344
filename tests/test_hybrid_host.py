"""The layered hybrid decoder without a GPU: the plain restatement against itself and closed forms, config.json and the
registry, the trace runner's bookkeeping -- and the device code itself on the CPU, under sanitizers (tests/cpu_emu)."""
import glob
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import hybrid_util as hu
from oracle import hybrid_plain as hp

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
EMU = os.path.join(ROOT, "tests", "cpu_emu")


# ------------------------------------------------------------------ the plain restatement
def test_plain_mechanisms_in_closed_form():
    # one dimension, constant decay: the WKV state is a geometric sum
    w, T = 0.5, 6
    one = np.ones((T, 1, 1))
    o = hp.wkv_recurrence(one, one, one, one * w, np.full((1, 1), 3.0), np.zeros((1, 1, 1)))
    assert np.allclose(o[:, 0, 0], [3.0 + sum(w ** i for i in range(t)) for t in range(T)])
    # the delta rule with full writes stores the last value of a key and returns it at once
    k = np.zeros((3, 1, 2))
    k[[0, 2], 0, 0] = 1
    k[1, 0, 1] = 1
    v = np.array([5.0, 7.0, 9.0]).reshape(3, 1, 1)
    S = np.zeros((1, 2, 1))
    o = hp.delta_recurrence(k, k, v, np.ones((3, 1, 2)), np.ones((3, 1)), S)
    assert np.allclose(o[:, 0, 0], [5, 7, 9]) and np.allclose(S[0, :, 0], [9, 7])
    # equal scores average the window; a distance bias weighs it
    z = np.zeros((5, 1, 1))
    v = np.arange(5.0).reshape(5, 1, 1)
    assert np.allclose(hp.window_attention(z, z, v, 1.0, 0.0, [0.0], [1.0], 3)[:, 0, 0], [0, 0.5, 1, 2, 3])
    got = hp.window_attention(z, z, v, 1.0, 9.0, [1.0], [1.0], 2)[4, 0, 0]  # weights 1 and 1 / 2
    assert np.isclose(got, (4 + 3 * 0.5) / 1.5)
    assert np.allclose(hp.polynorm(np.array([2.0, -2.0]), [1, 0, 0, 0.5], 0.0), [1.5, -0.5])
    assert np.allclose(hp.polynorm(np.array([2.0, -2.0]), [0, 1, 0, 0], 0.0), [1, 1])
    taps = np.array([[1.0, 10.0]])
    assert np.allclose(hp.causal_conv_silu(np.array([[1.0], [2.0]]), taps), hp.silu(np.array([[10.0], [21.0]])))


def test_plain_model_is_causal_and_loops_with_its_own_states():
    cfg = hu.config(24, 30, [hu.delta(2, 1, 6, 8, ff=20), hu.attention(2, 1, 6, 8, 5), hu.wkv(2, 6)], loop=(0, 2, 2))
    P = hu.make_params(cfg, seed=1)
    toks = np.arange(14) % 30
    a = hp.forward(cfg, P, toks)
    b = hp.forward(cfg, P, np.concatenate([toks[:9], [3, 3, 3]]))
    assert np.allclose(a[:9], b[:9])
    assert [r for r in hp.layer_runs(cfg)] == [(0, 0), (1, None), (0, 1), (1, None), (2, None)]


# ------------------------------------------------------------------ configuration, registry
def test_config_reader(tmp_path):
    from lumen_amd.hybrid import pinavik_config
    from lumen_amd.registry import tensor_shape
    cfg = hu.config(24, 30, [hu.delta(4, 2, 6, 10, conv=5, ff=20), hu.attention(2, 1, 6, 8, 7, scale=0.3, softcap=11.0), hu.wkv(2, 6, ff=9)],
                    loop=(1, 3, 4), eps=1e-4, residual_mult=0.25, scale=2.5)
    P = hu.make_params(cfg, ranks=(5, 11))
    path = os.path.join(hu.write_model(tmp_path, cfg, P), "model.safetensors")
    hc = pinavik_config(cfg, lambda n: tensor_shape(path, n), 77, "bf16")
    d, a, w = hc.layers
    assert (d.mixer, d.heads, d.kv_heads, d.dim, d.vdim, d.conv, d.rank_lo, d.rank_hi, d.ff) == ("channel_delta", 4, 2, 6, 10, 5, 5, 11, 20)
    assert (a.mixer, a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.scale, a.softcap, a.ff) == ("attention", 2, 1, 6, 8, 7, 0.3, 11.0, 0)
    assert (w.mixer, w.heads, w.kv_heads, w.dim, w.vdim, w.rank_lo, w.ff) == ("wkv", 2, 2, 6, 6, 5, 9)
    assert (hc.loop_start, hc.loop_stop, hc.loop_times) == (1, 3, 4)
    assert (hc.vocab_size, hc.width, hc.embed_scale, hc.norm_eps, hc.norm_offset, hc.residual_mult) == (30, 24, 2.5, 1e-4, 1.0, 0.25)
    assert (hc.max_seq_len, hc.weight_dtype) == (77, "bf16")
    del cfg["loop"]
    assert pinavik_config(cfg, lambda n: P[n].shape, 77, "f32").loop_times == 0


def test_unknown_designs_are_refused():
    from lumen_amd._lib import LumenError
    from lumen_amd.hybrid import pinavik_config
    from lumen_amd.registry import ARCHITECTURES, architecture
    assert {"Pinavik", "LlamaForCausalLM", "Qwen3ForCausalLM"} <= set(ARCHITECTURES)
    assert architecture({"architecture": "Pinavik"}) == "Pinavik"
    assert architecture({"architectures": ["Qwen3ForCausalLM"]}) == "Qwen3ForCausalLM"
    for bad in ({}, {"architecture": "Other"}, {"architectures": []}):
        with pytest.raises(LumenError):
            architecture(bad)
    cfg = hu.config(8, 8, [hu.wkv(1, 4)])
    cfg["layers"][0]["type"] = "other"
    with pytest.raises(LumenError, match="unknown mixer"):
        pinavik_config(cfg, lambda n: (1, 1), 8, "f32")
    cfg = hu.config(8, 8, [hu.wkv(1, 4, ff=8)])
    cfg["layers"][0]["mlp"]["kind"] = "other"
    with pytest.raises(LumenError, match="unknown feed-forward"):
        pinavik_config(cfg, lambda n: (1, 1), 8, "f32")


# ------------------------------------------------------------------ trace runner, command line
class Echo:
    """A model whose logits say which token of which sequence they belong to."""
    vocab_size = 3

    def __init__(self):
        self.pos, self.resets = 0, 0

    def step(self, tokens, want):
        rows = np.array([[self.pos + w, tokens[w], self.resets] for w in want], np.float32).reshape(-1, 3)
        self.pos += len(tokens)
        return rows

    def reset(self):
        self.pos = 0
        self.resets += 1


def test_trace_steps(tmp_path):
    from lumen_amd.trace import run_step
    m, out = Echo(), str(tmp_path)
    live = run_step(m, None, {"step": 0, "entries": [{"id": "a", "tokens": [5, 6, 7], "want": [2, 0, 2]}], "end": []}, out)
    assert live == "a"
    assert np.fromfile(tmp_path / "0.f32", "<f4").reshape(-1, 3).tolist() == [[2, 7, 0], [0, 5, 0], [2, 7, 0]]
    live = run_step(m, live, {"step": 1, "entries": [{"id": "a", "tokens": [8], "want": []}], "end": []}, out)
    assert live == "a" and not (tmp_path / "1.f32").exists()
    with pytest.raises(ValueError):
        run_step(m, live, {"step": 2, "entries": [{"id": "b", "tokens": [1], "want": [0]}], "end": []}, out)
    live = run_step(m, "a", {"step": 3, "entries": [{"id": "a", "tokens": [9], "want": [0]}], "end": ["a"]}, out)
    assert live is None and m.resets == 1 and m.pos == 0
    run_step(m, live, {"step": 4, "entries": [{"id": "b", "tokens": [1], "want": [0]}], "end": ["b"]}, out)
    assert np.fromfile(tmp_path / "4.f32", "<f4").tolist() == [0, 1, 1]


def test_trace_main_answers_every_step_before_it_reads_the_next(tmp_path, monkeypatch, capsys):
    from lumen_amd import trace
    monkeypatch.setattr(trace, "load_model", lambda folder, dtype, n: Echo())
    lines = "".join(json.dumps({"step": i, "entries": [{"id": "a", "tokens": [i], "want": [0]}], "end": ["a"] if i == 2 else []}) + "\n" for i in range(3))
    monkeypatch.setattr(sys, "stdin", io.StringIO(lines))
    assert trace.main(["--model", "m", "--dtype", "bfloat16", "--out", str(tmp_path), "--max-tokens", "9"]) == 0
    assert capsys.readouterr().out.split("\n")[:3] == ["done 0", "done 1", "done 2"]
    assert np.fromfile(tmp_path / "2.f32", "<f4").tolist() == [2, 2, 0]


def test_command_line_help():
    r = subprocess.run([sys.executable, "-m", "lumen_amd", "--help"], cwd=ROOT, capture_output=True, text=True, timeout=100)
    assert r.returncode == 0 and "generate" in r.stdout and "trace" in r.stdout
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--help"], capture_output=True, text=True, timeout=100)
    assert r.returncode == 0 and "--max-tokens" in r.stdout


# ------------------------------------------------------------------ the device code on the CPU
@pytest.fixture(scope="module")
def emulation():
    subprocess.run(["make", "-C", EMU, "-j8"], check=True, stdout=subprocess.DEVNULL, stderr=subprocess.PIPE)
    runtime = glob.glob("/opt/rocm/llvm/lib/clang/*/lib/linux/libclang_rt.asan-x86_64.so")
    if not runtime:
        pytest.skip("no shared sanitizer runtime")
    return dict(os.environ, LUMEN_HIP_LIB=os.path.join(EMU, "build", "liblumen_emu.so"), LD_PRELOAD=runtime[0],
                ASAN_OPTIONS="detect_leaks=0")


# (single cases of the GPU suite: both recurrences over portions, the three forms of window attention, the row
# operations, and one model end to end -- prompt, portions, decoding)
@pytest.mark.parametrize("cases", [
    "test_wkv_recurrence[1-3] or test_channel_delta_recurrence[1-1-4-3] or test_polynorm[3-7] or test_token_shift_carries_the_last_token[33]",
    "test_window_attention_in_prompts_portions_and_decoding[2-1-10-7-2-40] or test_convolution_and_unit_vectors[2-3-1-5-9] or test_operators_refuse",
    "test_model_against_the_plain_one[float32-once]",
])
def test_hybrid_kernels_on_the_cpu_under_sanitizers(emulation, cases):
    ids = ["tests/test_gpu_hybrid.py::" + c for c in cases.split(" or ") if "[" in c]
    if "refuse" in cases:
        ids.append("tests/test_gpu_hybrid.py::test_operators_refuse_what_they_cannot_do")
    r = subprocess.run([sys.executable, "-m", "pytest", "-q", "-m", "gpu", "-p", "no:cacheprovider", *ids], cwd=ROOT, env=emulation,
                       capture_output=True, text=True, timeout=900)
    assert r.returncode == 0, (r.stdout[-3000:], r.stderr[-3000:])
    assert "%d passed" % len(ids) in r.stdout
    assert "AddressSanitizer" not in r.stderr and "runtime error" not in r.stderr, r.stderr[-3000:]
