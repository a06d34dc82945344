"""Deterministic synthetic weights and token ids for the benchmark configurations.

Every tensor gets its own PCG64 stream keyed by (seed, crc32(name)), so tensors
can be generated in any order (or lazily, one at a time) and always hold the
same bytes.  Weights are N(0, 0.02) f32, RMSNorm gains are 1.0; prompts are
uniform ids in [0, vocab).  Parameter names are the HF names the reference
exposes from LlamaModel::named_parameters (src/models/llama.rs:218-279).
"""
import zlib

import numpy as np

# --- model shapes named by the benchmark configurations ----------------------
TINYLLAMA_1B = dict(vocab_size=32000, hidden_size=2048, intermediate_size=5632, num_hidden_layers=22,
                    num_attention_heads=32, num_key_value_heads=4, rms_norm_eps=1e-5, max_seq_len=2048,
                    rope_theta=10000.0)  # src/models/llama.rs:23-37, src/main.rs:171-181
TINYLLAMA_1B_LONG = dict(TINYLLAMA_1B, max_seq_len=4096)
QWEN3_0P6B = dict(vocab_size=151936, hidden_size=1024, intermediate_size=3072, num_hidden_layers=28,
                  num_attention_heads=16, num_key_value_heads=8, rms_norm_eps=1e-6, max_seq_len=1024,
                  rope_theta=1.0e6, head_dim=128, qk_norm=True, tie_embeddings=True)
LLAMA2_7B = dict(vocab_size=32000, hidden_size=4096, intermediate_size=11008, num_hidden_layers=32,
                 num_attention_heads=32, num_key_value_heads=32, rms_norm_eps=1e-5, max_seq_len=1024,
                 rope_theta=10000.0, weight_dtype="bf16")


def head_dim(cfg):
    return cfg.get("head_dim") or cfg["hidden_size"] // cfg["num_attention_heads"]


def param_shapes(cfg):
    """Ordered {hf_name: shape}; weights are [out, in] (src/layers/basic/linear.rs:8)."""
    H, I, V = cfg["hidden_size"], cfg["intermediate_size"], cfg["vocab_size"]
    D = head_dim(cfg)
    qd, kvd = cfg["num_attention_heads"] * D, cfg["num_key_value_heads"] * D
    shapes = {"model.embed_tokens.weight": (V, H)}
    for i in range(cfg["num_hidden_layers"]):
        p = "model.layers.%d." % i
        shapes[p + "self_attn.q_proj.weight"] = (qd, H)
        shapes[p + "self_attn.k_proj.weight"] = (kvd, H)
        shapes[p + "self_attn.v_proj.weight"] = (kvd, H)
        shapes[p + "self_attn.o_proj.weight"] = (H, qd)
        if cfg.get("qk_norm"):
            shapes[p + "self_attn.q_norm.weight"] = (D,)
            shapes[p + "self_attn.k_norm.weight"] = (D,)
        shapes[p + "mlp.gate_proj.weight"] = (I, H)
        shapes[p + "mlp.up_proj.weight"] = (I, H)
        shapes[p + "mlp.down_proj.weight"] = (H, I)
        shapes[p + "input_layernorm.weight"] = (H,)
        shapes[p + "post_attention_layernorm.weight"] = (H,)
    shapes["model.norm.weight"] = (H,)
    if not cfg.get("tie_embeddings"):
        shapes["lm_head.weight"] = (V, H)
    return shapes


def _rng(seed, name):
    return np.random.Generator(np.random.PCG64(np.random.SeedSequence([int(seed), zlib.crc32(name.encode())])))


def is_norm_gain(name):
    return name.endswith("norm.weight") or name.endswith("layernorm.weight")


def make_param(name, shape, seed=0, std=0.02, gains_one=True):
    """One f32 tensor.  With gains_one=False the norm gains are 1 + N(0, 0.1), which
    makes a missing or misplaced gain visible in parity tests."""
    n = int(np.prod(shape))
    if is_norm_gain(name):
        if gains_one:
            return np.ones(shape, np.float32)
        return (1.0 + 0.1 * _rng(seed, name).standard_normal(n, dtype=np.float32)).reshape(shape)
    w = _rng(seed, name).standard_normal(n, dtype=np.float32)
    w *= np.float32(std)
    return w.reshape(shape)


def iter_params(cfg, seed=0, std=0.02, gains_one=True):
    for name, shape in param_shapes(cfg).items():
        yield name, make_param(name, shape, seed, std, gains_one)


def iter_params_threaded(cfg, seed=0, std=0.02, gains_one=True, workers=8, transform=None):
    """iter_params with the tensors generated (and passed through `transform(name, array)`, e.g. a bf16 rounding) by a
    pool of threads a few tensors ahead of the consumer; same bytes, same order (every tensor has its own stream)."""
    from collections import deque
    from concurrent.futures import ThreadPoolExecutor

    def job(name, shape):
        a = make_param(name, shape, seed, std, gains_one)
        return name, (transform(name, a) if transform else a)

    todo = iter(param_shapes(cfg).items())
    with ThreadPoolExecutor(max(1, workers)) as pool:
        ahead = deque()
        for name, shape in todo:
            ahead.append(pool.submit(job, name, shape))
            if len(ahead) >= 2 * workers:
                yield ahead.popleft().result()
        while ahead:
            yield ahead.popleft().result()


def make_params(cfg, seed=0, std=0.02, gains_one=True):
    return dict(iter_params(cfg, seed, std, gains_one))


def make_tokens(n, vocab, seed=0, stream="prompt"):
    return _rng(seed, stream).integers(0, vocab, size=n, dtype=np.int64).astype(np.int32)


def bf16_round(x):
    """f32 -> bf16 bits, round to nearest even (numpy, for test inputs)."""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    r = (u + (0x7FFF + ((u >> 16) & 1))) >> 16
    return r.astype(np.uint16)


def bf16_widen(bits):
    """bf16 bits -> f32, exact (the reference's load-time upcast, src/loader.rs:58)."""
    return (np.ascontiguousarray(bits, np.uint16).astype(np.uint32) << 16).view(np.float32)


# --- layered hybrid decoder (lumen_amd/hybrid.py) beside a Llama of the same size ----------------------
def hybrid_shape(width, weight_dtype="bf16", groups=3, max_seq_len=8192):
    """A HybridConfig whose layers resemble a real model's: groups of attention (window 1024), channel_delta, wkv,
    channel_delta, the middle group run twice; heads of 64 (attention, wkv) and 128 (delta), feed-forward 4 x width
    (two matrices of it hold what three of 8/3 x width do in a SwiGLU layer)."""
    from .hybrid import HybridConfig, HybridLayer
    ff = 4 * width
    delta = dict(heads=width // 128, kv_heads=width // 128, dim=128, vdim=128, conv=4, rank_lo=128, rank_hi=128, ff=ff)
    group = [HybridLayer("attention", heads=width // 64, kv_heads=max(width // 256, 1), dim=64, vdim=64, window=1024,
                         scale=0.125, softcap=30.0, ff=ff),
             HybridLayer("channel_delta", **delta),
             HybridLayer("wkv", heads=width // 64, kv_heads=width // 64, dim=64, vdim=64, rank_lo=64, ff=ff),
             HybridLayer("channel_delta", **delta)]
    mid = groups // 2 * 4
    return HybridConfig(32000, width, group * groups, mid, mid + 4, 2, embed_scale=width ** 0.5, norm_offset=1.0,
                        residual_mult=0.6, max_seq_len=max_seq_len, weight_dtype=weight_dtype)


def llama_beside(width, weight_dtype="bf16", layers=16, max_seq_len=8192):
    """The Llama shape of equal width, layer runs and feed-forward volume."""
    return dict(vocab_size=32000, hidden_size=width, intermediate_size=(8 * width // 3 + 127) // 128 * 128,
                num_hidden_layers=layers, num_attention_heads=width // 64, num_key_value_heads=max(width // 256, 1),
                rms_norm_eps=1e-6, max_seq_len=max_seq_len, rope_theta=10000.0, weight_dtype=weight_dtype)


def nufapel_shape(width, weight_dtype="bf16", groups=3, max_seq_len=8192):
    """A Nufapel HybridConfig of hybrid_shape's width, layer runs and loop: parallel mixers (attention as there but over all
    positions, a matrix memory of half the width beside it) and general delta rules in turn, a dense feed-forward in the
    first layer and 32 experts of width / 4, 8 at a time, in the others."""
    from .hybrid import HybridConfig, HybridLayer
    moe = dict(ff=width // 4, ff_kind="experts", experts=32, top=8, groups=8, keep=4, router_scale=1.0, limit=7.0)
    par = dict(heads=width // 64, kv_heads=max(width // 256, 1), dim=64, vdim=64, scale=0.125, bias_rows=32, bias_max=128,
               mem_heads=max(width // 256, 1), mem_dim=128, mem_vdim=128, gate_cap=15.0)
    gen = dict(heads=width // 64, kv_heads=width // 64, dim=64, vdim=64, rank_lo=64)
    layers = [HybridLayer("parallel" if i % 2 == 0 else "general_delta", **(gen if i % 2 else par),
                          **(moe if i else dict(ff=4 * width, ff_kind="gelu"))) for i in range(4 * groups)]
    mid = groups // 2 * 4
    return HybridConfig(32000, width, layers, mid, mid + 4, 2, max_seq_len=max_seq_len, weight_dtype=weight_dtype, norm_kind="dyt",
                        loop_kind="add", residual_gate=True, max_positions=max_seq_len, logit_softcap=30.0)


def hybrid_param(name, shape, seed):
    """A tensor of a hybrid model: N(0, fan_in^-1/2) matrices, decays that let the state live for tens of tokens."""
    rng = _rng(seed, name)
    leaf = name.split(".")[-1]
    a = rng.standard_normal(shape, dtype=np.float32)
    if name.endswith("conv"):
        return a * np.float32(shape[-1] ** -0.5)
    if leaf in ("norm1", "norm2") or name == "final.norm":
        return a * np.float32(0.1)
    if leaf == "norm":
        return 1 + a * np.float32(0.1)
    if name.startswith("loop.step"):
        return a * np.float32(0.1)
    if len(shape) == 2 and leaf not in ("u",):
        return a * np.float32(shape[-1] ** -0.5)
    if leaf == "act":
        return np.array([0.5, 0.3, 0.2, 0.05], np.float32) + a * np.float32(0.02)
    if leaf in ("r1", "r2") or ".mu." in name:
        return np.abs(a) * np.float32(0.3)
    if leaf in ("w0", "dt_bias"):
        return a * np.float32(0.5) - np.float32(2.5)
    return a * np.float32(0.3)


def nufapel_param(name, shape, seed):
    """A tensor of a Nufapel model: N(0, fan_in^-1/2) matrices; norms whose tanh bends, gates that remember for tens of
    tokens, sinks and distance biases of the size of a score."""
    rng = _rng(seed, name)
    a = rng.standard_normal(shape, dtype=np.float32)
    leaf = name.split(".")[-1]
    if leaf == "alpha":
        return np.float32(0.6) + np.float32(0.1) * np.asarray(a, np.float32)
    if name.endswith(".b") and "norm" in name or name in ("pos", "loop.step"):
        return a * np.float32(0.3)
    if leaf in ("norm1", "norm2", "norm", "out", "temp"):
        return 1 + a * np.float32(0.2)
    if leaf in ("rel", "sink"):
        return a
    if name.endswith(".f.b"):
        return 3 + a
    if name.endswith(".b") or leaf == "w0":
        return a
    if name == "embed":
        return a
    if len(shape) == 2:
        return a * np.float32(shape[-1] ** -0.5 * (2.0 if name.endswith(("mlp.router", "head", "left.q")) else 1.0))
    return a * np.float32(0.3)
