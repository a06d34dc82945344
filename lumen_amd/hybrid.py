"""The layered hybrid decoder (lumen_hybrid_*): layers with different sequence mixers -- sliding-window attention, WKV,
channel-wise gated delta rule, generalised delta rule, attention and a matrix memory side by side --, PolyNorm, GELU or
expert feed-forwards, and a range of layers that may run several times over.

HybridConfig holds a model of that family whatever its origin; pinavik_config and nufapel_config read the config.json of
the two designs into one.
"""
import ctypes as C
import warnings
from dataclasses import dataclass, field
from typing import List

import numpy as np

from . import _lib
from ._lib import ERR_INVALID, LumenError, check, lib
from .autograd import default_ctx
from .models import DecoderModel

MIXERS = {"attention": 0, "wkv": 1, "channel_delta": 2, "general_delta": 3, "parallel": 4}
FEED_FORWARDS = {"polynorm": 0, "gelu": 1, "experts": 2}
NORMS = {"rms": 0, "dyt": 1}
LOOPS = {"mix": 0, "add": 1}  # what enters a pass: W_in [x; x0] + step, or x + step


@dataclass
class HybridLayer:
    mixer: str
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    window: int = 0       # attention: positions a query sees, itself included; 0: all
    scale: float = 1.0    # attention
    softcap: float = 0.0  # attention; 0: none
    conv: int = 1         # channel_delta: taps
    rank_lo: int = 0      # inner size of the decay's low-rank product
    rank_hi: int = 0      # channel_delta: inner size of the gate's
    ff: int = 0           # 0: no feed-forward; of an expert where there are several
    ff_kind: str = "polynorm"
    bias_rows: int = 0    # parallel: rows of the learned distance bias
    bias_max: int = 0     # ... distance at which its last row is reached
    mem_heads: int = 0    # parallel: the matrix memory's heads, their key and value sizes
    mem_dim: int = 0
    mem_vdim: int = 0
    gate_cap: float = 0.0
    experts: int = 0
    top: int = 0          # experts a token uses
    groups: int = 1
    keep: int = 1         # groups a token's experts may come from
    router_scale: float = 1.0
    limit: float = 0.0    # clamp inside an expert


@dataclass
class HybridConfig:
    vocab_size: int
    width: int
    layers: List[HybridLayer] = field(default_factory=list)
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 0
    embed_scale: float = 1.0
    norm_eps: float = 1e-6
    norm_offset: float = 0.0  # added to the stored weights of the stream's norms
    residual_mult: float = 1.0
    unit_eps: float = 1e-6
    max_seq_len: int = 32768
    max_chunk: int = 0
    weight_dtype: str = "f32"
    norm_kind: str = "rms"
    loop_kind: str = "mix"
    residual_gate: bool = False
    max_positions: int = 0      # learned position vectors; 0: none
    logit_softcap: float = 0.0  # 0: none


class HybridModel(DecoderModel):
    ABI = "lumen_hybrid_"
    KERNEL_CLASSES = ("embedding", "loop_gemv", "attn_proj_gemv", "attn", "wkv_proj_gemv", "wkv", "delta_proj_gemv",
                      "delta", "out_gemv", "up_gemv", "down_gemv", "head_gemv", "general_proj_gemv", "general", "parallel_proj_gemv",
                      "memory", "pair", "experts_up", "experts_down")

    def __init__(self, config, ctx=None):
        self.config = config
        self.vocab_size = config.vocab_size
        self.ctx = ctx or default_ctx()
        n = len(config.layers)
        layers = (_lib.HybridLayerStruct * max(n, 1))(*[
            _lib.HybridLayerStruct(MIXERS[y.mixer], y.heads, y.kv_heads, y.dim, y.vdim, y.window, y.scale, y.softcap,
                                   y.conv, y.rank_lo, y.rank_hi, y.ff, FEED_FORWARDS[y.ff_kind], y.bias_rows, y.bias_max,
                                   y.mem_heads, y.mem_dim, y.mem_vdim, y.gate_cap, y.experts, y.top, y.groups, y.keep,
                                   y.router_scale, y.limit) for y in config.layers])
        c = _lib.HybridConfigStruct(
            config.vocab_size, config.width, n, config.loop_start, config.loop_stop, config.loop_times,
            config.embed_scale, config.norm_eps, config.norm_offset, config.residual_mult, config.unit_eps,
            config.max_seq_len, config.max_chunk,
            _lib.DTYPE_BF16 if config.weight_dtype == "bf16" else _lib.DTYPE_F32, NORMS[config.norm_kind],
            LOOPS[config.loop_kind], int(config.residual_gate), config.max_positions, config.logit_softcap)
        h = C.c_void_p()
        check(lib.lumen_hybrid_create(self.ctx.handle, C.byref(c), layers, C.byref(h)))
        self.handle = h

    def named_parameter_shapes(self):
        n = C.c_int()
        self._call("num_params", C.byref(n))
        out = {}
        name, shape, ndim = C.create_string_buffer(128), (C.c_int64 * 4)(), C.c_int()
        for i in range(n.value):
            self._call("param_info", i, name, 128, shape, C.byref(ndim))
            out[name.value.decode()] = tuple(shape[:ndim.value])
        return out

    @property
    def length(self):
        """Tokens the live sequence holds."""
        n = C.c_int()
        self._call("len", C.byref(n))
        return n.value

    @property
    def num_runs(self):
        n = C.c_int()
        self._call("num_runs", C.byref(n))
        return n.value

    def step(self, token_ids, want, residual=False):
        """residual=True: also the residual stream after every layer run, [runs, tokens, width]."""
        ids = np.ascontiguousarray(token_ids, np.int32).reshape(-1)
        want = np.ascontiguousarray(want, np.int32).reshape(-1)
        out = np.empty((want.size, self.vocab_size), np.float32)
        taps = np.empty((self.num_runs, ids.size, self.config.width), np.float32) if residual else None
        self._call("forward", ids.ctypes.data, ids.size, want.ctypes.data, want.size, out.ctypes.data,
                   taps.ctypes.data if residual else None)
        return (out, taps) if residual else out


def _known(d, keys, where):
    extra = sorted(set(d) - set(keys))
    if extra:
        warnings.warn("config.json: %s: ignoring unknown %s" % (where, ", ".join(extra)))


def pinavik_config(cfg, shape_of, max_seq_len, weight_dtype):
    """config.json of a Pinavik model -> HybridConfig.  shape_of(name) gives a tensor's shape: the inner sizes of the
    low-rank products are stated nowhere else."""
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        kind, m, mlp = entry["type"], entry["mixer"], entry.get("mlp")
        if kind not in ("attention", "wkv", "channel_delta"):
            raise LumenError(ERR_INVALID, "config.json: layer %d: unknown mixer %r" % (i, kind))
        if mlp is not None and mlp["kind"] != "dense":
            raise LumenError(ERR_INVALID, "config.json: layer %d: unknown feed-forward %r" % (i, mlp["kind"]))
        y = HybridLayer(kind, m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"]),
                        ff=mlp["ff"] if mlp is not None else 0)
        pre = "l%d.mix." % i
        if kind == "attention":
            _known(m, ("heads", "kv_heads", "dim", "vdim", "mask", "scale", "softcap"), "attention of layer %d" % i)
            y.window, y.scale, y.softcap = m["mask"]["size"], m["scale"], m.get("softcap") or 0.0
        elif kind == "wkv":
            _known(m, ("heads", "dim"), "wkv of layer %d" % i)
            y.rank_lo = shape_of(pre + "w1")[0]
        else:
            _known(m, ("heads", "kv_heads", "dim", "vdim", "conv"), "channel_delta of layer %d" % i)
            y.conv, y.rank_lo, y.rank_hi = m["conv"], shape_of(pre + "a1")[0], shape_of(pre + "g1")[0]
        layers.append(y)
    loop = cfg.get("loop") or {"start": 0, "stop": 0, "times": 0}
    return HybridConfig(cfg["vocab"], cfg["width"], layers, loop["start"], loop["stop"], loop["times"],
                        embed_scale=cfg.get("embedding", {}).get("scale", 1.0), norm_eps=cfg["norm"]["eps"], norm_offset=1.0,
                        residual_mult=cfg.get("residual_mult", 1.0), unit_eps=1e-6, max_seq_len=max_seq_len,
                        weight_dtype=weight_dtype)


def nufapel_config(cfg, shape_of, max_seq_len, weight_dtype):
    """config.json of a Nufapel model -> HybridConfig.  shape_of(name) gives a tensor's shape: the rows of the distance bias
    and the inner size of the decay's low-rank product are stated nowhere else."""
    layers = []
    for i, entry in enumerate(cfg["layers"]):
        kind, m, mlp = entry["type"], entry["mixer"], entry.get("mlp")
        pre, where = "l%d.mix." % i, "layer %d" % i
        if kind == "general_delta":
            _known(m, ("heads", "dim"), "general_delta of " + where)
            y = HybridLayer(kind, m["heads"], m["heads"], m["dim"], m["dim"], rank_lo=shape_of(pre + "w1")[0])
        elif kind == "parallel":
            a, r = m["left"], m["right"]
            _known(a, ("heads", "kv_heads", "dim", "vdim", "scale", "bias_max"), "left mixer of " + where)
            _known(r, ("heads", "dim", "vdim", "gate_cap"), "right mixer of " + where)
            y = HybridLayer(kind, a["heads"], a.get("kv_heads", a["heads"]), a["dim"], a.get("vdim", a["dim"]), scale=a["scale"],
                            bias_rows=shape_of(pre + "left.rel")[0], bias_max=a["bias_max"], mem_heads=r["heads"], mem_dim=r["dim"],
                            mem_vdim=r.get("vdim", r["dim"]), gate_cap=r["gate_cap"])
        else:
            raise LumenError(ERR_INVALID, "config.json: layer %d: unknown mixer %r" % (i, kind))
        if mlp is not None:
            if mlp["kind"] == "dense":
                y.ff, y.ff_kind = mlp["ff"], "gelu"
            elif mlp["kind"] == "moe":
                e, r = mlp["expert"], mlp["router"]
                _known(e, ("ff", "limit"), "experts of " + where)
                _known(r, ("experts", "top", "scale", "groups"), "router of " + where)
                g = r.get("groups") or {"count": 1, "keep": 1}
                y.ff, y.ff_kind, y.limit = e["ff"], "experts", e["limit"]
                y.experts, y.top, y.router_scale, y.groups, y.keep = r["experts"], r["top"], r.get("scale", 1.0), g["count"], g["keep"]
            else:
                raise LumenError(ERR_INVALID, "config.json: layer %d: unknown feed-forward %r" % (i, mlp["kind"]))
        layers.append(y)
    loop = cfg.get("loop") or {"start": 0, "stop": 0, "times": 0}
    positions = cfg["max_positions"]
    return HybridConfig(cfg["vocab"], cfg["width"], layers, loop["start"], loop["stop"], loop["times"], norm_eps=cfg["norm"]["eps"],
                        unit_eps=1e-6, max_seq_len=min(max_seq_len, positions), weight_dtype=weight_dtype, norm_kind="dyt", loop_kind="add",
                        residual_gate=True, max_positions=positions, logit_softcap=cfg.get("logit_softcap") or 0.0)
