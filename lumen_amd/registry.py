"""Models by the architecture their config.json names.

load_model(folder) reads config.json, picks the model class, builds it and loads model.safetensors.  A further
architecture is one function that turns (config, shape_of, max_seq_len, weight_dtype) into a model, registered under the
name its config.json carries.
"""
import ctypes as C
import json
import os

from . import _lib
from ._lib import ERR_INVALID, LumenError, check, lib
from .hybrid import HybridModel, nufapel_config, pinavik_config
from .models import LlamaConfig, LlamaModel

ARCHITECTURES = {}
WEIGHT_DTYPES = {"bfloat16": "bf16", "bf16": "bf16", "float32": "f32", "f32": "f32"}
DEFAULT_MAX_SEQ_LEN = 32768


def register(*names):
    def add(fn):
        for n in names:
            ARCHITECTURES[n] = fn
        return fn
    return add


@register("LlamaForCausalLM", "Qwen3ForCausalLM")
def _llama(cfg, shape_of, max_seq_len, weight_dtype):
    return LlamaModel(LlamaConfig(
        vocab_size=cfg["vocab_size"], hidden_size=cfg["hidden_size"], intermediate_size=cfg["intermediate_size"],
        num_hidden_layers=cfg["num_hidden_layers"], num_attention_heads=cfg["num_attention_heads"],
        num_key_value_heads=cfg.get("num_key_value_heads") or cfg["num_attention_heads"],
        rms_norm_eps=cfg["rms_norm_eps"], max_seq_len=max_seq_len, rope_theta=cfg.get("rope_theta", 10000.0),
        head_dim=cfg.get("head_dim") or 0, qk_norm="Qwen3ForCausalLM" in cfg.get("architectures", ()),
        tie_embeddings=bool(cfg.get("tie_word_embeddings")), weight_dtype=weight_dtype))


@register("Pinavik")
def _pinavik(cfg, shape_of, max_seq_len, weight_dtype):
    return HybridModel(pinavik_config(cfg, shape_of, max_seq_len, weight_dtype))


@register("Nufapel")
def _nufapel(cfg, shape_of, max_seq_len, weight_dtype):
    return HybridModel(nufapel_config(cfg, shape_of, max_seq_len, weight_dtype))


def tensor_shape(path, name):
    """Shape of a tensor in a safetensors file."""
    dtype, ndim, begin, end = C.c_int(), C.c_int(8), C.c_uint64(), C.c_uint64()
    shape = (C.c_int64 * 8)()
    check(lib.lumen_safetensors_find(str(path).encode(), name.encode(), C.byref(dtype), shape, C.byref(ndim),
                                     C.byref(begin), C.byref(end)))
    return tuple(shape[:ndim.value])


def architecture(cfg):
    """The registered name a config.json carries ("architecture", or the first of "architectures")."""
    name = cfg.get("architecture") or (cfg.get("architectures") or [None])[0]
    if name not in ARCHITECTURES:
        raise LumenError(ERR_INVALID, "architecture %r is not one of %s" % (name, ", ".join(sorted(ARCHITECTURES))))
    return name


def load_model(folder, dtype="bfloat16", max_seq_len=None):
    """The model in `folder` (config.json, model.safetensors), weights stored as `dtype`; its sequence may hold
    max_seq_len tokens (None: what the config states, or DEFAULT_MAX_SEQ_LEN)."""
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    weights = os.path.join(folder, "model.safetensors")
    build = ARCHITECTURES[architecture(cfg)]
    model = build(cfg, lambda name: tensor_shape(weights, name),
                  max_seq_len or cfg.get("max_position_embeddings") or DEFAULT_MAX_SEQ_LEN, WEIGHT_DTYPES[dtype])
    _, missing = model.load_safetensors(weights)
    if missing:
        raise LumenError(ERR_INVALID, "%s lacks %d parameters of the model" % (weights, missing))
    return model
