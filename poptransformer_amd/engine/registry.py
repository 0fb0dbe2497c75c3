"""Checkpoint directories -> decoders: which family a config.json names, and how its specification and weights are made."""
import json
import os

from . import loader


def _zekilix(cfg, path, max_len, batch, dtype, slots):
    from ..utils import checkpoint
    from .hybrid import HybridDecoder
    spec = loader.zekilix_spec(cfg, max_len, batch, dtype=dtype)
    return HybridDecoder(spec, loader.hybrid_weights(checkpoint.load_state_dict(path, floats="fp32"), spec), slots=slots)


def _ruperax(cfg, path, max_len, batch, dtype, slots):
    from ..utils import checkpoint
    from .parallel import ParallelDecoder
    spec = loader.ruperax_spec(cfg, max_len, batch, dtype=dtype)
    return ParallelDecoder(spec, loader.parallel_weights(checkpoint.load_state_dict(path, floats="fp32"), spec), slots=slots)


def _golapel(cfg, path, max_len, batch, dtype, slots):
    from ..utils import checkpoint
    from .result_norm import ResultNormDecoder
    spec = loader.golapel_spec(cfg, max_len, batch, dtype=dtype)
    return ResultNormDecoder(spec, loader.result_norm_weights(checkpoint.load_state_dict(path, floats="fp32"), spec), slots=slots)


def _sabolorn(cfg, path, max_len, batch, dtype, slots):
    from ..utils import checkpoint
    from .depth import DepthDecoder
    spec = loader.sabolorn_spec(cfg, max_len, batch, dtype=dtype)
    return DepthDecoder(spec, loader.depth_weights(checkpoint.load_state_dict(path, floats="fp32"), spec), slots=slots)


def _fused(spec_of, weights_of):
    def make(cfg, path, max_len, batch, dtype, slots):
        from ..utils import checkpoint
        from .fused import FusedDecoder
        _only_fp16(dtype)
        return FusedDecoder(spec_of(cfg, max_len, batch), weights_of(checkpoint.load_state_dict(path), cfg))
    return make


def _rwkv(cfg, path, max_len, batch, dtype, slots):
    from ..utils import checkpoint
    from .rwkv import RWKVDecoder
    _only_fp16(dtype)
    return RWKVDecoder(loader.rwkv_spec(cfg, max_len, batch), loader.rwkv_weights(checkpoint.load_state_dict(path), cfg))


def _only_fp16(dtype):
    if dtype not in (None, "float16"):
        raise NotImplementedError(f"this family's executor computes in float16, not {dtype}")


# config.json's "architecture" (or the first of "architectures") -> (libraries it needs, maker)
ARCHITECTURES = {
    "Zekilix": (("hybrid",), _zekilix),
    "Ruperax": (("hybrid",), _ruperax),
    "Golapel": (("hybrid",), _golapel),
    "Sabolorn": (("hybrid",), _sabolorn),
    "GPT2LMHeadModel": (("hip", "hybrid"), _fused(loader.gpt2_spec, loader.gpt2_weights)),
    "LlamaForCausalLM": (("hip", "hybrid"), _fused(loader.llama2_spec, loader.llama2_weights)),
    "ChatGLMModel": (("hip", "hybrid"), _fused(loader.chatglm2_spec, loader.chatglm2_weights)),
    "RwkvForCausalLM": (("hip", "hybrid"), _rwkv),
}


def read_config(path):
    with open(os.path.join(path, "config.json")) as f:
        return json.load(f)


def architecture(cfg):
    """(name, libraries, maker) of a configuration."""
    name = cfg.get("architecture") or (cfg.get("architectures") or [None])[0]
    if name not in ARCHITECTURES:
        raise ValueError(f"unknown architecture {name}; known: {sorted(ARCHITECTURES)}")
    return (name, *ARCHITECTURES[name])


def open_decoder(path, max_len, batch=1, dtype=None, slots=None):
    """The decoder of the checkpoint directory `path` (config.json beside the weights)."""
    cfg = read_config(path)
    _, _, make = architecture(cfg)
    return make(cfg, path, max_len, batch, dtype, slots)
