"""ctypes binding of libpoptransformer_hybrid.so (include/poptransformer_hybrid.h): the counterpart of `_lib` for the
kernels of decoders with recurrent layers and a 32-bit residual.  A missing library is an error, there is no fallback.
"""
import ctypes
import os
from ctypes import POINTER, c_char_p, c_float, c_int, c_size_t, c_void_p

from ._lib import PTA_EINVAL, PTA_EUNSUPPORTED, PTA_OK, PtaError

LIB_PATH = os.path.join(os.path.dirname(os.path.abspath(__file__)), "libpoptransformer_hybrid.so")

BF16, FP32 = 0, 1
PAIR_NONE, PAIR_SWIGLU, PAIR_CLAMPED = 0, 1, 2
ACT_NONE, ACT_GELU_TANH, ACT_RELU_SQUARE, ACT_SIGMOID = 0, 1, 2, 3
SCORE_SOFTMAX, SCORE_SIGMOID = 0, 1
WINDOW_TILE = 128
MLSTM_SLICE = 32
CONV_TILE = 128
LATENT_TILE = 128
HEAD_TILE = 128
MAX_EXPERTS = 1024


def _struct(name, fields):
    return type(name, (ctypes.Structure,), {"_fields_": fields})


_P, _I, _F = c_void_p, c_int, c_float
WideLinearArgs = _struct("WideLinearArgs", [
    ("dtype", _I), ("X", _P), ("M", _I), ("K", _I), ("N", _I), ("W", _P), ("W2", _P), ("pair", _I), ("limit", _F), ("slope", _F),
    ("cap", _F), ("Y", _P), ("ld", _I), ("n_main", _I), ("out_f32", _I), ("tail", _P), ("tail_count", _I), ("tail_bias", _P),
    ("workspace", _P), ("workspace_bytes", c_size_t), ("bias", _P), ("bias2", _P), ("act", _I), ("mul", _P), ("accumulate", _I)])
StreamsArgs = _struct("StreamsArgs", [
    ("dtype", _I), ("rows", _I), ("width", _I), ("S", _I), ("streams", _P), ("table", _P), ("vocab", _I), ("embed_scale", _F),
    ("ids", _P), ("ids_stride", _I), ("ids_index", _P), ("pos_out", _P), ("y", _P), ("out", _P), ("mix", _P), ("mult", _F),
    ("write_streams", _I), ("gather", _P), ("next_in", _P), ("weight", _P), ("eps", _F), ("h", _P), ("h_ld", _I), ("sum_out", _P)])
WindowArgs = _struct("WindowArgs", [
    ("dtype", _I), ("rows", _I), ("H", _I), ("G", _I), ("D", _I), ("q", _P), ("k", _P), ("gate", _P), ("ld", _I), ("q_norm", _P),
    ("k_norm", _P), ("eps", _F), ("scale", _F), ("slopes", _P), ("window", _I), ("ring", _P), ("rinv", _P), ("ring_len", _I),
    ("slot", _P), ("pos", _P), ("q_scale", _P), ("tile_row", _P), ("tile_count", _P), ("tiles", _I), ("splits", _I),
    ("workspace", _P), ("workspace_bytes", c_size_t), ("out", _P), ("out_ld", _I)])
ShiftNormArgs = _struct("ShiftNormArgs", [
    ("dtype", _I), ("rows", _I), ("width", _I), ("groups", _I), ("x", _P), ("table", _P), ("pos_table", _P), ("vocab", _I),
    ("positions", _I), ("embed_scale", _F), ("ids", _P), ("ids_stride", _I), ("ids_index", _P), ("pos", _P), ("pos_out", _P),
    ("gather", _P), ("eps", _F), ("w1", _P), ("w2", _P), ("shift", _P), ("state", _P), ("slot", _P), ("last", _P), ("h1", _P),
    ("h2", _P), ("hm", _P), ("h_ld", _I)])
LatentArgs = _struct("LatentArgs", [
    ("dtype", _I), ("rows", _I), ("H", _I), ("D", _I), ("P", _I), ("E", _I), ("R", _I), ("q_rank", _I), ("kv_rank", _I), ("proj", _P),
    ("ld", _I), ("q_norm", _P), ("kv_norm", _P), ("eps", _F), ("cq", _P), ("cos_sin", _P), ("positions", _I), ("ring", _P),
    ("ring_len", _I), ("slot", _P), ("pos", _P), ("q", _P), ("uk_t", _P), ("q_latent", _P), ("scale", _F), ("window", _I),
    ("splits", _I), ("part_o", _P), ("part_ml", _P), ("uv", _P), ("gate", _P), ("feature_gate", _P), ("gate_ld", _I), ("out", _P), ("keys", _I), ("key_slot", _P),
    ("key_pos", _P), ("key_latent", _P), ("key_rot", _P), ("kv", _P), ("tile_row", _P), ("tile_count", _P), ("tile_key", _P),
    ("tiles", _I)])
MlstmArgs = _struct("MlstmArgs", [
    ("dtype", _I), ("rows", _I), ("H", _I), ("D", _I), ("E", _I), ("q", _P), ("k", _P), ("v", _P), ("ld", _I), ("gates", _P),
    ("cap", _F), ("state", _P), ("slot", _P), ("seq_row", _P), ("seq_count", _P), ("seqs", _I), ("longest", _I), ("chunked", _I),
    ("o", _P), ("workspace", _P), ("workspace_bytes", c_size_t)])
Conv = _struct("Conv", [("channels", _I), ("taps", _I), ("weight", _P), ("bias", _P), ("silu", _I), ("ring", _P)])
ShortConvArgs = _struct("ShortConvArgs", [
    ("dtype", _I), ("c", Conv), ("x", _P), ("ld_x", _I), ("y", _P), ("ld_y", _I), ("slot", _P), ("pos", _P), ("last", _P), ("tile_row", _P),
    ("tile_count", _P), ("tiles", _I)])
SsdArgs = _struct("SsdArgs", [
    ("dtype", _I), ("rows", _I), ("H", _I), ("G", _I), ("D", _I), ("E", _I), ("x", _P), ("b", _P), ("c", _P), ("ld", _I), ("dt", _P),
    ("dt_bias", _P), ("a_log", _P), ("skip", _P), ("state", _P), ("slot", _P), ("pos", _P), ("seq_row", _P), ("seq_count", _P), ("seqs", _I),
    ("longest", _I), ("chunked", _I), ("y", _P), ("workspace", _P), ("workspace_bytes", c_size_t), ("conv", Conv)])
GatedNormArgs = _struct("GatedNormArgs", [
    ("dtype", _I), ("rows", _I), ("H", _I), ("E", _I), ("vdim", _I), ("parts", _I), ("y", _P), ("z", _P), ("ld_z", _I), ("weight", _P),
    ("eps", _F), ("out", _P)])
HeadArgs = _struct("HeadArgs", [
    ("dtype", _I), ("rows", _I), ("H", _I), ("G", _I), ("maps", _I), ("D", _I), ("E", _I), ("dim", _I), ("vdim", _I), ("q", _P), ("k", _P),
    ("v", _P), ("ld", _I), ("q_norm", _P), ("k_norm", _P), ("eps", _F), ("scale", _F), ("cos_sin", _P), ("positions", _I), ("rot", _I),
    ("window", _I), ("keep", _I), ("chunk", _I), ("keys", _P), ("values", _P), ("ring_len", _I), ("slot", _P), ("pos", _P), ("sink", _P),
    ("lambda_", _F), ("diff", _F), ("head_gate", _P), ("gate", _P), ("tile_row", _P), ("tile_count", _P), ("tiles", _I), ("splits", _I),
    ("workspace", _P), ("workspace_bytes", c_size_t), ("out", _P), ("far1", _P), ("far2", _P), ("conv", Conv)])
Routing = _struct("Routing", [("experts", _I), ("top", _I), ("shared", _I), ("scale", _F), ("chosen", _P), ("weights", _P), ("score", _I),
                              ("correction", _P), ("groups", _I), ("keep", _I), ("share", _I)])
ResultNormArgs = _struct("ResultNormArgs", [
    ("dtype", _I), ("rows", _I), ("width", _I), ("x", _P), ("table", _P), ("vocab", _I), ("embed_scale", _F), ("ids", _P),
    ("ids_stride", _I), ("ids_index", _P), ("pos_out", _P), ("y", _P), ("y_weight", _P), ("parts", _P), ("n_parts", _I), ("parts_ld", _I), ("part_f32", _I),
    ("part_weight", _P), ("weights_ld", _I), ("weight", _P), ("eps", _F), ("final_weight", _P), ("h", _P), ("h_ld", _I), ("router", _P),
    ("routing", Routing)])
DepthNormArgs = _struct("DepthNormArgs", [
    ("dtype", _I), ("rows", _I), ("width", _I), ("history", _P), ("depth_stride", c_size_t), ("depth", _I), ("weights", _P), ("y", _P),
    ("y_weight", _P), ("next", _P), ("centred", _I), ("norm_weight", _P), ("eps", _F), ("h", _P), ("h_ld", _I), ("table", _P), ("vocab", _I),
    ("embed_scale", _F), ("ids", _P), ("ids_stride", _I), ("ids_index", _P), ("pos_out", _P), ("side_table", _P), ("side", _P),
    ("side_layers", _I), ("side_ld", _I), ("side_stride", c_size_t), ("router", _P), ("routing", Routing)])
AddPartsArgs = _struct("AddPartsArgs", [
    ("dtype", _I), ("rows", _I), ("width", _I), ("x", _P), ("parts", _P), ("n_parts", _I), ("parts_ld", _I), ("part_f32", _I),
    ("part_weight", _P), ("weights_ld", _I), ("h", _P), ("h_ld", _I)])
ExpertWeights = _struct("ExpertWeights", [("W", _P), ("W2", _P), ("K", _I), ("N", _I), ("n_main", _I), ("pair", _I), ("limit", _F), ("slope", _F)])
ExpertsArgs = _struct("ExpertsArgs", [
    ("dtype", _I), ("rows", _I), ("experts", _I), ("top", _I), ("choices", _I), ("chosen", _P), ("X", _P), ("ld_x", _I),
    ("routed", ExpertWeights), ("shared", ExpertWeights), ("Y", _P), ("ld_y", _I), ("out_f32", _I), ("lists", _P), ("tile_rows", _I)])

SIGNATURES = {
    "pta_hybrid_last_error": (c_char_p, []),
    "pta_bf16_tiled_bytes": (c_size_t, [_I, _I]),
    "pta_bf16_tile": (_I, [_P, _P, _I, _I, _P]),
    "pta_wide_linear_workspace_bytes": (c_size_t, [_I, _I]),
    "pta_wide_linear": (_I, [POINTER(WideLinearArgs), _P]),
    "pta_wide_linear_group": (_I, [POINTER(WideLinearArgs), _I, _P]),
    "pta_shift_norm": (_I, [POINTER(ShiftNormArgs), _P]),
    **{f"pta_latent_{n}": (_I, [POINTER(LatentArgs), _P]) for n in ("append", "absorb", "rows", "values", "gather", "tiles")},
    "pta_latent_tiles_fit": (_I, [_I, _I, _I, _I]),
    "pta_streams_norm": (_I, [POINTER(StreamsArgs), _P]),
    "pta_window_attention_workspace_bytes": (c_size_t, [_I, _I, _I, _I]),
    "pta_window_append": (_I, [POINTER(WindowArgs), _P]),
    "pta_window_attention": (_I, [POINTER(WindowArgs), _P]),
    "pta_window_decode": (_I, [POINTER(WindowArgs), _P]),
    "pta_head_attention_workspace_bytes": (c_size_t, [_I, _I, _I, _I, _I]),
    **{f"pta_head_{n}": (_I, [POINTER(HeadArgs), _P]) for n in ("append", "attention", "decode")},
    "pta_result_norm": (_I, [POINTER(ResultNormArgs), _P]),
    "pta_route": (_I, [_P, _I, POINTER(Routing), _P]),
    "pta_route_rows": (_I, [_P, _I, _I, _P, POINTER(Routing), _P]),
    "pta_expert_lists_size": (c_size_t, [_I, _I, _I, _I]),
    "pta_group_experts": (_I, [_P, _I, _I, _I, _I, _I, _P, _P]),
    "pta_experts": (_I, [POINTER(ExpertsArgs), _P]),
    "pta_short_conv": (_I, [POINTER(ShortConvArgs), _P]),
    "pta_ssd_state_floats": (c_size_t, [_I, _I, _I]),
    "pta_ssd_workspace_bytes": (c_size_t, [POINTER(SsdArgs)]),
    "pta_ssd": (_I, [POINTER(SsdArgs), _P]),
    "pta_gated_norm": (_I, [POINTER(GatedNormArgs), _P]),
    "pta_depth_norm": (_I, [POINTER(DepthNormArgs), _P]),
    "pta_add_parts": (_I, [POINTER(AddPartsArgs), _P]),
    "pta_mlstm_state_floats": (c_size_t, [_I, _I, _I]),
    "pta_mlstm_workspace_bytes": (c_size_t, [POINTER(MlstmArgs)]),
    "pta_mlstm": (_I, [POINTER(MlstmArgs), _P]),
    "pta_head_norm_gate": (_I, [_I, _P, _P, _P, _I, _P, _I, _I, _I, _I, _F, _P]),
    "pta_argmax_f32": (_I, [_P, _P, _P, _I, _I, _P]),
    "pta_topk_f32": (_I, [_P, _P, _P, _I, _I, _I, _P]),
}

_lib = None


def load():
    """Load the shared library and declare every prototype. Raises if it has not been built."""
    global _lib
    if _lib is None:
        if not os.path.exists(LIB_PATH):
            raise PtaError(f"{LIB_PATH} is missing: build it with `python -m poptransformer_amd.build` "
                           "(there is no CPU fallback for the HIP kernels)")
        lib = ctypes.CDLL(LIB_PATH)
        for name, (res, args) in SIGNATURES.items():
            fn = getattr(lib, name)
            fn.restype, fn.argtypes = res, args
        _lib = lib
    return _lib


def check(rc):
    """Status code -> the exception `_lib.check` raises for it."""
    if rc == PTA_OK:
        return
    msg = load().pta_hybrid_last_error().decode()
    raise {PTA_EINVAL: ValueError, PTA_EUNSUPPORTED: NotImplementedError}.get(rc, PtaError)(msg)
