"""State dict (numpy, reference key names) -> device weights of the fused executor.

Mirrors what the reference layers do when they bind their weights
(poptransformer/layers/linear.py:28-40 with utils/param_handler/precision_strategy.py:24-51):
an int8 `<ctx>.weight` is a packed INT4 matrix [out, in/2] with `<ctx>.weight_scale`; other
Linear weights are fp16 [out, in].  Weights are re-tiled on the device once, here.
"""
import numpy as np
import torch

from .. import kernels as K
from .fused import BlockWeights, DecoderSpec, LinearWeights, ModelWeights


def _dev(a, device):
    return torch.from_numpy(np.ascontiguousarray(a)).to(device)


def f143_encode_device(w, scale):
    """fp32/fp16 device tensor -> F143 bytes with exponent `scale` (the bind-time conversion of
    utils/param_handler/precision_strategy.py:44-51), through the library's own encoder."""
    sc = torch.tensor([scale], dtype=torch.int32, device=w.device)
    return K.half_to_fp8(w.half().contiguous(), sc, "F143"), sc


def linear_from_state_dict(sd, ctx, use_bias, device="cuda", precision="fp16", fp8_scale=-1):
    w = sd[ctx + ".weight"]
    w = w if isinstance(w, np.ndarray) else np.asarray(w)
    bias = _dev(np.asarray(sd[ctx + ".bias"], np.float16), device) if use_bias else None
    if precision in ("fp8", "fp8_weight"):
        w8, sc = f143_encode_device(_dev(w.astype(np.float16), device), fp8_scale)
        return LinearWeights(K.F8Weight(w8, sc, "F143"), bias, act_fp8=precision == "fp8", scale_value=fp8_scale)
    if w.dtype == np.int8:
        scale = sd.get(ctx + ".weight_scale")
        if scale is None:
            raise KeyError(f"{ctx}.weight is packed INT4 but {ctx}.weight_scale is missing")
        tw = K.W4Weight(_dev(w, device), _dev(np.asarray(scale, np.float16), device))
    else:
        tw = K.F16Weight(_dev(w.astype(np.float16), device))
    return LinearWeights(tw, bias)


def llama2_weights(sd, cfg, device="cuda"):
    d = cfg["hidden_size"]
    hd = d // cfg["num_attention_heads"]
    blocks = []
    for i in range(cfg["num_hidden_layers"]):
        p = f"model.layers.{i}."
        blocks.append(BlockWeights(
            norm1=(_dev(sd[p + "input_layernorm.weight"], device), None),
            norm2=(_dev(sd[p + "post_attention_layernorm.weight"], device), None),
            qkv=[linear_from_state_dict(sd, p + "self_attn." + n, False, device) for n in ("q_proj", "k_proj", "v_proj")],
            out=linear_from_state_dict(sd, p + "self_attn.o_proj", False, device),
            mlp_in=[linear_from_state_dict(sd, p + "mlp." + n, False, device) for n in ("gate_proj", "up_proj")],
            mlp_out=linear_from_state_dict(sd, p + "mlp.down_proj", False, device)))
    inv_freq = np.array([1.0 / (10000 ** (i / hd)) for i in range(0, hd, 2)]).astype(np.float16)
    return ModelWeights(embed=_dev(sd["model.embed_tokens.weight"], device), pos_embed=None, blocks=blocks,
                        final_norm=(_dev(sd["model.norm.weight"], device), None),
                        head=linear_from_state_dict(sd, "lm_head", False, device), inv_freq=_dev(inv_freq, device))


def llama2_spec(cfg, max_len, batch, pad_id=0, eos_id=2, early_stop=False, fp8_cache=False):
    d, h = cfg["hidden_size"], cfg["num_attention_heads"]
    return DecoderSpec("llama2", cfg["num_hidden_layers"], d, h, h, d // h, cfg["vocab_size"], max_len, batch,
                       cfg["rms_norm_eps"], pad_id, eos_id, early_stop, fp8_cache=fp8_cache)


def gpt2_weights(sd, cfg, device="cuda"):
    blocks = []
    for i in range(cfg["n_layer"]):
        p = f"transformer.h.{i}."
        blocks.append(BlockWeights(
            norm1=(_dev(sd[p + "ln_1.weight"], device), _dev(sd[p + "ln_1.bias"], device)),
            norm2=(_dev(sd[p + "ln_2.weight"], device), _dev(sd[p + "ln_2.bias"], device)),
            qkv=[linear_from_state_dict(sd, p + "attn.c_attn", True, device)],
            out=linear_from_state_dict(sd, p + "attn.c_proj", True, device),
            mlp_in=[linear_from_state_dict(sd, p + "mlp.c_fc", True, device)],
            mlp_out=linear_from_state_dict(sd, p + "mlp.c_proj", True, device)))
    wte = _dev(sd["transformer.wte.weight"], device)
    return ModelWeights(embed=wte, pos_embed=_dev(sd["transformer.wpe.weight"], device), blocks=blocks,
                        final_norm=(_dev(sd["transformer.ln_f.weight"], device), _dev(sd["transformer.ln_f.bias"], device)),
                        head=LinearWeights(K.F16Weight(wte)), inv_freq=None)


def gpt2_spec(cfg, max_len, batch, pad_id=50257, eos_id=50256, early_stop=False):
    d, h = cfg["n_embd"], cfg["n_head"]
    return DecoderSpec("gpt2", cfg["n_layer"], d, h, h, d // h, cfg["vocab_size"], max_len, batch,
                       cfg["layer_norm_epsilon"], pad_id, eos_id, early_stop)


def chatglm2_weights(sd, cfg, precision="fp16", scales=None, device="cuda"):
    scales = scales or {}
    hd = cfg["hidden_size"] // cfg["num_attention_heads"]

    def lin(ctx, bias):
        return linear_from_state_dict(sd, ctx, bias, device, precision, scales.get(ctx, -1))

    blocks = []
    for i in range(cfg["num_layers"]):
        p = f"transformer.encoder.layers.{i}."
        blocks.append(BlockWeights(
            norm1=(_dev(sd[p + "input_layernorm.weight"], device), None),
            norm2=(_dev(sd[p + "post_attention_layernorm.weight"], device), None),
            qkv=[lin(p + "self_attention.query", True), lin(p + "self_attention.key_value", True)],
            out=lin(p + "self_attention.dense", False),
            mlp_in=[lin(p + "mlp.dense_h_to_4h_1", False), lin(p + "mlp.dense_h_to_4h_2", False)],
            mlp_out=lin(p + "mlp.dense_4h_to_h", False)))
    rot = hd // 2
    inv_freq = np.array([1.0 / (10000 ** (i / rot)) for i in range(0, rot, 2)]).astype(np.float32)
    return ModelWeights(embed=_dev(sd["transformer.embedding.word_embeddings.weight"], device), pos_embed=None,
                        blocks=blocks, final_norm=(_dev(sd["transformer.encoder.final_layernorm.weight"], device), None),
                        head=lin("transformer.output_layer", False), inv_freq=_dev(inv_freq, device))


def chatglm2_spec(cfg, max_len, batch, pad_id=0, eos_id=2, early_stop=False):
    d, h = cfg["hidden_size"], cfg["num_attention_heads"]
    return DecoderSpec("chatglm2", cfg["num_layers"], d, h, cfg["multi_query_group_num"], d // h,
                       cfg["padded_vocab_size"], max_len, batch, cfg["layernorm_epsilon"], pad_id, eos_id, early_stop)


def rwkv_weights(sd, cfg, device="cuda"):
    from .rwkv import RWKVBlockWeights, RWKVWeights

    def ln(key):
        return (_dev(sd[key + ".weight"], device), _dev(sd[key + ".bias"], device))

    def vec(key):
        return _dev(np.asarray(sd[key], np.float16).reshape(-1), device)

    blocks = []
    for i in range(cfg["num_hidden_layers"]):
        p = f"rwkv.blocks.{i}."
        blocks.append(RWKVBlockWeights(
            pre_ln=ln(p + "pre_ln") if i == 0 else None, ln1=ln(p + "ln1"), ln2=ln(p + "ln2"),
            att_key=linear_from_state_dict(sd, p + "attention.key", False, device),
            att_value=linear_from_state_dict(sd, p + "attention.value", False, device),
            att_receptance=linear_from_state_dict(sd, p + "attention.receptance", False, device),
            att_output=linear_from_state_dict(sd, p + "attention.output", False, device),
            time_decay=vec(p + "attention.time_decay"), time_first=vec(p + "attention.time_first"),
            att_mix=[vec(p + f"attention.time_mix_{n}") for n in ("key", "value", "receptance")],
            ffn_key=linear_from_state_dict(sd, p + "feed_forward.key", False, device),
            ffn_receptance=linear_from_state_dict(sd, p + "feed_forward.receptance", False, device),
            ffn_value=linear_from_state_dict(sd, p + "feed_forward.value", False, device),
            ffn_mix=[vec(p + f"feed_forward.time_mix_{n}") for n in ("key", "receptance")]))
    return RWKVWeights(embed=_dev(sd["rwkv.embeddings.weight"], device), blocks=blocks, ln_out=ln("rwkv.ln_out"),
                       head=linear_from_state_dict(sd, "head", False, device))


def rwkv_spec(cfg, max_len, batch, pad_id=0, eos_id=-1, early_stop=False):
    from .rwkv import RWKVSpec
    return RWKVSpec(cfg["num_hidden_layers"], cfg["hidden_size"], cfg["attention_hidden_size"], cfg["intermediate_size"],
                    cfg["vocab_size"], max_len, batch, cfg["layer_norm_epsilon"], cfg["rescale_every"], pad_id, eos_id,
                    early_stop)


def hybrid_layers(layers):
    """The `layers` list of a hybrid configuration -> [HybridLayer].  `weights_of` may point to a layer that itself
    uses another one's tensors."""
    from .hybrid import ClampedGLU, HybridLayer, MemoryMixer, WindowMixer
    out = []
    for i, c in enumerate(layers):
        m, kind = c["mixer"], c["type"]
        if kind == "attention":
            if m.get("vdim", m["dim"]) != m["dim"]:
                raise ValueError(f"layer {i}: the values are the keys, so vdim ({m['vdim']}) must equal dim ({m['dim']})")
            mixer = WindowMixer(m["heads"], m["kv_heads"], m["dim"], float(m["scale"]), (m.get("mask") or {}).get("size"))
        elif kind == "mlstm":
            mixer = MemoryMixer(m["heads"], m["dim"], m["vdim"], float(m["gate_cap"]))
        else:
            raise NotImplementedError(f"layer {i}: mixer {kind}")
        f = c.get("mlp")
        if f is not None and f.get("kind", "dense") != "dense":
            raise NotImplementedError(f"layer {i}: feed-forward {f['kind']}")
        source = i
        while layers[source].get("weights_of") is not None:
            source = layers[source]["weights_of"]
        out.append(HybridLayer(mixer, ClampedGLU(f["ff"], float(f["limit"])) if f is not None else None, source))
    return out


def zekilix_spec(cfg, max_len, batch, pad_id=0, eos_id=-1, early_stop=False, dtype="bfloat16", topk=1):
    from .hybrid import HybridSpec
    return HybridSpec("zekilix", hybrid_layers(cfg["layers"]), cfg["width"], cfg["vocab"], cfg.get("streams") or 1,
                      cfg["norm"]["eps"], cfg["residual_mult"], cfg["embedding"]["scale"], cfg.get("logit_softcap") or 0.0, max_len, batch, pad_id, eos_id,
                      early_stop, topk, dtype)


def _lookup(tensors, device):
    """(tensor of a name and shape on the device, fp32 vector of a name and length) over name -> tensor or array."""
    def get(name, shape):
        if name not in tensors:
            raise KeyError(f"tensor {name} is missing")
        t = tensors[name]
        t = (t if torch.is_tensor(t) else torch.from_numpy(np.ascontiguousarray(t))).to(device)
        if tuple(t.shape) != tuple(shape):
            raise ValueError(f"tensor {name} is {tuple(t.shape)}, expected {tuple(shape)}")
        return t

    def vec(name, n):
        return get(name, (n,)).float().contiguous()
    return get, vec


def hybrid_weights(tensors, spec, device="cuda"):
    """tensors: name -> tensor or array (names as in a checkpoint of the design).  Concatenates the projections of a mixer,
    pads, and lays the weights out for the device; layers that use another one's tensors have no entry of their own."""
    from .. import hybrid_kernels as HK
    from .hybrid import HybridLayerWeights, HybridWeights
    dtype = HK.DTYPES[spec.dtype]
    get, vec = _lookup(tensors, device)
    d, S = spec.width, spec.streams
    layers = []
    for i, lay in enumerate(spec.layers):
        if lay.source != i:
            layers.append(None)
            continue
        p, m = f"l{i}.", lay.mixer
        mix = p + "mix."

        def connect(q):
            hc = p + f"hc{q}."
            if S == 1 and hc + "in" not in tensors:            # a plain residual
                one = torch.ones(1, dtype=torch.float32, device=device)
                return (one, one, one)
            return (vec(hc + "in", S), vec(hc + "out", S), get(hc + "mix", (S, S)).float().contiguous())

        N = m.out_channels
        lw = dict(norm1=vec(p + "norm1", d), connect1=connect(1), out=HK.WideWeight(get(mix + "o", (d, N)), dtype))
        if m.kind == "attention":
            KD = m.kv_heads * m.dim
            parts = [get(mix + "q", (N, d)), get(mix + "k", (KD, d)), get(mix + "g", (N, d))]
            lw.update(proj=HK.WideWeight(torch.cat(parts), dtype), q_norm=vec(mix + "q.norm", N), k_norm=vec(mix + "k.norm", KD),
                      slopes=torch.tensor(m.slopes(), dtype=torch.float32, device=device))
        else:
            QD = m.heads * m.dim
            parts = [get(mix + "q", (QD, d)), get(mix + "k", (QD, d)), get(mix + "v", (N, d)), get(mix + "g", (N, d)),
                     get(mix + "i", (m.heads, d)), get(mix + "f", (m.heads, d))]
            bias = torch.cat([vec(mix + "i.b", m.heads), vec(mix + "f.b", m.heads)])
            lw.update(proj=HK.WideWeight(torch.cat(parts), dtype, tail=2 * m.heads, tail_bias=bias), head_norm=vec(mix + "norm", N))
        if lay.mlp is not None:
            ff, mlp = lay.mlp.ff, p + "mlp."
            lw.update(norm2=vec(p + "norm2", d), connect2=connect(2),
                      gate=HK.WideWeight(get(mlp + "gate", (ff, d)), dtype, main_to=HK.pad8(ff)),
                      up=HK.WideWeight(get(mlp + "up", (ff, d)), dtype, main_to=HK.pad8(ff)),
                      down=HK.WideWeight(get(mlp + "down", (d, ff)), dtype))
        layers.append(HybridLayerWeights(**lw))
    return HybridWeights(get("embed", (spec.vocab, d)).to(dtype).contiguous(), layers, vec("final.norm", d),
                         HK.WideWeight(get("head", (spec.vocab, d)), dtype))


# ----------------------------------------------------------------------------------- layers with sublayers side by side
def latent_layers(layers):
    """The `layers` list of a configuration with latent attention -> [HybridLayer]."""
    from .hybrid import BiasedSwiGLU, HybridLayer, LatentMixer, Rotation
    out = []
    for i, c in enumerate(layers):
        if c["type"] != "latent_attention":
            raise NotImplementedError(f"layer {i}: mixer {c['type']}")
        m, rot = c["mixer"], c["mixer"]["rot"]
        if rot["dims"] % 2 or rot["dims"] > m["rot_dim"]:
            raise ValueError(f"layer {i}: {rot['dims']} rotated features of {m['rot_dim']}")
        source = m.get("kv_from")
        mixer = LatentMixer(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"], float(m["scale"]),
                            (m.get("mask") or {}).get("size"), Rotation(float(rot["base"]), rot["dims"]), source)
        if source is not None:
            if not 0 <= source < i or out[source].mixer.source is not None:
                raise ValueError(f"layer {i}: kv_from {source} names no earlier layer with a cache of its own")
            o = out[source].mixer
            if (o.kv_rank, o.rot_dim, o.rot) != (mixer.kv_rank, mixer.rot_dim, mixer.rot):
                raise ValueError(f"layer {i}: the latent or the rotation differs from layer {source}'s")
        f = c.get("mlp")
        if f is not None and f.get("kind", "dense") != "dense":
            raise NotImplementedError(f"layer {i}: feed-forward {f['kind']}")
        out.append(HybridLayer(mixer, BiasedSwiGLU(f["ff"]) if f is not None else None, i, shift=True))
    return out


def ruperax_spec(cfg, max_len, batch, pad_id=0, eos_id=-1, early_stop=False, dtype="bfloat16", topk=1):
    from .hybrid import HybridSpec
    scale = (cfg.get("embedding") or {}).get("scale")
    return HybridSpec("ruperax", latent_layers(cfg["layers"]), cfg["width"], cfg["vocab"], 1, cfg["norm"]["eps"], 1.0,
                      1.0 if scale is None else scale, 0.0, max_len, batch, pad_id, eos_id, early_stop, topk, dtype,
                      norm_groups=cfg["norm"].get("groups") or 1, positions=cfg["max_positions"])


def _padded(t, *shape):
    """t in the corner of a zero tensor of the given shape."""
    if tuple(t.shape) == shape:
        return t
    out = torch.zeros(shape, dtype=t.dtype, device=t.device)
    out[tuple(slice(n) for n in t.shape)] = t
    return out


def _latent_tensors(get, vec, mix, m, d, dtype, device):
    """Of a layer with latent attention: the rows of its projection up to the gate, and the weights behind it."""
    from .. import hybrid_kernels as HK
    heads, D, P, E, R, q_rank, kv_rank = m.sizes
    Qp, pairs = HK.pad8(q_rank), torch.from_numpy(m.pairs()).to(device)
    parts = [_padded(get(mix + "dq", (q_rank, d)), Qp, d)]
    if m.source is None:
        dkv = get(mix + "dkv", (kv_rank + m.rot_dim, d))
        parts += [_padded(dkv[:kv_rank], R, d), _padded(dkv[kv_rank:][pairs], P, d)]
    uq = get(mix + "uq", (heads * (m.dim + m.rot_dim), q_rank)).view(heads, m.dim + m.rot_dim, q_rank)
    uq = torch.cat([_padded(uq[:, :m.dim], heads, D, q_rank), _padded(uq[:, m.dim:][:, pairs], heads, P, q_rank)], 1)
    uk = _padded(get(mix + "uk", (heads * m.dim, kv_rank)).view(heads, m.dim, kv_rank), heads, D, R)
    uv = _padded(get(mix + "uv", (heads * m.vdim, kv_rank)).view(heads, m.vdim, kv_rank), heads, E, R)
    o = _padded(get(mix + "o", (d, heads * m.vdim)).view(d, heads, m.vdim), d, heads, E)
    kv = HK.WideWeight(torch.cat([uk.reshape(-1, R), uv.reshape(-1, R)]), dtype) if HK.latent_tiles_fit(dtype, D, P, E) else None
    return parts, dict(q_norm=vec(mix + "dq.norm", q_rank), kv_norm=vec(mix + "dkv.norm", kv_rank) if m.source is None else None,
                       uq=HK.WideWeight(uq.reshape(-1, q_rank), dtype), uk_t=uk.transpose(1, 2).to(dtype).contiguous(),
                       uv=uv.to(dtype).contiguous(), kv=kv, out=HK.WideWeight(o.reshape(d, -1), dtype))


def parallel_weights(tensors, spec, device="cuda"):
    """As hybrid_weights, for layers with latent attention whose sublayers stand side by side.  Every head size is rounded up to
    what the kernels take, with zeros; the two features of a rotated pair come to stand side by side, in queries and keys."""
    from .. import hybrid_kernels as HK
    from .parallel import ParallelLayerWeights, ParallelWeights
    dtype = HK.DTYPES[spec.dtype]
    get, vec = _lookup(tensors, device)
    d = spec.width
    layers = []
    for i, lay in enumerate(spec.layers):
        p, m = f"l{i}.", lay.mixer
        mix = p + "mix."
        parts, latent = _latent_tensors(get, vec, mix, m, d, dtype, device)
        parts.append(get(mix + "g", (m.heads, d)))
        lw = dict(norm1=vec(p + "norm1", d), shift=vec(p + "shift", d), gate1=HK.WideWeight(get(p + "rg1", (d, d)), dtype),
                  gate1_bias=vec(p + "rg1.b", d), proj=HK.WideWeight(torch.cat(parts), dtype, tail=m.heads), **latent)
        if lay.mlp is not None:
            ff, mlp = lay.mlp.ff, p + "mlp."
            n = HK.pad8(ff)
            lw.update(norm2=vec(p + "norm2", d), gate2=HK.WideWeight(get(p + "rg2", (d, d)), dtype), gate2_bias=vec(p + "rg2.b", d),
                      gate=HK.WideWeight(get(mlp + "gate", (ff, d)), dtype, main_to=n), gate_bias=_padded(vec(mlp + "gate.b", ff), n),
                      up=HK.WideWeight(get(mlp + "up", (ff, d)), dtype, main_to=n), up_bias=_padded(vec(mlp + "up.b", ff), n),
                      down=HK.WideWeight(get(mlp + "down", (d, ff)), dtype), down_bias=vec(mlp + "down.b", d))
        layers.append(ParallelLayerWeights(**lw))
    return ParallelWeights(get("embed", (spec.vocab, d)).to(dtype).contiguous(), get("pos", (spec.positions, d)).to(dtype).contiguous(),
                           layers, vec("final.norm", d), HK.WideWeight(get("head", (spec.vocab, d)), dtype))


# ----------------------------------------------------------------------------------- residual that takes normed results
def _rotation(rot, neighbours, yarn, where):
    from .hybrid import Rotation
    if rot is None:
        return None
    if rot["dims"] % 2 or rot["dims"] < 2:
        raise ValueError(f"{where}: {rot['dims']} rotated features")
    s = rot.get("scaling")
    if s is None:
        return Rotation(float(rot["base"]), rot["dims"], neighbours)
    return Rotation(float(rot["base"]), rot["dims"], neighbours, float(s["factor"]),
                    (float(s["original"]), float(s["fast"]), float(s["slow"])) if yarn else None)


def head_layers(layers):
    """The `layers` list of a configuration with attention by heads and feed-forwards that may be mixtures of experts ->
    [HybridLayer].  Types: `attention` (sliding window with kept first positions, sinks, values that are the keys), `attention_2`
    (differential, within chunks, no rotation), `attention_3` (within chunks)."""
    from .hybrid import ClampedGLU, Experts, HeadMixer, HybridLayer, SwiGLU
    out = []
    for i, c in enumerate(layers):
        m, kind = c["mixer"], c["type"]
        mask, where = m.get("mask") or {}, f"layer {i}"
        mixer = HeadMixer(m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["scale"]))
        if kind == "attention":
            mixer.window, mixer.keep = mask.get("size"), mask.get("keep_first") or 0
            mixer.rot = _rotation(m.get("rot"), False, False, where)
            mixer.keys_are_values, mixer.biases, mixer.sink, mixer.gate = True, "qk", True, "head"
            if mixer.vdim != mixer.dim:
                raise ValueError(f"{where}: the values are the keys, so vdim ({mixer.vdim}) must equal dim ({mixer.dim})")
        elif kind == "attention_2":
            mixer.chunk, mixer.diff = mask.get("size"), float(m["diff"])
        elif kind == "attention_3":
            mixer.chunk, mixer.biases, mixer.gate = mask.get("size"), "qkv", "feature"
            mixer.rot = _rotation(m.get("rot"), True, True, where)
        else:
            raise NotImplementedError(f"{where}: mixer {kind}")
        if mixer.heads % mixer.kv_heads or (mixer.rot is not None and mixer.rot.dims > mixer.dim):
            raise ValueError(f"{where}: {mixer.heads} heads on {mixer.kv_heads}, rotation {m.get('rot')} of {mixer.dim} features")
        f, mlp = c.get("mlp"), None
        if f is not None and f.get("kind", "dense") == "dense":
            mlp = SwiGLU(f["ff"])
        elif f is not None and f["kind"] == "moe":
            r, s = f["router"], f.get("shared")
            mlp = Experts(r["experts"], r["top"], float(r["scale"]), ClampedGLU(f["expert"]["ff"], float(f["expert"]["limit"])),
                          ClampedGLU(s["ff"], float(s["limit"])) if s is not None else None)
        elif f is not None:
            raise NotImplementedError(f"{where}: feed-forward {f['kind']}")
        out.append(HybridLayer(mixer, mlp, i))
    return out


def golapel_spec(cfg, max_len, batch, pad_id=0, eos_id=-1, early_stop=False, dtype="bfloat16", topk=1):
    from .hybrid import HybridSpec
    return HybridSpec("golapel", head_layers(cfg["layers"]), cfg["width"], cfg["vocab"], 1, cfg["norm"]["eps"], 1.0, cfg["embedding"]["scale"],
                      0.0, max_len, batch, pad_id, eos_id, early_stop, topk, dtype)


def _head_rows(t, heads, size, which, stored):
    """[heads * size, ...] in the order `which` of every head's features, each head padded to `stored`"""
    t = t.view(heads, size, -1)[:, which]
    return _padded(t, heads, stored, t.shape[2]).reshape(heads * stored, -1)


def _glu(get, make, names, ff, d, dtype):
    """Gate, up and down of one feed-forward or of several alike.  make(tensors, dtype, further keywords) -> weight; names: prefixes of
    their tensors"""
    from .. import hybrid_kernels as HK
    from .result_norm import FeedForwardWeights
    n = HK.pad8(ff)
    gate, up = (make([get(p + part, (ff, d)) for p in names], dtype, main_to=n) for part in ("gate", "up"))
    return FeedForwardWeights(gate, up, make([get(p + "down", (d, ff)) for p in names], dtype))


def result_norm_weights(tensors, spec, device="cuda"):
    """As hybrid_weights, for layers with attention by heads.  Head sizes are rounded up to whole pieces of eight features with
    zeros; the two features of a rotated pair come to stand side by side in queries and keys (and so in values that are keys)."""
    from .. import hybrid_kernels as HK
    from .hybrid import Experts
    from .result_norm import ResultNormLayerWeights, ResultNormWeights
    dtype = HK.DTYPES[spec.dtype]
    get, vec = _lookup(tensors, device)
    d = spec.width

    layers = []
    for i, lay in enumerate(spec.layers):
        p, m, mlp = f"l{i}.", lay.mixer, lay.mlp
        mix = p + "mix."
        H, G, M, D, E = m.heads, m.kv_heads, m.maps, m.stored_dim, m.stored_vdim
        pairs = torch.from_numpy(m.rot.pairs(m.dim) if m.rot is not None else np.arange(m.dim)).to(device)
        order = pairs if m.keys_are_values else torch.arange(m.vdim, device=device)

        rows = _head_rows
        parts = [("q", H * M, m.dim, pairs, D), ("k", G * M, m.dim, pairs, D)]
        if not m.keys_are_values:
            parts.append(("v", G, m.vdim, order, E))
        if m.gate == "feature":
            parts.append(("g", H, m.vdim, order, E))
        weights = [rows(get(mix + n, (heads * size, d)), heads, size, which, stored) for n, heads, size, which, stored in parts]
        if m.gate == "head":
            weights.append(get(mix + "g", (H, d)))
        bias = None
        if m.biases:
            bias = torch.cat([rows(vec(mix + n + ".b", heads * size) if n in m.biases else torch.zeros(heads * size, device=device),
                                   heads, size, which, stored).reshape(-1) for n, heads, size, which, stored in parts]).contiguous()
        o = get(mix + "o", (d, H * m.vdim)).view(d, H, m.vdim)[:, :, order]
        lw = dict(norm1=vec(p + "norm1", d), proj=HK.WideWeight(torch.cat(weights), dtype, tail=H if m.gate == "head" else 0), proj_bias=bias,
                  out=HK.WideWeight(_padded(o, d, H, E).reshape(d, -1), dtype), q_norm=_padded(vec(mix + "q.norm", m.dim)[pairs], D),
                  k_norm=_padded(vec(mix + "k.norm", m.dim)[pairs], D), sink=vec(mix + "sink", H) if m.sink else None)
        if m.diff is not None:
            a1, b1, a2, b2 = (vec(mix + n, m.dim).double() for n in ("lq1", "lk1", "lq2", "lk2"))
            lw.update(lam=float(torch.exp((a1 * b1).sum()) - torch.exp((a2 * b2).sum())) + m.diff)
        if mlp is not None:
            lw.update(norm2=vec(p + "norm2", d))
        mp = p + "mlp."
        if isinstance(mlp, Experts):
            lw.update(ff=_glu(get, HK.ExpertWeight, [f"{mp}e{e}." for e in range(mlp.count)], mlp.expert.ff, d, dtype), top=mlp.top)
            router = [get(mp + "router", (mlp.count, d))]
            if mlp.shared is not None:
                lw.update(shared=_glu(get, HK.ExpertWeight, [mp + "shared."], mlp.shared.ff, d, dtype))
                router.append(get(mp + "shared.sg", (1, d)))
            router = torch.cat(router)
            lw.update(router=_padded(router, router.shape[0], HK.pad8(d)).to(dtype).contiguous(), router_linear=HK.WideWeight(router, dtype))
        elif mlp is not None:
            lw.update(ff=_glu(get, lambda w, *a, **kw: HK.WideWeight(w[0], *a, **kw), [mp], mlp.ff, d, dtype))
        layers.append(ResultNormLayerWeights(**lw))
    embed = get("embed", (spec.vocab, d)).to(dtype).contiguous()
    return ResultNormWeights(embed, layers, vec("final.norm", d), HK.WideWeight(embed, dtype))


# ----------------------------------------------------------------------------------- results averaged over the depths
def depth_layers(layers):
    """The `layers` list of a configuration with latent attention (an output gate per feature, neighbours rotated), attention by heads
    (short convolutions, a penalty of the distance) and the state-space recurrence -> [HybridLayer]."""
    from .hybrid import Experts, HeadMixer, HybridLayer, LatentMixer, SquaredReLU, StateSpaceMixer, SwiGLU
    out = []
    for i, c in enumerate(layers):
        m, kind, where = c["mixer"], c["type"], f"layer {i}"
        if kind == "latent_attention":
            rot, source = _rotation(m["rot"], True, True, where), m.get("kv_from")
            if rot.dims > m["rot_dim"]:
                raise ValueError(f"{where}: {rot.dims} rotated features of {m['rot_dim']}")
            mixer = LatentMixer(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"], float(m["scale"]), None, rot, source,
                                "feature")
            if source is not None:
                o = out[source].mixer if 0 <= source < i else None
                if getattr(o, "kind", None) != "latent" or o.source is not None:
                    raise ValueError(f"{where}: kv_from {source} names no earlier layer with a cache of its own")
                if (o.kv_rank, o.rot_dim, o.rot) != (mixer.kv_rank, mixer.rot_dim, rot):
                    raise ValueError(f"{where}: the latent or the rotation differs from layer {source}'s")
        elif kind == "attention":
            mixer = HeadMixer(m["heads"], m["kv_heads"], m["dim"], m["vdim"], float(m["scale"]), biases="qkv", norms=False, far=True,
                              taps=m["conv"])
            if mixer.heads % mixer.kv_heads:
                raise ValueError(f"{where}: {mixer.heads} heads on {mixer.kv_heads}")
        elif kind == "mamba2":
            mixer = StateSpaceMixer(m["heads"], m["groups"], m["state"], m["vdim"], m["conv"], m["norm_groups"])
            if mixer.heads % mixer.groups or mixer.heads * mixer.vdim % mixer.norm_parts:
                raise ValueError(f"{where}: {mixer.heads} heads of {mixer.vdim} in {mixer.groups} groups, normed in {mixer.norm_parts}")
        else:
            raise NotImplementedError(f"{where}: mixer {kind}")
        f, mlp = c.get("mlp"), None
        if f is not None and f.get("kind", "dense") == "dense":
            mlp = SquaredReLU(f["ff"])
        elif f is not None and f["kind"] == "moe":
            r = f["router"]
            g = r.get("groups") or {"count": 1, "keep": 1}
            if r["experts"] % g["count"] or r["experts"] // g["count"] * g["keep"] < r["top"]:
                raise ValueError(f"{where}: {r['top']} of {r['experts']} experts, {g['keep']} of {g['count']} groups")
            mlp = Experts(r["experts"], r["top"], 1.0, SwiGLU(f["expert"]["ff"]), None, "sigmoid", True, g["count"], g["keep"], True)
        elif f is not None:
            raise NotImplementedError(f"{where}: feed-forward {f['kind']}")
        out.append(HybridLayer(mixer, mlp, i))
    return out


def sabolorn_spec(cfg, max_len, batch, pad_id=0, eos_id=-1, early_stop=False, dtype="bfloat16", topk=1):
    from .hybrid import HybridSpec
    scale = (cfg.get("embedding") or {}).get("scale")
    return HybridSpec("sabolorn", depth_layers(cfg["layers"]), cfg["width"], cfg["vocab"], 1, cfg["norm"]["eps"], 1.0, 1.0 if scale is None else scale,
                      cfg.get("logit_softcap") or 0.0, max_len, batch, pad_id, eos_id, early_stop, topk, dtype, side_dim=cfg["token_side"]["dim"])


def depth_weights(tensors, spec, device="cuda"):
    """As hybrid_weights, for layers whose results are averaged over the depths.  Head and state sizes are rounded up to whole pieces of
    eight features (latent ones as _latent_tensors does) with zeros."""
    from .. import hybrid_kernels as HK
    from .depth import DepthLayerWeights, DepthWeights
    from .hybrid import Experts
    dtype = HK.DTYPES[spec.dtype]
    get, vec = _lookup(tensors, device)
    d, n_side = spec.width, spec.side_dim

    def by_heads(t, heads, size, stored):
        return _head_rows(t, heads, size, slice(None), stored)

    layers = []
    for i, lay in enumerate(spec.layers):
        p, m, mlp = f"l{i}.", lay.mixer, lay.mlp
        mix = p + "mix."
        side = HK.pad8(n_side)
        lw = dict(norm=vec(p + "norm1", d), average=vec(p + "dwa", i + 2), side_norm=vec(p + "side.norm", d),
                  side_gate=HK.WideWeight(get(p + "side.gate", (n_side, d)), dtype, main_to=side),
                  side_proj=HK.WideWeight(get(p + "side.proj", (d, n_side)), dtype))
        if m.kind == "latent":
            parts, latent = _latent_tensors(get, vec, mix, m, d, dtype, device)
            E = m.sizes[3]
            parts.append(by_heads(get(mix + "g", (m.heads * m.vdim, d)), m.heads, m.vdim, E))
            lw.update(latent, proj=HK.WideWeight(torch.cat(parts), dtype))
        elif m.kind == "heads":
            H, G, D, E = m.heads, m.kv_heads, m.stored_dim, m.stored_vdim
            parts = [("q", H, m.dim, D), ("k", G, m.dim, D), ("v", G, m.vdim, E)]
            lw.update(proj=HK.WideWeight(torch.cat([by_heads(get(mix + n, (h * s, d)), h, s, e) for n, h, s, e in parts]), dtype),
                      proj_bias=torch.cat([by_heads(vec(mix + n + ".b", h * s), h, s, e).reshape(-1) for n, h, s, e in parts]).contiguous(),
                      conv=HK.ShortConv(torch.cat([by_heads(get(mix + n + ".conv", (h * s, m.taps)).float(), h, s, e) for n, h, s, e in parts])
                                        .t().contiguous()),
                      far=(vec(mix + "r1", H), vec(mix + "r2", H)))
        else:
            H, G, D, E = m.heads, m.groups, m.stored_dim, m.stored_vdim
            inner, states = H * m.vdim, G * m.dim
            columns = [(inner, H, m.vdim, E), (states, G, m.dim, D), (states, G, m.dim, D)]                # x | b | c

            def convolved(t):
                return torch.cat([by_heads(u, h, s, e) for u, (_, h, s, e) in zip(torch.split(t, [c[0] for c in columns]), columns)])
            w = get(mix + "in", (2 * inner + 2 * states + H, d))
            lw.update(proj=HK.WideWeight(torch.cat([by_heads(w[:inner], H, m.vdim, E), convolved(w[inner:-H]), w[-H:]]), dtype, tail=H),
                      conv=HK.ShortConv(convolved(get(mix + "conv", (inner + 2 * states, m.taps)).float()).t().contiguous(),
                                        convolved(vec(mix + "conv.b", inner + 2 * states)).reshape(-1).contiguous(), silu=True),
                      ssd=(vec(mix + "dt_bias", H), vec(mix + "A_log", H), vec(mix + "D", H)),
                      head_norm=by_heads(vec(mix + "norm", inner), H, m.vdim, E).reshape(-1).contiguous())
        if m.kind != "latent":
            o = get(mix + "o", (d, m.heads * m.vdim)).view(d, m.heads, m.vdim)
            lw.update(out=HK.WideWeight(_padded(o, d, m.heads, m.stored_vdim).reshape(d, -1), dtype))
        mp = p + "mlp."
        if isinstance(mlp, Experts):
            router = get(mp + "router", (mlp.count, d))
            lw.update(ff=_glu(get, HK.ExpertWeight, [f"{mp}e{e}." for e in range(mlp.count)], mlp.expert.ff, d, dtype), top=mlp.top,
                      router=_padded(router, mlp.count, HK.pad8(d)).to(dtype).contiguous(), router_linear=HK.WideWeight(router, dtype, whole=True),
                      correction=vec(mp + "correction", mlp.count))
        elif mlp is not None:
            lw.update(up=HK.WideWeight(get(mp + "up", (mlp.ff, d)), dtype, main_to=HK.pad8(mlp.ff)),
                      down=HK.WideWeight(get(mp + "down", (d, mlp.ff)), dtype))
        layers.append(DepthLayerWeights(**lw))
    embed = get("embed", (spec.vocab, d)).to(dtype).contiguous()
    own = get("side.embed", (spec.vocab, len(layers) * n_side)).view(spec.vocab, len(layers), n_side)
    own = _padded(own, spec.vocab, len(layers), HK.pad8(n_side)).to(dtype).contiguous()
    return DepthWeights(embed, own, layers, vec("final.norm", d), HK.WideWeight(embed, dtype))
