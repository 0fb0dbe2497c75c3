"""Zekilix decoder: windowed attention and matrix-memory (mLSTM) layers over parallel residual streams.

hf_config: the design's config.json (keys architecture, embedding, layers, logit_softcap, norm, residual_mult, streams,
vocab, width).  Layer i's tensors start with `l<i>.`; a layer with `weights_of` uses another layer's, with a cache or
state of its own.  The model is recorded one token per loop iteration, as the other decoders are; the constants a fused
executor needs are recorded under names of their own (`l<i>.window` and so on).
"""
import numpy as np

from ... import ops
from ...layers import BaseLayer
from ...layers.streams import NamedLinear, StreamConnection, WeightNorm, rms_normalised, scalar
from ..base_model import HFDecBaseModel


def softcapped(graph, x, cap, name):
    c = scalar(graph, cap, name)
    return ops.mul(graph, ops.tanh(graph, ops.div(graph, x, c)), c)


class WindowAttention(BaseLayer):
    """Attention over the newest `window` positions: query / key RMS norm over the whole projection, no rotation, a
    distance bias per head, values that are the keys before their norm, and a sigmoid gate on the result."""

    def __init__(self, context, name, width, eps, max_length, heads, kv_heads, dim, scale, mask=None, vdim=None):
        super().__init__(context, name)
        if vdim not in (None, dim):
            raise ValueError(f"the values are the keys: vdim ({vdim}) must equal dim ({dim})")
        self.heads, self.kv_heads, self.dim, self.scale = heads, kv_heads, dim, scale
        self.window = (mask or {}).get("size")
        self.rows = min(self.window or max_length, max_length)         # cache rows: what slides out of the window is dropped
        H, G = heads * dim, kv_heads * dim
        self.q, self.k, self.g = (NamedLinear(self.context, n, width, c) for n, c in (("q", H), ("k", G), ("g", H)))
        self.q_norm = WeightNorm(self.context, "q.norm", H, eps, centred=False)
        self.k_norm = WeightNorm(self.context, "k.norm", G, eps, centred=False)
        self.o = NamedLinear(self.context, "o", H, width)

    def slopes(self):
        return 2.0 ** (-8.0 * (np.arange(self.heads) + 1) / self.heads)

    def __call__(self, graph, h, layer_id, step, attention_mask):
        B, H, G, D, W = self.batch_size, self.heads, self.kv_heads, self.dim, self.rows
        with graph.nameScope(self.context):
            for fact, value in (("window", self.window or 0), ("heads", H), ("kv_heads", G)):
                ops.constant(graph, np.array(value).astype(np.int32), f"l{layer_id}.{fact}")
            k = self.k(graph, h)
            q = ops.reshape(graph, self.q_norm(graph, self.q(graph, h)), [B, G, H // G, D])
            rows = ops.concat(graph, self.k_norm(graph, k), k, 0)
            past = ops.kv_cache(graph, step, ops.reshape(graph, rows, [2, B, G, 1, D]), W, 3, 1)      # newest first
            past_k, past_v = ops.split(graph, past, 2, axis=0, splits=[1, 1], name="split_past")
            past_k = ops.transpose(graph, ops.squeeze(graph, past_k, [0]), [0, 1, 3, 2])
            s = ops.mul(graph, ops.matmul(graph, q, past_k), scalar(graph, self.scale, f"l{layer_id}.scale"))
            bias = -(self.slopes()[:, None] * np.arange(W)[None]).reshape(1, G, H // G, W)            # entry j: j positions back
            s = ops.add(graph, s, ops.constant(graph, bias.astype(np.float32), "distance_bias"))
            s = ops.add(graph, s, ops.static_slice(graph, attention_mask, [0], [W], [3]))
            p = ops.softmax_ce(graph, s, -1, stable_mode=True)
            o = ops.matmul(graph, p, ops.squeeze(graph, past_v, [0]))
            o = ops.reshape(graph, o, [B, 1, H * D])
            return self.o(graph, ops.mul(graph, o, ops.sigmoid(graph, self.g(graph, h))))


class MatrixMemory(BaseLayer):
    """mLSTM: per head a matrix memory with exponential gates under a running maximum; the state (S, n, m) is carried by
    the loop in fp32."""

    def __init__(self, context, name, width, eps, heads, dim, vdim, gate_cap):
        super().__init__(context, name)
        self.heads, self.dim, self.vdim, self.gate_cap, self.eps = heads, dim, vdim, gate_cap, eps
        N = heads * vdim
        self.q, self.k, self.v, self.g = (NamedLinear(self.context, n, width, c) for n, c in
                                          (("q", heads * dim), ("k", heads * dim), ("v", N), ("g", N)))
        self.i, self.f = (NamedLinear(self.context, n, width, heads, use_bias=True) for n in ("i", "f"))
        self.norm_id = self.add_initialized_input_tensor(
            np.asarray(self.get_param_from_state_dict(f"{self.context}.norm", [N]), np.float32), f"{self.context}.norm")
        self.o = NamedLinear(self.context, "o", N, width)

    def state_shapes(self):
        B, H = self.batch_size, self.heads
        return [B, H, self.dim, self.vdim], [B, H, self.dim, 1], [B, H, 1, 1]

    def __call__(self, graph, h, layer_id, state):
        B, H, D, E = self.batch_size, self.heads, self.dim, self.vdim
        S, n, m = state
        with graph.nameScope(self.context):
            ops.constant(graph, np.array(H).astype(np.int32), f"l{layer_id}.heads")
            q = ops.mul(graph, self.q(graph, h), scalar(graph, D ** -0.5, "query_scale"))
            q = ops.reshape(graph, q, [B, H, 1, D])
            k = ops.reshape(graph, self.k(graph, h), [B, H, D, 1])
            v = ops.reshape(graph, self.v(graph, h), [B, H, 1, E])
            cap = f"l{layer_id}.gate_cap"
            i = softcapped(graph, ops.reshape(graph, self.i(graph, h), [B, H, 1, 1]), self.gate_cap, cap)
            f = softcapped(graph, ops.reshape(graph, self.f(graph, h), [B, H, 1, 1]), self.gate_cap, cap)
            minus = scalar(graph, -1.0, "minus_one")
            f = ops.mul(graph, ops.softplus(graph, ops.mul(graph, f, minus)), minus)                  # log sigmoid
            carried = ops.add(graph, f, m)
            m = ops.maximum(graph, carried, i)
            keep, take = ops.exp(graph, ops.sub(graph, carried, m)), ops.exp(graph, ops.sub(graph, i, m))
            k = ops.mul(graph, k, take)
            S = ops.add(graph, ops.mul(graph, S, keep), ops.mul(graph, k, v))
            n = ops.add(graph, ops.mul(graph, n, keep), k)
            den = ops.abs(graph, ops.matmul(graph, q, n))
            den = ops.maximum(graph, den, ops.exp(graph, ops.mul(graph, m, minus)))
            o = ops.div(graph, ops.matmul(graph, q, S), ops.add(graph, den, scalar(graph, 1e-6, "denominator_eps")))
            o = ops.reshape(graph, rms_normalised(graph, o, self.eps), [B, 1, H * E])
            o = ops.mul(graph, ops.mul(graph, o, self.norm_id), ops.sigmoid(graph, self.g(graph, h)))
            return self.o(graph, o), [S, n, m]


class ClampedGLU(BaseLayer):
    """g = min(W_gate h, limit), u = clamp(W_up h, -limit, limit): W_down (g sigmoid(slope g) (u + 1))."""

    def __init__(self, context, name, width, ff, limit, kind="dense", slope=1.702):
        super().__init__(context, name)
        if kind != "dense":
            raise ValueError(f"Invalid feed-forward {kind}, options: ['dense']")
        self.limit, self.slope = limit, slope
        self.gate, self.up = NamedLinear(self.context, "gate", width, ff), NamedLinear(self.context, "up", width, ff)
        self.down = NamedLinear(self.context, "down", ff, width)

    def __call__(self, graph, h, layer_id):
        with graph.nameScope(self.context):
            ops.constant(graph, np.array(self.limit).astype(np.float32), f"l{layer_id}.limit")
            g = ops.clip(graph, self.gate(graph, h), clip_min=None, clip_max=self.limit)
            u = ops.clip(graph, self.up(graph, h), clip_min=-self.limit, clip_max=self.limit)
            g = ops.mul(graph, g, ops.sigmoid(graph, ops.mul(graph, g, scalar(graph, self.slope, "gate_slope"))))
            return self.down(graph, ops.mul(graph, g, ops.add(graph, u, scalar(graph, 1.0, "one"))))


class Block(BaseLayer):
    """One layer's tensors: mixer and feed-forward with their norms and connections."""

    def __init__(self, context, layer, width, eps, streams, mult, max_length):
        super().__init__(None, context)
        self.kind = layer["type"]
        plain = not streams
        S = streams or 1
        self.norm1 = WeightNorm(self.context, "norm1", width, eps, centred=True)
        self.connect1 = StreamConnection(self.context, "hc1", S, mult, plain)
        if self.kind == "attention":
            self.mixer = WindowAttention(self.context, "mix", width, eps, max_length, **layer["mixer"])
        elif self.kind == "mlstm":
            self.mixer = MatrixMemory(self.context, "mix", width, eps, **layer["mixer"])
        else:
            raise ValueError(f"Invalid mixer {self.kind}, options: ['attention', 'mlstm']")
        self.mlp = None
        if layer.get("mlp") is not None:
            self.norm2 = WeightNorm(self.context, "norm2", width, eps, centred=True)
            self.connect2 = StreamConnection(self.context, "hc2", S, mult, plain)
            self.mlp = ClampedGLU(self.context, "mlp", width, **layer["mlp"])

    def __call__(self, graph, streams, shape, layer_id, step, attention_mask, state):
        new_state = list(state)

        def mix(g, u):
            h = self.norm1(g, u)
            if self.kind == "attention":
                return self.mixer(g, h, layer_id, step, attention_mask)
            y, new_state[:] = self.mixer(g, h, layer_id, state)
            return y

        streams = self.connect1(graph, streams, shape, mix)
        if self.mlp is not None:
            streams = self.connect2(graph, streams, shape, lambda g, u: self.mlp(g, self.norm2(g, u), layer_id))
        return streams, new_state


class ZekilixDecModel(HFDecBaseModel):
    """Greedy or top-k decoder of the design (precision 'bf16' or 'fp32')."""

    def __init__(self, **kwargs):
        super().__init__(**kwargs)
        c = self.hf_config
        if self.precision not in ("bf16", "fp32"):
            raise ValueError(f"Invalid precision {self.precision}, options: ['bf16', 'fp32']")
        self.topk = kwargs.get("topk", 1)
        eps = c.norm["eps"]
        streams = getattr(c, "streams", None)
        self.embed_id = self._tensor("embed", [c.vocab, c.width])
        self.blocks, self.sources = {}, []
        for i, layer in enumerate(c.layers):
            source = i
            while c.layers[source].get("weights_of") is not None:
                source = c.layers[source]["weights_of"]
            self.sources.append(source)
            if source == i:
                self.blocks[i] = Block(f"l{i}", layer, c.width, eps, streams, c.residual_mult, self.max_length)
        self.final_norm = WeightNorm(None, "final.norm", c.width, eps, centred=True)
        self.head = NamedLinear(None, "head", c.width, c.vocab)

    def _tensor(self, key, shape):
        value = self.state_dict.get(key)
        if value is None:
            raise KeyError(f"tensor {key} is missing")
        value = np.asarray(value, np.float32)
        if list(value.shape) != list(shape):
            raise ValueError(f"tensor {key} is {value.shape}, expected {shape}")
        return self.graph.addInitializedInputTensor(value, debugContext=key)

    def _memory_layers(self):
        return [i for i, s in enumerate(self.sources) if self.blocks[s].kind == "mlstm"]

    def build_model_graph_inputs(self, graph, inputs):
        inputs = super().build_model_graph_inputs(graph, inputs)
        with graph.nameScope("states"):
            for i in self._memory_layers():
                for j, shape in enumerate(self.blocks[self.sources[i]].mixer.state_shapes()):
                    inputs[f"state_{i}_{j}"] = ops.constant(self.graph, np.zeros(shape, np.float32), f"layer{i}_{j}")
        return inputs

    def build_model_graph(self, model_graph, model_graph_inputs, sequence_length=1):
        g, c, step = model_graph, self.hf_config, model_graph_inputs["step"]
        S = getattr(c, "streams", None) or 1
        shape = [self.batch_size, 1, c.width]
        ids = ops.dynamic_slice(g, model_graph_inputs["input_ids_container"], step, axes=[1], sizes=[sequence_length])
        mask = ops.unsqueeze(g, model_graph_inputs["attention_mask"], [1, 2])
        x = ops.mul(g, ops.gather(g, self.embed_id, ids), scalar(g, c.embedding["scale"], "embedding_scale"))
        streams = ops.tile(g, ops.reshape(g, x, [1, -1]), [S, 1])
        states = {}
        for i, source in enumerate(self.sources):
            ops.constant(g, np.array(source).astype(np.int32), f"l{i}.source")
            state = [model_graph_inputs[f"state_{i}_{j}"] for j in range(3)] if f"state_{i}_0" in model_graph_inputs else []
            streams, states[i] = self.blocks[source](g, streams, shape, i, step, mask, state)
        x = ops.reshape(g, ops.reduce_sum(g, streams, axes=[0], keepdims=True), shape)
        logits = self.head(g, self.final_norm(g, x))
        if getattr(c, "logit_softcap", None):
            logits = softcapped(g, logits, c.logit_softcap, "logit_softcap")
        if self.topk != 1:
            next_ids = ops.random_sample(g, logits, k=self.topk, dim=2)
        else:
            _, next_ids = ops.topk(g, logits, axis=2, k=1)
        out = {"next_ids": ops.squeeze(g, next_ids, [2]), "stage_offset": 1}
        for i in self._memory_layers():
            for j, t in enumerate(states[i]):
                out[f"states/layer_{i}_{j}"] = t
        return out

    def build_post_model_graph(self, model_graph, model_graph_inputs, model_outputs):
        with self.device_scope(model_graph, 0, pipeline_stage_id=model_outputs["stage_offset"]):
            container, step, mask, new_ids = self.step_containers(
                model_graph, model_graph_inputs["input_ids_container"], model_graph_inputs["step"],
                model_graph_inputs["attention_mask"], model_outputs["next_ids"])
            stop_mask, keep_going = self.step_loop_cond(model_graph, new_ids, model_graph_inputs["stop_mask"])
        self.add_output_tensor(model_graph, [keep_going, container, step, mask, stop_mask] +
                               [v for k, v in model_outputs.items() if k.startswith("states/")])
