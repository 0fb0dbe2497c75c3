"""Ruperax decoder: latent attention over a sliding window beside a SwiGLU feed-forward, both gated, on one residual.

hf_config: the design's config.json (keys architecture, embedding, layers, max_positions, norm, vocab, width).  Layer i's
tensors start with `l<i>.`; a layer whose mixer has `kv_from` reads another layer's cache.  The model is recorded one token
per loop iteration, as the other decoders are; what a fused executor needs is recorded in constants of the layers (`l<i>.mixer`,
`l<i>.rotation`).
"""
import numpy as np

from ... import ops
from ...engine.loader import latent_layers
from ...layers import BaseLayer
from ...layers.latent import LatentAttention
from ...layers.parallel import BiasedSwiGLU, GroupedRMSNorm, ResultGate, RotaryTable, TokenShift
from ...layers.streams import NamedLinear, WeightNorm, scalar
from ..base_model import HFDecBaseModel


class Block(BaseLayer):
    """x + gate1 * mixer(shift(norm1(x))) + gate2 * ff(norm2(x))."""

    def __init__(self, context, layer, width, eps, groups, max_length, rotation):
        super().__init__(None, context)
        self.norm1 = GroupedRMSNorm(self.context, "norm1", width, eps, groups)
        self.shift = TokenShift(self.context, "shift", width)
        self.mixer = LatentAttention(self.context, "mix", width, eps, max_length, layer.mixer, rotation)
        self.gate1 = ResultGate(self.context, "rg1", width)
        self.mlp = None
        if layer.mlp is not None:
            self.norm2 = GroupedRMSNorm(self.context, "norm2", width, eps, groups)
            self.mlp = BiasedSwiGLU(self.context, "mlp", width, layer.mlp.ff)
            self.gate2 = ResultGate(self.context, "rg2", width)

    def __call__(self, graph, x, layer_id, step, attention_mask, before, caches, cache_rows):
        h1 = self.norm1(graph, x)
        h, before = self.shift(graph, h1, before)
        source = self.mixer.mixer.source
        if source is None:
            source, caches[layer_id] = layer_id, self.mixer.cache(graph, h, step, cache_rows)
        y = self.gate1(graph, h1, self.mixer(graph, h, layer_id, step, attention_mask, caches[source]))
        if self.mlp is not None:
            h2 = self.norm2(graph, x)
            y = ops.add(graph, y, self.gate2(graph, h2, self.mlp(graph, h2)))
        return ops.add(graph, x, y), before


class RuperaxDecModel(HFDecBaseModel):
    """Greedy or top-k decoder of the design (precision 'bf16' or 'fp32')."""

    def __init__(self, **kwargs):
        super().__init__(**kwargs)
        c = self.hf_config
        if self.precision not in ("bf16", "fp32"):
            raise ValueError(f"Invalid precision {self.precision}, options: ['bf16', 'fp32']")
        if self.max_length > c.max_positions:
            raise ValueError(f"max_length {self.max_length}: the model has {c.max_positions} positions")
        self.topk = kwargs.get("topk", 1)
        eps, groups = c.norm["eps"], c.norm.get("groups") or 1
        self.embed_id = self._tensor("embed", [c.vocab, c.width])
        self.pos_id = self._tensor("pos", [c.max_positions, c.width])
        rotations = {}
        self.blocks = []
        for i, layer in enumerate(latent_layers(c.layers)):
            rot = layer.mixer.rot
            key = (rot.base, rot.dims)
            if key not in rotations:
                rotations[key] = RotaryTable(f"rotary{len(rotations)}", self.max_length, *key)
            self.blocks.append(Block(f"l{i}", layer, c.width, eps, groups, self.max_length, rotations[key]))
        self.final_norm = GroupedRMSNorm(None, "final.norm", c.width, eps, groups)
        self.head = NamedLinear(None, "head", c.width, c.vocab)
        # a cache holds what the widest window over it sees
        self.cache_rows = [max(b.mixer.rows for j, b in enumerate(self.blocks) if i in (j, b.mixer.mixer.source)) for i in range(len(self.blocks))]

    def _tensor(self, key, shape):
        value = self.state_dict.get(key)
        if value is None:
            raise KeyError(f"tensor {key} is missing")
        value = np.asarray(value, np.float32)
        if list(value.shape) != list(shape):
            raise ValueError(f"tensor {key} is {value.shape}, expected {shape}")
        return self.graph.addInitializedInputTensor(value, debugContext=key)

    def build_model_graph_inputs(self, graph, inputs):
        inputs = super().build_model_graph_inputs(graph, inputs)
        with graph.nameScope("states"):
            for i, b in enumerate(self.blocks):
                inputs[f"state_{i}"] = ops.constant(self.graph, np.zeros(b.shift.state_shape(), np.float32), f"layer{i}")
        return inputs

    def build_model_graph(self, model_graph, model_graph_inputs, sequence_length=1):
        g, c, step = model_graph, self.hf_config, model_graph_inputs["step"]
        shape = [self.batch_size, 1, c.width]
        ids = ops.dynamic_slice(g, model_graph_inputs["input_ids_container"], step, axes=[1], sizes=[sequence_length])
        mask = ops.unsqueeze(g, model_graph_inputs["attention_mask"], [1, 2])
        ops.constant(g, np.array(self.final_norm.groups).astype(np.int32), "norm_groups")
        x = ops.mul(g, ops.gather(g, self.embed_id, ids), scalar(g, c.embedding["scale"], "embedding_scale"))
        pos = ops.dynamic_slice(g, self.pos_id, step, axes=[0], sizes=[1])
        x = ops.add(g, ops.reshape(g, x, shape), ops.reshape(g, pos, [1, 1, c.width]))
        out, caches = {"stage_offset": 1}, {}
        for i, block in enumerate(self.blocks):
            x, out[f"states/layer_{i}"] = block(g, x, i, step, mask, model_graph_inputs[f"state_{i}"], caches, self.cache_rows[i])
        logits = self.head(g, self.final_norm(g, x))
        if self.topk != 1:
            next_ids = ops.random_sample(g, logits, k=self.topk, dim=2)
        else:
            _, next_ids = ops.topk(g, logits, axis=2, k=1)
        out["next_ids"] = ops.squeeze(g, next_ids, [2])
        return out

    def build_post_model_graph(self, model_graph, model_graph_inputs, model_outputs):
        with self.device_scope(model_graph, 0, pipeline_stage_id=model_outputs["stage_offset"]):
            container, step, mask, new_ids = self.step_containers(
                model_graph, model_graph_inputs["input_ids_container"], model_graph_inputs["step"],
                model_graph_inputs["attention_mask"], model_outputs["next_ids"])
            stop_mask, keep_going = self.step_loop_cond(model_graph, new_ids, model_graph_inputs["stop_mask"])
        self.add_output_tensor(model_graph, [keep_going, container, step, mask, stop_mask] +
                               [v for k, v in model_outputs.items() if k.startswith("states/")])
