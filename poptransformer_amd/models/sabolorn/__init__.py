"""Sabolorn decoder: latent attention, attention by heads behind short convolutions and the state-space recurrence, each beside a
feed-forward that may be a mixture of experts; a part of the token's own in every layer; an average over all depths between them.

hf_config: the design's config.json (keys architecture, embedding, layers, logit_softcap, norm, token_side, vocab, width).  Layer i's
tensors start with `l<i>.`; a latent layer with `kv_from` reads another layer's cache; the embedding table is the head.  The model is
recorded one token per loop iteration, as the other decoders are; what a fused executor needs is recorded in constants of the
layers (`l<i>.mixer`, `l<i>.rotation`, `l<i>.experts`).
"""
import numpy as np

from ... import ops
from ...engine.hybrid import Experts
from ...engine.loader import depth_layers
from ...layers import BaseLayer
from ...layers.depth import DepthAverage, SquaredReLU, TokenInput
from ...layers.heads import ExpertMixture, HeadAttention, VisibleKeys, numbers
from ...layers.latent import LatentAttention
from ...layers.parallel import RotaryTable
from ...layers.state_space import StateSpace
from ...layers.streams import WeightNorm, scalar
from ..base_model import HFDecBaseModel
from ..zekilix import softcapped


class Block(BaseLayer):
    """x + mixer(norm1(x)) + ff(norm1(x)), then the token's own part."""

    def __init__(self, context, layer, width, eps, side_dim, max_length, rotation, visible):
        super().__init__(None, context)
        m = layer.mixer
        self.kind = m.kind
        self.norm = WeightNorm(self.context, "norm1", width, eps, centred=True)
        if m.kind == "latent":
            self.mixer = LatentAttention(self.context, "mix", width, eps, max_length, m, rotation)
        elif m.kind == "heads":
            self.mixer = HeadAttention(self.context, "mix", width, eps, m, None, visible)
        else:
            self.mixer = StateSpace(self.context, "mix", width, eps, m)
        self.mlp = None
        if layer.mlp is not None:
            self.mlp = ExpertMixture(self.context, "mlp", width, layer.mlp) if isinstance(layer.mlp, Experts) \
                else SquaredReLU(self.context, "mlp", width, layer.mlp.ff)
        self.side = TokenInput(self.context, "side", width, side_dim, eps)

    def state_shapes(self):
        """Shapes of what the loop carries for this layer (None: nothing)"""
        return [] if self.kind == "latent" else self.mixer.state_shapes()

    def __call__(self, graph, x, e, layer_id, step, attention_mask, state, caches, max_length):
        h = self.norm(graph, x)
        if self.kind == "latent":
            source = self.mixer.mixer.source
            if source is None:
                caches[layer_id] = self.mixer.cache(graph, h, step, max_length)
            y = self.mixer(graph, h, layer_id, step, attention_mask, caches[layer_id if source is None else source])
        elif self.kind == "heads":
            y, state = self.mixer(graph, h, layer_id, step, state)
        else:
            y, state = self.mixer(graph, h, layer_id, state)
        if self.mlp is not None:
            y = ops.add(graph, y, self.mlp(graph, h, layer_id))
        return self.side(graph, ops.add(graph, x, y), e), state


class SabolornDecModel(HFDecBaseModel):
    """Greedy or top-k decoder of the design (precision 'bf16' or 'fp32')."""

    def __init__(self, **kwargs):
        super().__init__(**kwargs)
        c, L = self.hf_config, self.max_length
        if self.precision not in ("bf16", "fp32"):
            raise ValueError(f"Invalid precision {self.precision}, options: ['bf16', 'fp32']")
        self.topk = kwargs.get("topk", 1)
        self.eps, self.side_dim = c.norm["eps"], c.token_side["dim"]
        layers = depth_layers(c.layers)
        self.embed_id = self._table("embed", [c.vocab, c.width])
        self.side_id = self._table("side.embed", [c.vocab, len(layers) * self.side_dim])
        rotations, visible, self.blocks, self.averages = {None: None}, None, [], []
        for i, layer in enumerate(layers):
            m = layer.mixer
            rot = getattr(m, "rot", None)
            key = None if rot is None else tuple(rot.numbers())
            if key not in rotations:
                f, amplitude = rot.frequencies()
                rotations[key] = RotaryTable(f"rotary{len(rotations)}", L, rot.base, rot.dims, rot.neighbours, f, amplitude)
            if m.kind == "heads" and visible is None:
                visible = VisibleKeys("visible", L, L, m)
            self.blocks.append(Block(f"l{i}", layer, c.width, self.eps, self.side_dim, L, rotations[key], visible))
            self.averages.append(DepthAverage(f"l{i}", "dwa", i + 2))
        self.final_norm = WeightNorm(None, "final.norm", c.width, self.eps, centred=True)

    def _table(self, key, shape):
        value = self.state_dict.get(key)
        if value is None or list(value.shape) != shape:
            raise ValueError(f"tensor {key} must be {shape}")
        return self.graph.addInitializedInputTensor(np.asarray(value, np.float32), debugContext=key)

    def _carried(self):
        return [(i, j, shape) for i, b in enumerate(self.blocks) for j, shape in enumerate(b.state_shapes()) if shape is not None]

    def build_model_graph_inputs(self, graph, inputs):
        inputs = super().build_model_graph_inputs(graph, inputs)
        with graph.nameScope("states"):
            for i, j, shape in self._carried():
                inputs[f"state_{i}_{j}"] = ops.constant(self.graph, np.zeros(shape, np.float32), f"layer{i}_{j}")
        return inputs

    def build_model_graph(self, model_graph, model_graph_inputs, sequence_length=1):
        g, c, step = model_graph, self.hf_config, model_graph_inputs["step"]
        shape, n = [self.batch_size, 1, c.width], self.side_dim
        ids = ops.dynamic_slice(g, model_graph_inputs["input_ids_container"], step, axes=[1], sizes=[sequence_length])
        mask = ops.unsqueeze(g, model_graph_inputs["attention_mask"], [1, 2])
        numbers(g, self.eps, "eps")
        scale = (getattr(c, "embedding", None) or {}).get("scale")
        x = ops.mul(g, ops.gather(g, self.embed_id, ids), scalar(g, 1.0 if scale is None else scale, "embedding_scale"))
        x = ops.reshape(g, x, shape)
        side = ops.reshape(g, ops.gather(g, self.side_id, ids), [self.batch_size, 1, len(self.blocks) * n])
        history, caches, states, out = [x], {}, {}, {"stage_offset": 1}
        for i, (block, average) in enumerate(zip(self.blocks, self.averages)):
            state = [model_graph_inputs.get(f"state_{i}_{j}") for j in range(len(block.state_shapes()))]
            e = ops.static_slice(g, side, [i * n], [(i + 1) * n], [2])
            x, states[i] = block(g, x, e, i, step, mask, state, caches, self.max_length)
            history.append(x)
            x = average(g, history)
        logits = ops.matmul(g, self.final_norm(g, x), ops.transpose(g, self.embed_id, [1, 0]))
        if getattr(c, "logit_softcap", None):
            logits = softcapped(g, logits, c.logit_softcap, "logit_softcap")
        if self.topk != 1:
            next_ids = ops.random_sample(g, logits, k=self.topk, dim=2)
        else:
            _, next_ids = ops.topk(g, logits, axis=2, k=1)
        out["next_ids"] = ops.squeeze(g, next_ids, [2])
        for i, j, _ in self._carried():
            out[f"states/layer_{i}_{j}"] = states[i][j]
        return out

    def build_post_model_graph(self, model_graph, model_graph_inputs, model_outputs):
        with self.device_scope(model_graph, 0, pipeline_stage_id=model_outputs["stage_offset"]):
            container, step, mask, new_ids = self.step_containers(
                model_graph, model_graph_inputs["input_ids_container"], model_graph_inputs["step"],
                model_graph_inputs["attention_mask"], model_outputs["next_ids"])
            stop_mask, keep_going = self.step_loop_cond(model_graph, new_ids, model_graph_inputs["stop_mask"])
        self.add_output_tensor(model_graph, [keep_going, container, step, mask, stop_mask] +
                               [v for k, v in model_outputs.items() if k.startswith("states/")])
