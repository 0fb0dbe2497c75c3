"""Golapel decoder: three kinds of attention by heads (a window that keeps the first tokens, with sinks; differential within
chunks; within chunks with stretched rotation), feed-forwards that may be mixtures of experts, and a residual that takes the
RMS norms of the sublayers' results.

hf_config: the design's config.json (keys architecture, embedding, layers, norm, vocab, width).  Layer i's tensors start with
`l<i>.`; the embedding table is the head.  The model is recorded one token per loop iteration, as the other decoders are; what a
fused executor needs is recorded in constants of the layers (`l<i>.mixer`, `l<i>.rotation`, `l<i>.experts`).
"""
import numpy as np

from ... import ops
from ...engine.hybrid import Experts
from ...engine.loader import head_layers
from ...layers import BaseLayer
from ...layers.heads import ExpertMixture, HeadAttention, SwiGLU, VisibleKeys, numbers
from ...layers.parallel import RotaryTable
from ...layers.streams import WeightNorm, scalar
from ..base_model import HFDecBaseModel


class Block(BaseLayer):
    """x + norm1(mixer(x)), then x + norm2(ff(x))."""

    def __init__(self, context, layer, width, eps, rotation, visible):
        super().__init__(None, context)
        self.mixer = HeadAttention(self.context, "mix", width, eps, layer.mixer, rotation, visible)
        self.norm1 = WeightNorm(self.context, "norm1", width, eps, centred=False)
        self.mlp = None
        if layer.mlp is not None:
            self.norm2 = WeightNorm(self.context, "norm2", width, eps, centred=False)
            self.mlp = ExpertMixture(self.context, "mlp", width, layer.mlp) if isinstance(layer.mlp, Experts) \
                else SwiGLU(self.context, "mlp", width, layer.mlp.ff)

    def __call__(self, graph, x, layer_id, step):
        x = ops.add(graph, x, self.norm1(graph, self.mixer(graph, x, layer_id, step)))
        if self.mlp is not None:
            x = ops.add(graph, x, self.norm2(graph, self.mlp(graph, x, layer_id)))
        return x


class GolapelDecModel(HFDecBaseModel):
    """Greedy or top-k decoder of the design (precision 'bf16' or 'fp32')."""

    def __init__(self, **kwargs):
        super().__init__(**kwargs)
        c, L = self.hf_config, self.max_length
        if self.precision not in ("bf16", "fp32"):
            raise ValueError(f"Invalid precision {self.precision}, options: ['bf16', 'fp32']")
        self.topk = kwargs.get("topk", 1)
        eps = c.norm["eps"]
        value = self.state_dict.get("embed")
        if value is None or list(value.shape) != [c.vocab, c.width]:
            raise ValueError(f"tensor embed must be {[c.vocab, c.width]}")
        self.embed_id = self.graph.addInitializedInputTensor(np.asarray(value, np.float32), debugContext="embed")
        rotations, tables, self.blocks = {None: None}, {}, []
        for i, layer in enumerate(head_layers(c.layers)):
            m, rot = layer.mixer, layer.mixer.rot
            key = None if rot is None else tuple(rot.numbers())
            if key not in rotations:
                f, amplitude = rot.frequencies()
                rotations[key] = RotaryTable(f"rotary{len(rotations)}", L, rot.base, rot.dims, rot.neighbours, f, amplitude)
            rows = L if m.keep else min(m.span, L)                     # what slides out of sight is dropped
            seen = (m.window, m.keep, m.chunk)
            if seen not in tables:
                tables[seen] = VisibleKeys(f"visible{len(tables)}", L, rows, m)
            self.blocks.append(Block(f"l{i}", layer, c.width, eps, rotations[key], tables[seen]))
        self.final_norm = WeightNorm(None, "final.norm", c.width, eps, centred=False)

    def build_model_graph(self, model_graph, model_graph_inputs, sequence_length=1):
        g, c, step = model_graph, self.hf_config, model_graph_inputs["step"]
        ids = ops.dynamic_slice(g, model_graph_inputs["input_ids_container"], step, axes=[1], sizes=[sequence_length])
        numbers(g, c.norm["eps"], "eps")
        x = ops.mul(g, ops.gather(g, self.embed_id, ids), scalar(g, c.embedding["scale"], "embedding_scale"))
        x = ops.reshape(g, x, [self.batch_size, 1, c.width])
        for i, block in enumerate(self.blocks):
            x = block(g, x, i, step)
        logits = ops.matmul(g, self.final_norm(g, x), ops.transpose(g, self.embed_id, [1, 0]))
        if self.topk != 1:
            next_ids = ops.random_sample(g, logits, k=self.topk, dim=2)
        else:
            _, next_ids = ops.topk(g, logits, axis=2, k=1)
        return {"next_ids": ops.squeeze(g, next_ids, [2]), "stage_offset": 1}
