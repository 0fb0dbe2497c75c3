"""Attention whose cache holds one latent and one shared rotated key part per token.

Recorded in FLOAT, as `streams` is."""
from .. import ops
from .base_layer import BaseLayer
from .heads import numbers
from .streams import NamedLinear, WeightNorm, scalar


class LatentAttention(BaseLayer):
    """Attention over the newest `window` positions with keys and values made from a cached latent and one rotated key part
    that the heads share (a LatentMixer); queries through a latent of their own, a sigmoid gate per head or per feature.  Tensors
    `<context>.dq`, `.dq.norm`, `.uq`, `.dkv`, `.dkv.norm` (of a layer with a cache of its own), `.uk`, `.uv`, `.g`, `.o`."""

    def __init__(self, context, name, width, eps, max_length, mixer, rotation):
        super().__init__(context, name)
        m = self.mixer = mixer
        self.rotation = rotation
        self.rows = min(m.window or max_length, max_length)
        self.dq = NamedLinear(self.context, "dq", width, m.q_rank)
        self.q_norm = WeightNorm(self.context, "dq.norm", m.q_rank, eps, centred=False)
        self.uq = NamedLinear(self.context, "uq", m.q_rank, m.heads * (m.dim + m.rot_dim))
        if m.source is None:
            self.dkv = NamedLinear(self.context, "dkv", width, m.kv_rank + m.rot_dim)
            self.kv_norm = WeightNorm(self.context, "dkv.norm", m.kv_rank, eps, centred=False)
        self.uk, self.uv = (NamedLinear(self.context, n, m.kv_rank, m.heads * c) for n, c in (("uk", m.dim), ("uv", m.vdim)))
        self.g = NamedLinear(self.context, "g", width, m.heads * (m.vdim if m.gate == "feature" else 1))
        self.o = NamedLinear(self.context, "o", m.heads * m.vdim, width)

    def cache(self, graph, h, step, rows):
        """The newest `rows` cache entries [B, rows, kv_rank + rot_dim], newest first."""
        B, R, P = self.batch_size, self.mixer.kv_rank, self.mixer.rot_dim
        with graph.nameScope(self.context):
            c, k = ops.split(graph, self.dkv(graph, h), 2, axis=2, splits=[R, P], name="split_latent")
            entry = ops.concat(graph, self.kv_norm(graph, c), self.rotation(graph, k, step, P), 2)
            past = ops.kv_cache(graph, step, ops.reshape(graph, entry, [B, 1, 1, R + P]), rows, 2, 1)
            return ops.reshape(graph, past, [B, rows, R + P])

    def __call__(self, graph, h, layer_id, step, attention_mask, cache):
        m, B, W = self.mixer, self.batch_size, self.rows
        H, D, P, E, R = m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank
        with graph.nameScope(self.context):
            numbers(graph, m.numbers(), f"l{layer_id}.mixer")
            numbers(graph, m.rot.numbers(), f"l{layer_id}.rotation")
            q = self.uq(graph, self.q_norm(graph, self.dq(graph, h)))
            q, q_rot = ops.split(graph, ops.reshape(graph, q, [B, H, D + P]), 2, axis=2, splits=[D, P], name="split_query")
            q = ops.concat(graph, q, self.rotation(graph, q_rot, step, P), 2)
            past = ops.static_slice(graph, cache, [0], [W], [1])
            c, k_rot = ops.split(graph, past, 2, axis=2, splits=[R, P], name="split_cache")
            k = ops.transpose(graph, ops.reshape(graph, self.uk(graph, c), [B, W, H, D]), [0, 2, 3, 1])
            k_rot = ops.tile(graph, ops.transpose(graph, ops.reshape(graph, k_rot, [B, W, 1, P]), [0, 2, 3, 1]), [1, H, 1, 1])
            v = ops.transpose(graph, ops.reshape(graph, self.uv(graph, c), [B, W, H, E]), [0, 2, 1, 3])
            s = ops.matmul(graph, ops.reshape(graph, q, [B, H, 1, D + P]), ops.concat(graph, k, k_rot, 2))
            s = ops.mul(graph, s, scalar(graph, m.scale, "score_scale"))
            s = ops.add(graph, s, ops.static_slice(graph, attention_mask, [0], [W], [3]))
            o = ops.matmul(graph, ops.softmax_ce(graph, s, -1, stable_mode=True), v)
            gate = ops.reshape(graph, ops.sigmoid(graph, self.g(graph, h)), [B, H, 1, E if m.gate == "feature" else 1])
            return self.o(graph, ops.reshape(graph, ops.mul(graph, o, gate), [B, 1, H * E]))
