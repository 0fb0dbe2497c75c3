"""Executor of decoders whose fp32 residual takes the norms of its sublayers' results,

    x <- x + norm1(mixer(x)),    x <- x + norm2(ff(x)),

with attention by heads and feed-forwards that may be mixtures of experts.  The sublayers read x itself.  Rows, sequences,
sampling and the decode loop are HybridDecoder's.

Launches of a layer in a decode iteration: projections; attention (norms, rotation and cache entry with it, the parts of the
visible keys merged by a second launch); output projection; result norm, which also routes the row; gate / up pair and down
projection of the chosen experts and the shared one (or of the dense feed-forward); result norm.  Passes of many rows work
through the experts' lists of rows, and route in a launch of its own.
"""
from dataclasses import dataclass
from typing import List, Optional

import torch

from .. import _hybrid_lib as H
from .. import hybrid_kernels as HK
from .hybrid import F32, Experts, HybridDecoder


@dataclass
class FeedForwardWeights:
    """Gate, up and down of a feed-forward, or of every expert of a mixture."""
    gate: object                     # WideWeight, or ExpertWeight
    up: object
    down: object

    def linears(self):
        return [self.gate, self.up, self.down]


@dataclass
class ResultNormLayerWeights:
    norm1: torch.Tensor
    proj: HK.WideWeight              # q | k | v (none where the values are the keys) | gate per feature, tail: gates per head
    proj_bias: Optional[torch.Tensor]
    out: HK.WideWeight
    q_norm: torch.Tensor
    k_norm: torch.Tensor
    sink: Optional[torch.Tensor] = None
    lam: float = 0.0                 # weight of the second map
    norm2: Optional[torch.Tensor] = None
    ff: Optional[FeedForwardWeights] = None          # dense, or the routed experts
    shared: Optional[FeedForwardWeights] = None
    router: Optional[torch.Tensor] = None            # [experts (+ the shared one's gate), padded width]
    router_linear: Optional[HK.WideWeight] = None    # the same as a Linear
    top: int = 0

    def active_parameters(self):
        """Parameters of the products that one row goes through."""
        parts = [(w, 1) for w in (self.proj, self.out)] + [(w, max(self.top, 1)) for w in (self.ff.linears() if self.ff else ())]
        parts += [(w, 1) for w in (self.shared.linears() if self.shared else ())]
        return sum(w.n_main * w.K * times for w, times in parts)


@dataclass
class ResultNormWeights:
    embed: torch.Tensor
    layers: List[ResultNormLayerWeights]
    final_norm: torch.Tensor
    head: HK.WideWeight

    def nbytes(self, rows=1):
        """Bytes of the weights that a pass of `rows` rows reads: of a mixture the experts that so many choose on average, where every
        choice is as likely as another."""
        n = self.head.nbytes
        for lw in self.layers:
            n += lw.proj.nbytes + lw.out.nbytes
            for part in (lw.ff, lw.shared):
                if part is not None:
                    n += sum(w.nbytes for w in part.linears())
            if lw.router is not None:
                n += lw.router.numel() * lw.router.element_size()
                count = lw.ff.gate.count
                n += int((count * (1 - (1 - lw.top / count) ** rows) - 1) * sum(w.nbytes for w in lw.ff.linears()))
        return n


class ResultNormBuffers:
    """Activations of up to `rows` rows."""

    def __init__(self, spec, weights, rows, direct, dtype, device):
        def buf(*shape, dtype=dtype):
            return torch.zeros(shape, dtype=dtype, device=device)
        self.rows = rows
        self.x = buf(rows, spec.width, dtype=F32)
        self.h = buf(rows, HK.pad8(spec.width))
        self.y = buf(rows, spec.width, dtype=F32)
        self.proj = {n: buf(rows, n) for n in {lw.proj.n_main for lw in weights.layers}}
        self.head_gates = {n: buf(rows, n, dtype=F32) for n in {lw.proj.tail for lw in weights.layers} if n}
        self.ctx = {n: buf(rows, n) for n in {lay.mixer.out_channels for lay in spec.layers}}
        self.act, self.parts, self.routing, self.lists, self.logits = {}, {}, {}, {}, {}
        for lay, lw in zip(spec.layers, weights.layers):
            e = lay.mlp
            if not isinstance(e, Experts):
                if e is not None:
                    self.act[lw.ff.gate.n_main] = buf(rows, lw.ff.gate.n_main)
                continue
            key, choices = (e.count, e.top, e.shared is not None, e.scale), e.top + (e.shared is not None)
            if key not in self.routing:
                self.routing[key] = HK.Routing(rows, e.count, e.top, e.shared is not None, e.scale, device)
            n = lw.ff.gate.n_main
            if lw.shared is not None:
                self.act[lw.shared.gate.n_main] = buf(rows, lw.shared.gate.n_main)
                n = max(n, lw.shared.gate.n_main) if direct else n
            if (choices, n) not in self.act:
                self.act[choices, n] = buf(rows * choices, n)
            if choices not in self.parts:
                self.parts[choices] = buf(rows * choices, spec.width, dtype=F32 if direct else dtype)
            if dtype == F32:
                self.logits[lw.router.shape[0]] = buf(rows, lw.router.shape[0], dtype=F32)
            if not direct:
                for t in (128, 256):
                    self.lists[e.count, e.top, t] = HK.expert_lists(rows, e.top, e.count, t, device)
        channels = max([spec.width] + [lw.proj.N for lw in weights.layers])
        self.workspace = HK.linear_workspace(rows, channels, device) if rows > 16 else None


class ResultNormDecoder(HybridDecoder):
    direct_rows = 16                 # passes of up to this many bf16 rows find their experts' rows without lists
    # routers up to this size are multiplied in the norm's launch by passes of up to so many rows (every row reads all of it: 2048
    # rows of 4096 features and 33 logits take 43 us that way, 19 + 21 with a launch for the routing, 512 rows 16 against 10 + 15)
    router_bytes, router_rows = 1 << 20, 512
    tall_rows = 128                  # rows per expert, on average, above which their lists are cut into tiles of 256 (else 128)

    def __init__(self, spec, weights, device="cuda", slots=None):
        super().__init__(spec, weights, device, slots)
        self._angles = {}

    def _direct(self, rows):
        return self.dtype == torch.bfloat16 and rows <= self.direct_rows

    def _rows_buffers(self, rows):
        size = rows if rows <= 16 else max(64, 1 << (rows - 1).bit_length())
        if size not in self._buffers:
            self._buffers[size] = ResultNormBuffers(self.spec, self.w, size, self._direct(size), self.dtype, self.dev)
        return self._buffers[size]

    def _cos_sin(self, rot):
        if rot is None:
            return None
        key = (rot.base, rot.dims, rot.neighbours, rot.factor, rot.yarn)
        if key not in self._angles:
            self._angles[key] = torch.from_numpy(rot.angles(self.store.max_len)).to(self.dev)
        return self._angles[key]

    def _splits(self, rows, mixer):
        """Parts of the visible keys per (row, key head) of a decode pass, and the scratch they meet in: as HybridDecoder's."""
        m = mixer
        key = (rows, m.heads, m.kv_heads, m.stored_dim, m.stored_vdim, m.maps, m.keep, m.span)
        if key not in self._splits_for:
            group, most = m.heads // m.kv_heads, 4 // m.maps
            wgs = rows * m.kv_heads * -(-group // (group if group <= 2 // m.maps else most))
            keys = min(m.keep + m.span, self.store.max_len)
            splits = max(1, min(768 // wgs, -(-keys // 64), 64)) if keys > 256 else 1
            self._splits_for[key] = (splits, HK.head_workspace(rows, m, splits, self.dev) if splits > 1 else None)
        return self._splits_for[key]

    def _mixer(self, i, b, rows):
        spec, m, lw, n = self.spec, self.spec.layers[i].mixer, self.w.layers[i], rows.n
        proj, ctx, gates = b.proj[lw.proj.n_main], b.ctx[m.out_channels], b.head_gates[lw.proj.tail] if lw.proj.tail else None
        HK.linear(b.h, lw.proj, proj, n, tail=gates, bias=lw.proj_bias, workspace=b.workspace)
        att = HK.HeadAttention(m, spec.eps, lw.q_norm, lw.k_norm, self._cos_sin(m.rot), lw.sink, lw.lam, *self.store.stores[i], proj, n,
                               rows.slot, rows.pos, gates, ctx)
        if rows.single:
            att.decode(*self._splits(n, m))
        else:
            att.prompt(rows.tiles)
        HK.linear(ctx, lw.out, b.y, n, ld=spec.width, workspace=b.workspace)

    def _routing(self, i, b):
        e = self.spec.layers[i].mlp
        return b.routing[e.count, e.top, e.shared is not None, e.scale]

    def _routed_by_norm(self, i, b):
        """What the norm's launch needs to route the rows to layer i's experts, where it does."""
        lw = self.w.layers[i]
        if lw.router is None or b.rows > self.router_rows or lw.router.numel() * lw.router.element_size() > self.router_bytes:
            return {}
        return dict(router=lw.router, routing=self._routing(i, b))

    def _feed_forward(self, i, b, n):
        """The feed-forward's result, as arguments of result_norm."""
        spec, mlp, lw = self.spec, self.spec.layers[i].mlp, self.w.layers[i]
        if not isinstance(mlp, Experts):
            self._dense(b, n, lw.ff, pair=H.PAIR_SWIGLU)
            return dict(y=b.y)
        r = self._routing(i, b)
        if not self._routed_by_norm(i, b):
            if self.dtype == torch.bfloat16:
                r.by_product(b.h, lw.router_linear, n)
            else:
                logits = b.logits[lw.router.shape[0]]
                HK.linear(b.h, lw.router_linear, logits, n)
                r(logits, n)

        def clamped(glu):
            return dict(pair=H.PAIR_CLAMPED, limit=glu.limit, slope=glu.slope)
        parts = b.parts[r.choices]
        result = dict(parts=parts, parts_ld=r.choices, part_weight=r.weights)
        pair, down = dict(w=lw.ff.gate, up=lw.ff.up, **clamped(mlp.expert)), dict(w=lw.ff.down)
        if self._direct(b.rows):
            shared_pair = shared_down = None
            act_ld = lw.ff.gate.n_main
            if mlp.shared is not None:
                shared_pair, shared_down = dict(w=lw.shared.gate, up=lw.shared.up, **clamped(mlp.shared)), dict(w=lw.shared.down)
                act_ld = max(act_ld, lw.shared.gate.n_main)
            act = b.act[r.choices, act_ld]
            HK.experts(b.h, r, n, pair, act, shared_pair)
            HK.experts(act, r, n, down, parts, shared_down)
            return dict(result, n_parts=r.choices)
        tile = 256 if n * mlp.top > self.tall_rows * mlp.count else 128
        lists, act = b.lists[mlp.count, mlp.top, tile], b.act[r.choices, lw.ff.gate.n_main]
        HK.group_experts(r, n, tile, lists)
        HK.experts(b.h, r, n, pair, act, lists=lists, tile_rows=tile)
        HK.experts(act, r, n, down, parts, lists=lists, tile_rows=tile)
        result.update(n_parts=mlp.top)
        if mlp.shared is not None:
            self._dense(b, n, lw.shared, **clamped(mlp.shared))
            result.update(y=b.y, y_weight=(r.weights, mlp.top))
        return result

    def _dense(self, b, n, ff, **pair):
        act = b.act[ff.gate.n_main]
        HK.linear(b.h, ff.gate, act, n, up=ff.up, **pair)
        HK.linear(act, ff.down, b.y, n, ld=self.spec.width, workspace=b.workspace)

    def _layers(self, rows, pos_out=None):
        """All layers over the rows; h holds the model's norm of them."""
        spec, w, n = self.spec, self.w, rows.n
        b = self._rows_buffers(n)
        common = dict(x=b.x, rows=n, eps=spec.eps, h=b.h)
        HK.result_norm(table=w.embed, embed_scale=spec.embed_scale, ids=rows.ids, ids_index=rows.ids_index, pos_out=pos_out, **common)
        for i, layer in enumerate(spec.layers):
            lw, ff = w.layers[i], layer.mlp is not None
            last = dict(final_weight=w.final_norm) if i == len(spec.layers) - 1 else {}
            self._mixer(i, b, rows)
            HK.result_norm(y=b.y, weight=lw.norm1, **(self._routed_by_norm(i, b) if ff else last), **common)
            if ff:
                HK.result_norm(weight=lw.norm2, **self._feed_forward(i, b, n), **last, **common)
            if self.probe is not None:
                self.probe(i, b.x[:n].clone())
        return b, None

    def _logits(self, b, done, count, out, gather=None):
        h = b.h
        if gather is not None:
            if self._head_h is None:
                self._head_h = torch.zeros((self.head_rows, h.shape[1]), dtype=self.dtype, device=self.dev)
            h = self._head_h
            torch.index_select(b.h, 0, gather, out=h[:count])
        HK.linear(h, self.w.head, out, count, ld=self.spec.vocab)
