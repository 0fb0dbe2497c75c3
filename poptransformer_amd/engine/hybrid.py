"""Executor of decoders that mix windowed attention with recurrent (matrix memory) layers over fp32 residual streams; the
mixers, feed-forwards and the row handling that `parallel` uses for layers whose sublayers stand side by side, `result_norm`
for layers whose residual takes the norms of their sublayers' results, and `depth` for layers whose results are averaged over
the depths.  The mixers that several of them run are in `mixers`.

The model is a list of layers, each described by its mixer, its feed-forward (or none) and the layer whose tensors it
uses.  One forward function serves everything: it takes the ROWS of a pass (row = one token of the sequence in a slot, at
a position) through all layers.  A decode iteration is a pass with one row per sequence and depends on device state only
(it is recorded into a HIP graph); a prompt, or a batch of prompts of unequal lengths, is cut into passes of up to
`pass_rows` rows.  Both leave the same cache and state behind.

Per layer with a feed-forward the launches of a decode iteration are: projections, mixer (attention, with the parts of its
window merged by a second launch; or recurrence and head norm), output projection, stream update + norm, gate / up pair,
down projection, stream update + norm.
"""
import math
from dataclasses import dataclass
from typing import List, Optional

import numpy as np
import torch

from .. import _hybrid_lib as H
from .. import hybrid_kernels as HK
from .fused import NextToken
from .loop import DecodeLoop
from .sequences import SequenceStore

F32, I32 = torch.float32, torch.int32


@dataclass
class WindowMixer:
    """Attention over the last `window` positions (None: all), key heads shared by groups of query heads, values that are
    the raw keys, a distance bias of slope_h per position, and an output gate."""
    heads: int
    kv_heads: int
    dim: int
    scale: float
    window: Optional[int]
    kind = "attention"

    @property
    def out_channels(self):
        return self.heads * self.dim

    @property
    def gate_at(self):
        return (self.heads + self.kv_heads) * self.dim

    def slopes(self):
        return 2.0 ** (-8.0 * (np.arange(self.heads) + 1) / self.heads)


@dataclass
class MemoryMixer:
    """mLSTM: a matrix memory of dim x vdim per head."""
    heads: int
    dim: int
    vdim: int
    gate_cap: float
    kind = "mlstm"

    @property
    def out_channels(self):
        return self.heads * self.vdim

    @property
    def gate_at(self):
        return self.heads * (2 * self.dim + self.vdim)


@dataclass
class LatentMixer:
    """Attention over the last `window` positions (None: all) whose keys and values are made from a cached latent of kv_rank
    and one key part shared by the heads, which `rot` turns (its first features, the rest of it passes as it is); queries through a
    latent of q_rank, one output gate per "head" or "feature".  `source`: the layer whose cache is read (None: the layer's own)."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    window: Optional[int]
    rot: "Rotation"
    source: Optional[int] = None
    gate: str = "head"
    kind = "latent"

    @property
    def sizes(self):
        """(heads, D, P, E, R, q_rank, kv_rank) with the head sizes as they are stored."""
        return (self.heads, HK.pad32(self.dim), HK.pad32(self.rot_dim), (self.vdim + 15) // 16 * 16, HK.pad32(self.kv_rank),
                self.q_rank, self.kv_rank)

    @property
    def out_channels(self):
        return self.heads * self.sizes[3]

    @property
    def cache_row(self):
        return self.sizes[4] + self.sizes[2]

    def pairs(self):
        """Order of the rotated features in which the two of a pair follow each other."""
        return self.rot.pairs(self.rot_dim)

    def angles(self, positions):
        """[positions, P / 2, (cos, sin)] of those pairs."""
        return self.rot.angles(positions, HK.pad32(self.rot_dim) // 2)

    def numbers(self):
        """What the tensors' shapes do not tell but the rotation, as a flat list, which `LatentMixer.of` reads."""
        return [self.heads, self.scale, self.window or 0, -1 if self.source is None else self.source, ("head", "feature").index(self.gate)]

    @staticmethod
    def of(numbers, dim, rot_dim, vdim, q_rank, kv_rank, rot):
        heads, scale, window, source, gate = (float(v) for v in numbers)
        return LatentMixer(int(heads), dim, rot_dim, vdim, q_rank, kv_rank, scale, int(window) or None, rot, int(source) if source >= 0 else None,
                           ("head", "feature")[int(gate)])


@dataclass
class Rotation:
    """Rotary positions on the first `dims` features of a head, in pairs (i, i + dims / 2) or (`neighbours`) (2 i, 2 i + 1).  The
    frequencies base^(-2 i / dims) are divided by `factor`; with yarn = (original, fast, slow) only those that make fewer than
    `slow` turns in `original` positions, those of more than `fast` turns not at all, with a ramp in between."""
    base: float
    dims: int
    neighbours: bool = False
    factor: float = 1.0
    yarn: Optional[tuple] = None

    def frequencies(self):
        """(frequencies, factor of cos and sin)"""
        i = np.arange(self.dims // 2)
        f = float(self.base) ** (-2.0 * i / self.dims)
        if self.yarn is None:
            return f / self.factor, 1.0
        original, fast, slow = self.yarn

        def feature(turns):
            return self.dims * math.log(original / (2 * math.pi * turns)) / (2 * math.log(self.base))
        low, high = max(math.floor(feature(fast)), 0), min(math.ceil(feature(slow)), self.dims - 1)
        slowed = np.clip((i - low) / max(high - low, 0.001), 0.0, 1.0)
        return f * (slowed / self.factor + (1.0 - slowed)), 0.1 * math.log(self.factor) + 1.0

    def numbers(self):
        """The fields as a flat list, which `Rotation.of` reads."""
        return [self.base, self.dims, self.neighbours, self.factor, *(self.yarn or ())]

    @staticmethod
    def of(numbers):
        base, dims, neighbours, factor, *yarn = (float(v) for v in numbers)
        return Rotation(base, int(dims), bool(neighbours), factor, tuple(yarn) or None)

    def pairs(self, size):
        """Order of `size` features in which the two of a pair follow each other."""
        turned = np.arange(self.dims)
        if not self.neighbours:
            turned = turned.reshape(2, -1).T.reshape(-1)
        return np.concatenate([turned, np.arange(self.dims, size)])

    def angles(self, positions, pairs=None):
        """fp32 [positions, pairs, (cos, sin)] of those pairs, by default of whole pieces of eight features; the ones past `dims` stay
        as they are."""
        f, amplitude = self.frequencies()
        a = np.arange(positions)[:, None] * f
        out = np.zeros((positions, HK.pad8(self.dims) // 2 if pairs is None else pairs, 2), np.float32)
        out[..., 0] = 1.0
        out[:, :len(f), 0], out[:, :len(f), 1] = np.cos(a) * amplitude, np.sin(a) * amplitude
        return out


@dataclass
class HeadMixer:
    """Attention over cached keys and values of kv_heads heads: norms of queries and keys per head, rotation, and what is set of
    the rest.  Visible are the newest `window` positions (None: all) with the first `keep`, or those of the same `chunk`."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[Rotation] = None
    window: Optional[int] = None
    keep: int = 0
    chunk: Optional[int] = None
    keys_are_values: bool = False    # the values are the keys as projected
    biases: str = ""                 # which of "qkv" have biases
    sink: bool = False               # a learned score per head in the softmax's denominator
    gate: Optional[str] = None       # sigmoid gate of the result, one number per "head" or per "feature"
    diff: Optional[float] = None     # two maps per head, the second subtracted; part of their weight, and 1 - diff of the result
    norms: bool = True               # RMS norms of queries and keys, per head
    far: bool = False                # far1 ln(1 + far2 distance) is taken off the scores, with two numbers per head
    taps: int = 0                    # queries, keys and values pass a short convolution over so many tokens (0: none)
    kind = "heads"

    def numbers(self):
        """Everything but the feature sizes, the biases and the rotation as a flat list, which `HeadMixer.of` reads."""
        return [self.heads, self.kv_heads, self.scale, self.window or 0, self.keep, self.chunk or 0, self.keys_are_values, self.sink,
                (None, "head", "feature").index(self.gate), self.norms, self.far, self.taps, *(() if self.diff is None else (self.diff,))]

    @staticmethod
    def of(numbers, dim, vdim, biases, rot):
        heads, kv_heads, scale, window, keep, chunk, keys_are_values, sink, gate, norms, far, taps, *diff = (float(v) for v in numbers)
        return HeadMixer(int(heads), int(kv_heads), dim, vdim, scale, rot, int(window) or None, int(keep), int(chunk) or None,
                         bool(keys_are_values), biases, bool(sink), (None, "head", "feature")[int(gate)], diff[0] if diff else None, bool(norms),
                         bool(far), int(taps))

    def visible(self, positions):
        """bool [position of the query, distance back to the key]."""
        i, back = np.arange(positions)[:, None], np.arange(positions)[None]
        j = i - back
        near = j >= 0
        if self.window is not None:
            near &= (back < self.window) | (j < self.keep)
        if self.chunk is not None:
            near &= i // self.chunk == j // self.chunk
        return near

    @property
    def maps(self):
        return 1 if self.diff is None else 2

    @property
    def stored_dim(self):
        return HK.pad8(self.dim)

    @property
    def stored_vdim(self):
        return HK.pad8(self.vdim)

    @property
    def conv_channels(self):
        """Channels of the convolution: queries, keys and values, as stored."""
        return (self.heads + self.kv_heads) * self.maps * self.stored_dim + self.kv_heads * self.stored_vdim

    @property
    def span(self):
        """Most positions, besides the kept ones, that one sees."""
        return min(self.window or 1 << 30, self.chunk or 1 << 30)

    @property
    def out_channels(self):
        return self.heads * self.stored_vdim


@dataclass
class StateSpaceMixer:
    """Mamba-2: a state of dim x vdim per head, keys and queries (b and c) shared by the heads of a group; x, b and c pass a short
    convolution over `taps` tokens with silu; the result times silu of a gate, normed in norm_parts equal parts."""
    heads: int
    groups: int
    dim: int
    vdim: int
    taps: int
    norm_parts: int
    kind = "ssd"

    def numbers(self):
        """The fields as a flat list, which `StateSpaceMixer.of` reads."""
        return [self.heads, self.groups, self.dim, self.vdim, self.taps, self.norm_parts]

    @staticmethod
    def of(numbers):
        return StateSpaceMixer(*(int(v) for v in numbers))

    @property
    def stored_dim(self):
        return HK.pad8(self.dim)

    @property
    def stored_vdim(self):
        return HK.pad8(self.vdim)

    @property
    def out_channels(self):
        return self.heads * self.stored_vdim

    @property
    def conv_channels(self):
        return self.out_channels + 2 * self.groups * self.stored_dim


@dataclass
class SquaredReLU:
    """relu(u)^2 between the up and the down projection."""
    ff: int


@dataclass
class SwiGLU:
    """silu(g) u between the gate / up pair and the down projection."""
    ff: int


@dataclass
class BiasedSwiGLU:
    """silu(g) u between the gate / up pair and the down projection, all three with biases."""
    ff: int


@dataclass
class ClampedGLU:
    """min(g, limit) sigmoid(slope g) (clamp(u, -limit, limit) + 1) between the gate / up pair and the down projection."""
    ff: int
    limit: float
    slope: float = 1.702


@dataclass
class Experts:
    """Mixture of experts: of `count` feed-forwards every token has the `top` with the largest router scores, weighted by
    score * scale; `shared` runs for every token, weighted by a sigmoid of its own.  Scores are the router's "softmax" or "sigmoid";
    sigmoid scores may be `corrected` for the choice, and experts be chosen from the `keep` best of equal `groups` of neighbours only."""
    count: int
    top: int
    scale: float
    expert: object                   # ClampedGLU or SwiGLU
    shared: Optional[ClampedGLU] = None
    score: str = "softmax"
    corrected: bool = False
    groups: int = 1
    keep: int = 1
    share: bool = False              # weights are shares of the chosen scores' sum

    @property
    def routing_key(self):
        return self.count, self.top, self.shared is not None, self.scale, self.score, self.groups, self.keep, self.share

    def numbers(self):
        """Everything but the feed-forwards as a flat list, which `Experts.of` reads."""
        return [self.count, self.top, self.scale, ("softmax", "sigmoid").index(self.score), self.corrected, self.groups, self.keep, self.share]

    @staticmethod
    def of(numbers, expert, shared=None):
        count, top, scale, score, corrected, groups, keep, share = (float(v) for v in numbers)
        return Experts(int(count), int(top), scale, expert, shared, ("softmax", "sigmoid")[int(score)], bool(corrected), int(groups), int(keep),
                       bool(share))


@dataclass
class HybridLayer:
    mixer: object
    mlp: object                      # or None
    source: int                      # the layer whose tensors this one uses (itself, or an earlier one)
    shift: bool = False              # parallel layers: the mixer reads a mixture with the token before


@dataclass
class HybridSpec:
    family: str
    layers: List[HybridLayer]
    width: int
    vocab: int
    streams: int
    eps: float
    residual_mult: float
    embed_scale: float
    logit_cap: float                 # 0: none
    max_len: int
    batch: int
    pad_id: int = 0
    eos_id: int = -1
    early_stop: bool = False
    topk: int = 1
    dtype: str = "bfloat16"          # or float32: everything in true 32-bit
    norm_groups: int = 1             # parallel layers: equal parts of the width with a norm of their own
    positions: Optional[int] = None  # parallel layers: rows of the position table
    side_dim: int = 0                # depth-averaged layers: features of the token's own part of every layer


@dataclass
class HybridLayerWeights:
    norm1: torch.Tensor
    connect1: tuple                  # (in [S], out [S], mix [S, S] from -> to), fp32
    proj: HK.WideWeight              # attention: q | k | gate; mlstm: q | k | v | gate, tail: input and forget gates
    out: HK.WideWeight
    q_norm: Optional[torch.Tensor] = None
    k_norm: Optional[torch.Tensor] = None
    slopes: Optional[torch.Tensor] = None
    head_norm: Optional[torch.Tensor] = None
    norm2: Optional[torch.Tensor] = None
    connect2: Optional[tuple] = None
    gate: Optional[HK.WideWeight] = None
    up: Optional[HK.WideWeight] = None
    down: Optional[HK.WideWeight] = None

    def linears(self):
        return [w for w in (self.proj, self.out, self.gate, self.up, self.down) if w is not None]


@dataclass
class HybridWeights:
    embed: torch.Tensor
    layers: List[Optional[HybridLayerWeights]]      # None where a layer uses another one's
    final_norm: torch.Tensor
    head: HK.WideWeight

    def nbytes(self):
        """Bytes of the weights, each counted once (a layer that uses another one's reads them again)."""
        return self.head.nbytes + sum(w.nbytes for lay in self.layers if lay is not None for w in lay.linears())


class RowBuffers:
    """Activations of up to `rows` rows."""

    def __init__(self, spec, weights, rows, dtype, device):
        def buf(*shape, dtype=dtype):
            return torch.zeros(shape, dtype=dtype, device=device)
        mixers = [lay.mixer for lay in spec.layers]
        self.rows = rows
        self.streams = buf(rows, spec.streams, spec.width, dtype=F32)
        self.h = buf(rows, HK.pad8(spec.width))
        self.y = buf(rows, spec.width, dtype=F32)
        self.ctx = {n: buf(rows, n) for n in {HK.pad8(m.out_channels) for m in mixers}}
        used = [lw for lw in weights.layers if lw is not None]
        self.proj = {n: buf(rows, n) for n in {HK.pad8(lw.proj.n_main) for lw in used}}
        self.act = {n: buf(rows, n) for n in {lw.gate.n_main for lw in used if lw.gate is not None}}
        memory = [m for m in mixers if m.kind == "mlstm"]
        self.gates = buf(rows * 2 * max((m.heads for m in memory), default=0), dtype=F32)
        self.o = buf(rows * max((m.out_channels for m in memory), default=0), dtype=F32)
        self.q_scale = buf(rows, dtype=F32)
        self.workspace = HK.linear_workspace(rows, max((lw.out.N for lw in used), default=1), device) if rows > 16 else None


@dataclass
class Rows:
    """The rows of one pass, as device tensors: slot and position of every row; the sequences (first row, rows); the tiles
    the attention works on (first row, rows).  `single`: one row per sequence."""
    n: int
    slot: torch.Tensor
    pos: torch.Tensor
    seqs: tuple
    single: bool
    tiles: tuple = ()
    ids: Optional[torch.Tensor] = None
    ids_index: Optional[torch.Tensor] = None
    longest: int = 1
    last: Optional[torch.Tensor] = None      # of a sequence's first row: its last one, else -1 (None: one row each)
    portions: tuple = ()                     # (slot, position of the first row, rows) on the host


class HybridDecoder(DecodeLoop):
    """Two ways in, one set of layers, caches and kernels behind both:
      * the decode loop of the other executors (reset / run_steps / consume_prompt / run): `spec.batch` sequences in step;
      * `open` / `advance` / `close`: sequences that come, bring their next tokens in batches of any lengths, and go."""

    pass_rows = 2048                 # rows of a pass, at most
    head_rows = 256                  # rows whose logits are made at once

    def __init__(self, spec, weights, device="cuda", slots=None):
        self.spec, self.w, self.dev = spec, weights, device
        self.dtype = HK.DTYPES[spec.dtype]
        self.store = SequenceStore(spec, self.dtype, slots or max(spec.batch, 1), min(spec.max_len, spec.positions or spec.max_len),
                                   self.pass_rows, device)
        self.probe = None            # callable(layer index, fp32 [rows, width]): the summed streams after every layer
        self._buffers = {}
        self._stream = torch.cuda.Stream()
        self._splits_for = {}
        self._head_h = self._scratch_buf = None

    # ------------------------------------------------------------------ layers
    def _layer_weights(self, i):
        return self.w.layers[self.spec.layers[i].source]

    def _rows_buffers(self, rows):
        size = rows if rows <= 16 else max(64, 1 << (rows - 1).bit_length())
        if size not in self._buffers:
            self._buffers[size] = RowBuffers(self.spec, self.w, size, self.dtype, self.dev)
        return self._buffers[size]

    def _splits(self, rows, mixer):
        """Parts of the window per (row, key head) of a decode pass, and the scratch they meet in.  Fixed per shape (the
        launch is replayed while the context grows): enough workgroups to fill the machine, at least 64 keys per part."""
        key = (rows, mixer.heads, mixer.kv_heads, mixer.dim, mixer.window)
        if key not in self._splits_for:
            group = mixer.heads // mixer.kv_heads
            wgs = rows * mixer.kv_heads * -(-group // (group if group <= 2 else 4))
            keys = min(mixer.window or self.store.max_len, self.store.max_len)
            splits = max(1, min(768 // wgs, -(-keys // 64), 64)) if keys > 256 else 1
            self._splits_for[key] = (splits, HK.window_workspace(rows, mixer.heads, mixer.dim, splits, self.dev) if splits > 1 else None)
        return self._splits_for[key]

    def _scratch(self, nbytes):
        """Memory that the launches of a pass use one after the other."""
        if self._scratch_buf is None or self._scratch_buf.numel() < nbytes:
            self._scratch_buf = torch.empty(nbytes, dtype=torch.uint8, device=self.dev)
        return self._scratch_buf

    def _mixer(self, i, b, rows):
        spec, m, lw, store = self.spec, self.spec.layers[i].mixer, self._layer_weights(i), self.store.stores[i]
        n = rows.n
        proj, ctx = b.proj[HK.pad8(lw.proj.n_main)], b.ctx[HK.pad8(m.out_channels)]
        HK.linear(b.h, lw.proj, proj, n, ld=proj.shape[1], tail=b.gates if lw.proj.tail else None)
        if m.kind == "attention":
            att = HK.WindowAttention(m.heads, m.kv_heads, m.dim, m.scale, m.window, spec.eps, lw.q_norm, lw.k_norm, lw.slopes, *store)
            if rows.single:
                splits, ws = self._splits(n, m)
                att.decode(proj, n, rows.slot, rows.pos, ctx, splits, ws)
            else:
                att.prompt(proj, n, rows.slot, rows.pos, ctx, b.q_scale, rows.tiles)
        else:
            HK.mlstm(proj, n, m.heads, m.dim, m.vdim, b.gates, m.gate_cap, store[0], rows.slot, rows.seqs, rows.longest, b.o,
                     rows.longest > 8, self._scratch)
            HK.head_norm_gate(b.o, lw.head_norm, proj, m.gate_at, ctx, n, m.heads, m.vdim, spec.eps)
        HK.linear(ctx, lw.out, b.y, n, ld=spec.width, workspace=b.workspace)

    def _feed_forward(self, i, b, rows):
        mlp, lw = self.spec.layers[i].mlp, self._layer_weights(i)
        act = b.act[lw.gate.n_main]
        HK.linear(b.h, lw.gate, act, rows.n, up=lw.up, pair=H.PAIR_CLAMPED, limit=mlp.limit, slope=mlp.slope)
        HK.linear(act, lw.down, b.y, rows.n, ld=self.spec.width, workspace=b.workspace)

    def _layers(self, rows, pos_out=None):
        """All layers over the rows.  Returns the buffers with the last sublayer's result still to be added, and that
        sublayer's connections (`_logits` does both at once)."""
        spec, b = self.spec, self._rows_buffers(rows.n)
        norm = dict(eps=spec.eps, mult=spec.residual_mult, h=b.h)
        first = self._layer_weights(0)
        HK.streams_norm(b.streams, rows.n, table=self.w.embed, embed_scale=spec.embed_scale, ids=rows.ids, ids_index=rows.ids_index,
                        pos_out=pos_out, next_in=first.connect1[0], weight=first.norm1, **norm)
        done = None
        for i, layer in enumerate(spec.layers):
            lw = self._layer_weights(i)
            if i:
                HK.streams_norm(b.streams, rows.n, y=b.y, connect=done, next_in=lw.connect1[0], weight=lw.norm1, **norm)
            self._mixer(i, b, rows)
            done = lw.connect1[1:]
            if layer.mlp is not None:
                HK.streams_norm(b.streams, rows.n, y=b.y, connect=done, next_in=lw.connect2[0], weight=lw.norm2, **norm)
                self._feed_forward(i, b, rows)
                done = lw.connect2[1:]
            if self.probe is not None:
                total = torch.empty((rows.n, spec.width), dtype=F32, device=self.dev)
                HK.streams_norm(b.streams, rows.n, spec.eps, y=b.y, connect=done, mult=spec.residual_mult, write=False, sum_out=total,
                                dtype=self.dtype)
                self.probe(i, total)
        return b, done

    def _logits(self, b, done, count, out, gather=None):
        """Final norm and head of `count` rows: the pass's own, or those listed in `gather` (up to head_rows, repeats allowed)."""
        spec, h = self.spec, b.h
        if gather is not None:
            if self._head_h is None:
                self._head_h = torch.zeros((self.head_rows, h.shape[1]), dtype=self.dtype, device=self.dev)
            h = self._head_h
        HK.streams_norm(b.streams, count, spec.eps, y=b.y, connect=done, mult=spec.residual_mult, write=False, gather=gather,
                        weight=self.w.final_norm, h=h)
        HK.linear(h, self.w.head, out, count, ld=spec.vocab, cap=spec.logit_cap)

    # ------------------------------------------------------------------ sequences that come and go
    def open(self):
        capacity = self.store.capacity
        slot = self.store.open()
        if self.store.capacity != capacity:
            self.graph = None            # the recorded iteration addresses the memory the store has left
        return slot

    def close(self, slot):
        self.store.close(slot)

    def _pass(self, portions):
        """portions [(slot, token ids)]: device description of their rows."""
        ids = np.concatenate([np.asarray(t, np.int32) for _, t in portions])
        counts = np.array([len(t) for _, t in portions], np.int32)
        starts = np.concatenate([[0], np.cumsum(counts)[:-1]]).astype(np.int32)
        slots = np.repeat(np.array([s for s, _ in portions], np.int32), counts)
        pos = np.concatenate([self.store.length[s] + np.arange(len(t), dtype=np.int32) for s, t in portions]).astype(np.int32)
        tiles = [(a + k, min(H.WINDOW_TILE, c - k)) for a, c in zip(starts, counts) for k in range(0, c, H.WINDOW_TILE)]
        tr, tc = (np.array([t[j] for t in tiles], np.int32) for j in (0, 1))
        last = np.full(len(ids), -1, np.int32)
        last[starts] = starts + counts - 1
        flat = torch.from_numpy(np.concatenate([ids, slots, pos, last, starts, counts, tr, tc])).to(self.dev)
        parts = torch.split(flat, [len(ids)] * 4 + [len(counts)] * 2 + [len(tiles)] * 2)
        return Rows(len(ids), parts[1], parts[2], (parts[4], parts[5], len(counts)), bool((counts == 1).all()),
                    (parts[6], parts[7], len(tiles)), ids=parts[0], longest=int(counts.max()), last=parts[3],
                    portions=tuple((s, self.store.length[s], len(t)) for s, t in portions))

    def advance(self, entries):
        """entries [(slot, token ids, wanted places)]: the sequences' next tokens, as one batch, cut into passes where they
        are many.  Returns the logits fp32 [sum of wanted, vocab] at the wanted places, in their order."""
        spec, store = self.spec, self.store
        if len({e[0] for e in entries}) != len(entries):
            raise ValueError("advance: a sequence appears twice in one batch")
        for slot, tokens, want in entries:
            if store.length[slot] < 0:
                raise ValueError(f"advance: slot {slot} is not in use")
            if len(tokens) == 0 or store.length[slot] + len(tokens) > store.max_len:
                raise ValueError(f"advance: {len(tokens)} tokens after {store.length[slot]} (max_len {store.max_len})")
            if min(tokens) < 0 or max(tokens) >= spec.vocab:
                raise ValueError(f"advance: a token id outside [0, {spec.vocab})")
            if any(not 0 <= w < len(tokens) for w in want):
                raise ValueError("advance: a wanted place outside the tokens of its entry")
        out_at, total = {}, 0
        for e, (_, _, want) in enumerate(entries):
            for w in want:
                out_at.setdefault((e, w), []).append(total)
                total += 1
        logits = torch.empty((total, spec.vocab), dtype=F32, device=self.dev)
        at = [0] * len(entries)
        while any(a < len(e[1]) for a, e in zip(at, entries)):
            portions, rows_of, n = [], [], 0
            for e, (slot, tokens, _) in enumerate(entries):
                take = min(len(tokens) - at[e], store.portion, self.pass_rows - n)
                if take <= 0:
                    continue
                portions.append((slot, tokens[at[e]:at[e] + take]))
                rows_of += [(e, at[e] + k) for k in range(take)]
                at[e] += take
                n += take
            rows = self._pass(portions)
            b, done = self._layers(rows)
            picks = [(r, o) for r, key in enumerate(rows_of) for o in out_at.get(key, ())]
            for c in range(0, len(picks), self.head_rows):
                part = picks[c:c + self.head_rows]
                gather = torch.tensor([r for r, _ in part], dtype=I32, device=self.dev)
                got = torch.empty((len(part), spec.vocab), dtype=F32, device=self.dev)
                self._logits(b, done, len(part), got, gather)
                logits[torch.tensor([o for _, o in part], device=self.dev)] = got
            for slot, tokens in portions:
                store.length[slot] += len(tokens)
        return logits

    # ------------------------------------------------------------------ decode loop
    def _prepare_loop(self):
        s = self.spec
        if hasattr(self, "container"):
            return
        if self.store.max_len < s.max_len:
            raise ValueError(f"sequences of {s.max_len} tokens: the model has {self.store.max_len} positions")
        if self.store.capacity < s.batch:
            self.store._grow(s.batch)
        B = s.batch

        def zeros(*shape, dtype=I32):
            return torch.zeros(shape, dtype=dtype, device=self.dev)
        self.container, self.stop_mask, self.next_ids = zeros(B, s.max_len), zeros(B), zeros(B)
        self.step, self.keep_going = zeros(), zeros() + 1
        self.logits = zeros(B, s.vocab, dtype=F32)
        self.select = NextToken(B, s.vocab, s.topk, self.dev, f32_logits=True)
        lanes = torch.arange(B, dtype=I32, device=self.dev)
        self._loop_rows = Rows(B, lanes, zeros(B), (lanes, zeros(B) + 1, B), True, ids=self.container, ids_index=self.step)

    def reset(self, input_ids):
        ids = self.checked_ids(input_ids)
        self._prepare_loop()
        self.container.copy_(ids)
        self.stop_mask.zero_()
        self.step.zero_()
        self.keep_going.fill_(1)
        self.store.restart(range(self.spec.batch))

    def step_fn(self):
        from .. import kernels as K
        s, rows = self.spec, self._loop_rows
        b, done = self._layers(rows, pos_out=rows.pos)
        self._logits(b, done, rows.n, self.logits)
        self.select(self.logits, self.next_ids)
        K.step_update(self.container, None, self.stop_mask, self.step, self.next_ids, None, self.keep_going, s.pad_id, s.eos_id,
                      s.early_stop)

    def consume_prompt(self, n=None, rows_per_pass=None):
        """The first n loop iterations (default: all that only read the prompt) as passes over several positions of every
        sequence.  Cache, state and loop state end up as n iterations leave them.  Call after `reset`.  Returns n."""
        n = self.checked_prompt_count(n)
        B = self.spec.batch
        R = min(rows_per_pass or max(1, self.pass_rows // B), self.store.portion)
        if R < 1 or R * B > 4096:
            raise ValueError(f"consume_prompt: rows_per_pass * batch must lie in [1, 4096], got {R} * {B}")
        with torch.cuda.stream(self._stream):
            for p0 in range(0, n, R):
                ids = self._host_ids[:, p0:min(p0 + R, n)]
                self._layers(self._pass([(b, ids[b]) for b in range(B)]))
                for b in range(B):
                    self.store.length[b] += ids.shape[1]
            self.step.fill_(n)
        self._stream.synchronize()
        return n
