"""Torch-tensor front end of poptransformer_hybrid.h, as `kernels` is of poptransformer_hip.h: operands are checked on the
host, raw pointers go to the library on torch's current stream, nothing is computed on the CPU.
"""
import ctypes

import torch

from . import _hybrid_lib as H

F32, I32 = torch.float32, torch.int32
DTYPES = {"bfloat16": torch.bfloat16, "float32": torch.float32}
_CODE = {torch.bfloat16: H.BF16, torch.float32: H.FP32}


def _stream():
    return ctypes.c_void_p(torch.cuda.current_stream().cuda_stream)


def _p(t):
    return t.data_ptr() if t is not None else None


def _need(t, dtype, what, numel=None):
    if not t.is_cuda or t.dtype != dtype or not t.is_contiguous():
        raise ValueError(f"{what} must be a contiguous {dtype} device tensor")
    if numel is not None and t.numel() < numel:
        raise ValueError(f"{what} holds {t.numel()} elements, {numel} needed")


def pad8(n):
    return (n + 7) // 8 * 8


class WideWeight:
    """A Linear weight [N, K] in bf16 (tiled for the matrix unit) or fp32 (as it is).  K is padded with zeros to a multiple
    of 8.  The last `tail` channels may go to an fp32 buffer of their own, with a bias.  `main_to`: further zero channels
    after the main ones (results 0) up to that count, so that the result can be the padded input of another Linear.  `whole`: whole
    workgroup tiles of channels also where there are few, for launches of many rows that it shares with larger weights."""

    def __init__(self, w, dtype, tail=0, tail_bias=None, main_to=None, whole=False):
        n, k = w.shape
        main = n - tail
        self.n_main = main if main_to is None else main_to
        self.tail, self.K, self.dtype = tail, pad8(k), dtype
        if self.n_main != main and tail:
            raise ValueError("a weight with a tail takes no further channels")
        total = self.n_main + tail
        # many channels: whole workgroup tiles of 128 (the padding goes nowhere)
        self.N = (total + 127) // 128 * 128 if dtype == torch.bfloat16 and (whole or total >= 1024) else total
        full = torch.zeros((self.N, self.K), dtype=dtype, device=w.device)
        full[:n, :k] = w.to(dtype)
        self.tail_bias = tail_bias.to(F32).contiguous() if tail_bias is not None else None
        if dtype == torch.bfloat16:
            lib = H.load()
            self.data = torch.empty(lib.pta_bf16_tiled_bytes(self.N, self.K), dtype=torch.uint8, device=w.device)
            H.check(lib.pta_bf16_tile(full.data_ptr(), self.data.data_ptr(), self.N, self.K, _stream()))
            torch.cuda.current_stream().synchronize()      # `full` goes back to the allocator here
        else:
            self.data = full

    @property
    def nbytes(self):
        return (self.n_main + self.tail) * self.K * (2 if self.dtype == torch.bfloat16 else 4)


def linear_workspace(rows, channels, device):
    return torch.empty(H.load().pta_wide_linear_workspace_bytes(rows, channels), dtype=torch.uint8, device=device)


def _linear_args(x, w, out, rows, ld=None, tail=None, cap=0.0, up=None, pair=H.PAIR_NONE, limit=0.0, slope=0.0, workspace=None, bias=None,
                 bias2=None, act=H.ACT_NONE, mul=None, accumulate=False):
    _need(x, w.dtype, "x", rows * w.K)
    ld = w.n_main if ld is None else ld
    if out.dtype not in (w.dtype, F32):
        raise ValueError(f"out must be {w.dtype} or float32")
    _need(out, out.dtype, "out", rows * ld)
    if x.shape[-1] != w.K:
        raise ValueError(f"matmul: contracting dimensions differ ({x.shape[-1]} vs {w.K})")
    if up is not None and (up.N, up.K, up.dtype) != (w.N, w.K, w.dtype):
        raise ValueError("the weights of a pair must be alike")
    if w.tail:
        _need(tail, F32, "tail", rows * w.tail)
    for b in (bias, bias2):
        if b is not None:
            _need(b, F32, "bias", w.n_main)
    if mul is not None:
        _need(mul, w.dtype, "mul", rows * ld)
    return H.WideLinearArgs(_CODE[w.dtype], _p(x), rows, w.K, w.N, _p(w.data), _p(up.data) if up is not None else None, pair, limit, slope,
                            cap, _p(out), ld, w.n_main, int(out.dtype == F32), _p(tail) if w.tail else None, w.tail, _p(w.tail_bias),
                            _p(workspace), workspace.numel() if workspace is not None else 0, _p(bias), _p(bias2), act, _p(mul),
                            int(accumulate))


def linear(x, w, out, rows, **kw):
    """out[:rows] = x[:rows] @ w^T with the fused epilogues of pta_wide_linear; `up`: the second weight of a pair."""
    a = _linear_args(x, w, out, rows, **kw)
    H.check(H.load().pta_wide_linear(ctypes.byref(a), _stream()))
    return out


def linear_group(rows, *calls):
    """Several `linear`s (x, w, out, keywords) over inputs of one shape, in one launch where there are few rows."""
    a = (H.WideLinearArgs * len(calls))(*(_linear_args(x, w, out, rows, **kw) for x, w, out, kw in calls))
    H.check(H.load().pta_wide_linear_group(a, len(calls), _stream()))


def streams_norm(streams, rows, eps, weight=None, h=None, table=None, embed_scale=1.0, ids=None, ids_index=None, pos_out=None, y=None,
                 connect=None, mult=1.0, write=True, gather=None, next_in=None, sum_out=None, dtype=None):
    """One sublayer boundary (pta_streams_norm).  streams [R, S, width]; connect = (out [S], mix [S, S]) of the finished
    sublayer whose result is y; next_in [S] of the sublayer that follows (None: the plain sum)."""
    _, S, width = streams.shape
    _need(streams, F32, "streams", 0 if gather is not None else rows * S * width)
    code = _CODE[h.dtype if h is not None else dtype]
    if table is not None:
        _need(table, h.dtype if h is not None else dtype, "table")
        _need(ids, I32, "ids")
    if h is not None:
        _need(h, h.dtype, "h", rows * h.shape[-1])
        _need(weight, F32, "weight", width)
    if y is not None:
        _need(y, F32, "y")
    stride = ids.shape[-1] if ids is not None and ids.dim() == 2 else 1
    a = H.StreamsArgs(code, rows, width, S, _p(streams), _p(table), table.shape[0] if table is not None else 0, embed_scale, _p(ids),
                      stride, _p(ids_index), _p(pos_out), _p(y), _p(connect[0]) if connect is not None else None,
                      _p(connect[1]) if connect is not None else None, mult, int(write), _p(gather), _p(next_in), _p(weight), eps,
                      _p(h), h.shape[-1] if h is not None else 0, _p(sum_out))
    H.check(H.load().pta_streams_norm(ctypes.byref(a), _stream()))
    return h


def window_workspace(rows, heads, dim, splits, device):
    n = H.load().pta_window_attention_workspace_bytes(rows, heads, dim, splits)
    return torch.empty(max(n, 16), dtype=torch.uint8, device=device)


class WindowAttention:
    """The arguments of the windowed-attention calls over one set of row buffers and one layer's cache."""

    def __init__(self, heads, kv_heads, dim, scale, window, eps, q_norm, k_norm, slopes, ring, rinv):
        _need(q_norm, F32, "q_norm", heads * dim)
        _need(k_norm, F32, "k_norm", kv_heads * dim)
        _need(slopes, F32, "slopes", heads)
        if ring.dim() != 4 or ring.shape[1] != kv_heads or ring.shape[3] != pad8(dim):
            raise ValueError(f"ring must be [slots, {kv_heads}, length, {pad8(dim)}], got {tuple(ring.shape)}")
        self.H, self.G, self.D = heads, kv_heads, dim
        self.scale, self.window, self.eps = scale, window, eps
        self.q_norm, self.k_norm, self.slopes, self.ring, self.rinv = q_norm, k_norm, slopes, ring, rinv

    def _args(self, proj, rows, slot, pos, out, q_scale=None, tiles=None, splits=1, workspace=None):
        es, HD = proj.element_size(), self.H * self.D
        ring_len = self.ring.shape[2]
        _need(proj, self.ring.dtype, "projection", rows * proj.shape[-1])
        _need(slot, I32, "slot", rows)
        _need(pos, I32, "pos", rows)
        _need(out, proj.dtype, "out", rows * out.shape[-1])
        if proj.shape[-1] < 2 * HD + self.G * self.D:
            raise ValueError("the projection rows must hold q | k | gate")
        base = proj.data_ptr()
        tr, tc, nt = tiles if tiles is not None else (None, None, 0)
        return H.WindowArgs(_CODE[proj.dtype], rows, self.H, self.G, self.D, base, base + HD * es, base + (HD + self.G * self.D) * es,
                            proj.shape[-1], _p(self.q_norm), _p(self.k_norm), self.eps, self.scale, _p(self.slopes),
                            self.window or (1 << 30), _p(self.ring), _p(self.rinv), ring_len, _p(slot), _p(pos), _p(q_scale), _p(tr),
                            _p(tc), nt, splits, _p(workspace), workspace.numel() if workspace is not None else 0, _p(out), out.shape[-1])

    def decode(self, proj, rows, slot, pos, out, splits, workspace):
        """One row per sequence: norms, append and attention."""
        a = self._args(proj, rows, slot, pos, out, splits=splits, workspace=workspace)
        H.check(H.load().pta_window_decode(ctypes.byref(a), _stream()))

    def prompt(self, proj, rows, slot, pos, out, q_scale, tiles):
        """Rows of a pass with several rows per sequence; tiles = (first rows, row counts, how many)."""
        a = self._args(proj, rows, slot, pos, out, q_scale=q_scale, tiles=tiles)
        lib = H.load()
        H.check(lib.pta_window_append(ctypes.byref(a), _stream()))
        H.check(lib.pta_window_attention(ctypes.byref(a), _stream()))


def shift_norm(x, rows, groups, eps, w1, h1, w2=None, h2=None, shift=None, hm=None, state=None, slot=None, last=None, pos=None,
               positions=0, table=None, pos_table=None, embed_scale=1.0, ids=None, ids_index=None, pos_out=None, gather=None):
    """Front of a layer with parallel sublayers (pta_shift_norm).  x [R, width] fp32; h1, h2, hm [R, ld]."""
    width = x.shape[-1]
    _need(x, F32, "x", 0 if gather is not None else rows * width)
    _need(w1, F32, "w1", width)
    _need(h1, h1.dtype, "h1", rows * h1.shape[-1])
    for h, w in ((h2, w2), (hm, shift)):
        if h is not None:
            _need(h, h1.dtype, "result", rows * h1.shape[-1])
            _need(w, F32, "weight", width)
    if shift is not None:
        _need(state, F32, "state")
        _need(slot, I32, "slot", rows)
    if last is not None:
        _need(last, I32, "last", rows)
    if table is not None:
        _need(table, h1.dtype, "table")
        _need(ids, I32, "ids")
    if pos_table is not None:
        _need(pos_table, h1.dtype, "pos_table", positions * width)
    stride = ids.shape[-1] if ids is not None and ids.dim() == 2 else 1
    a = H.ShiftNormArgs(_CODE[h1.dtype], rows, width, groups, _p(x), _p(table), _p(pos_table), table.shape[0] if table is not None else 0,
                        positions, embed_scale, _p(ids), stride, _p(ids_index), _p(pos), _p(pos_out), _p(gather), eps, _p(w1), _p(w2),
                        _p(shift), _p(state), _p(slot), _p(last), _p(h1), _p(h2), _p(hm), h1.shape[-1])
    H.check(H.load().pta_shift_norm(ctypes.byref(a), _stream()))


class ShortConv:
    """A short causal convolution over `channels` channels: weight [taps, channels] (the last row is the current token's), bias
    [channels] or None.  ring [slots, taps, channels] holds the newest rows of every sequence as they were projected."""

    def __init__(self, weight, bias=None, silu=False):
        _need(weight, F32, "weight")
        self.weight, self.bias, self.silu = weight, bias, bool(silu)
        self.taps, self.channels = weight.shape
        if bias is not None:
            _need(bias, F32, "bias", self.channels)

    def args(self, ring):
        _need(ring, ring.dtype, "ring")
        if tuple(ring.shape[1:]) != (self.taps, self.channels):
            raise ValueError(f"ring must be [slots, {self.taps}, {self.channels}], got {tuple(ring.shape)}")
        return H.Conv(self.channels, self.taps, _p(self.weight), _p(self.bias), int(self.silu), _p(ring))

    def __call__(self, x, x_at, y, ring, rows, slot, pos, last, tiles):
        """y[:, :channels] = the convolved columns x_at .. of x, for rows of a pass; tiles = (first rows, row counts, how many)."""
        _need(x, ring.dtype, "x", rows * x.shape[-1])
        _need(y, ring.dtype, "y", rows * y.shape[-1])
        if x.shape[-1] < x_at + self.channels or x_at % 8:
            raise ValueError("the rows do not hold the channels")
        for t in (slot, pos, last):
            _need(t, I32, "rows' places", rows)
        tr, tc, n = tiles
        _need(tr, I32, "tiles", n)
        _need(tc, I32, "tiles", n)
        a = H.ShortConvArgs(_CODE[ring.dtype], self.args(ring), x.data_ptr() + x_at * x.element_size(), x.shape[-1], _p(y), y.shape[-1],
                            _p(slot), _p(pos), _p(last), _p(tr), _p(tc), n)
        H.check(H.load().pta_short_conv(ctypes.byref(a), _stream()))


def pad32(n):
    return (n + 31) // 32 * 32


class LatentAttention:
    """The latent-attention calls of one layer over one set of row buffers.  Sizes as stored; `proj` rows hold the query latent
    and, where `kv_norm` is given (the layer has a cache of its own), the row's cache entry."""

    def __init__(self, sizes, scale, window, eps, q_norm, kv_norm, cos_sin, ring, rows, slot, pos):
        """sizes = (heads, D, P, E, R, q_rank, kv_rank)."""
        self.H, self.D, self.P, self.E, self.R, self.q_rank, self.kv_rank = sizes
        _need(q_norm, F32, "q_norm", self.q_rank)
        if kv_norm is not None:
            _need(kv_norm, F32, "kv_norm", self.kv_rank)
        if ring.dim() != 3 or ring.shape[2] != self.R + self.P:
            raise ValueError(f"ring must be [slots, length, {self.R + self.P}], got {tuple(ring.shape)}")
        _need(ring, ring.dtype, "ring")
        _need(cos_sin, F32, "cos_sin")
        if cos_sin.shape[1:] != (self.P // 2, 2):
            raise ValueError("cos_sin must be [positions, P / 2, 2]")
        _need(slot, I32, "slot", rows)
        _need(pos, I32, "pos", rows)
        self.rows, self.dtype = rows, ring.dtype
        self.a = H.LatentArgs(_CODE[ring.dtype], rows, *sizes)
        a = self.a
        a.q_norm, a.kv_norm, a.eps, a.scale, a.window = _p(q_norm), _p(kv_norm), eps, scale, window or (1 << 30)
        a.cos_sin, a.positions, a.ring, a.ring_len, a.slot, a.pos = _p(cos_sin), cos_sin.shape[0], _p(ring), ring.shape[1], _p(slot), _p(pos)

    def _call(self, name):
        H.check(getattr(H.load(), "pta_latent_" + name)(ctypes.byref(self.a), _stream()))

    def append(self, proj, cq):
        """Normed query latents, and the rows' entries in the layer's own cache."""
        _need(proj, self.dtype, "projection", self.rows * proj.shape[-1])
        _need(cq, self.dtype, "cq", self.rows * pad8(self.q_rank))
        self.a.proj, self.a.ld, self.a.cq = _p(proj), proj.shape[-1], _p(cq)
        self._call("append")

    def _result(self, q, gate, out):
        """gate: fp32 [rows, H] per head, or (rows of a projection, first column) per feature"""
        _need(q, self.dtype, "q", self.rows * self.H * (self.D + self.P))
        _need(out, self.dtype, "out", self.rows * self.H * self.E)
        self.a.q, self.a.out = _p(q), _p(out)
        if isinstance(gate, tuple):
            proj, at = gate
            _need(proj, self.dtype, "gate", self.rows * proj.shape[-1])
            if proj.shape[-1] < at + self.H * self.E:
                raise ValueError("the projection does not hold the gate")
            self.a.feature_gate, self.a.gate_ld = proj.data_ptr() + at * proj.element_size(), proj.shape[-1]
        else:
            _need(gate, F32, "gate", self.rows * self.H)
            self.a.gate = _p(gate)

    def absorbed(self, q, uk_t, q_latent, splits, part_o, part_ml, uv, gate, out):
        """Every row over the cache itself, its window in `splits` parts."""
        n = self.rows * self.H
        self._result(q, gate, out)
        _need(uk_t, self.dtype, "uk_t", self.H * self.R * self.D)
        _need(q_latent, self.dtype, "q_latent", n * (self.R + self.P))
        _need(part_o, F32, "part_o", n * splits * self.R)
        _need(part_ml, F32, "part_ml", n * splits * 2)
        _need(uv, self.dtype, "uv", self.H * self.E * self.R)
        a = self.a
        a.uk_t, a.q_latent, a.splits, a.part_o, a.part_ml, a.uv = _p(uk_t), _p(q_latent), splits, _p(part_o), _p(part_ml), _p(uv)
        for name in ("absorb", "rows", "values"):
            self._call(name)

    def over_heads(self, q, keys, key_latent, key_rot, kv_weight, kv, tiles, gate, out):
        """Tiles of rows over keys and values of every head, which are made from the cache first.  keys = (slots, positions);
        tiles = (first rows, row counts, key row of position 0)."""
        n, (slot, pos), (tr, tc, tk) = keys[0].numel(), keys, tiles
        self._result(q, gate, out)
        for t, want in ((slot, n), (pos, n), (tr, len(tr)), (tc, len(tr)), (tk, len(tr))):
            _need(t, I32, "keys and tiles", want)
        _need(key_latent, self.dtype, "key_latent", n * self.R)
        _need(key_rot, self.dtype, "key_rot", n * self.P)
        _need(kv, self.dtype, "kv", n * kv_weight.n_main)
        if kv_weight.n_main != self.H * (self.D + self.E) or kv_weight.K != self.R:
            raise ValueError("kv_weight does not fit the sizes")
        a = self.a
        a.keys, a.key_slot, a.key_pos, a.key_latent, a.key_rot, a.kv = n, _p(slot), _p(pos), _p(key_latent), _p(key_rot), _p(kv)
        a.tile_row, a.tile_count, a.tile_key, a.tiles = _p(tr), _p(tc), _p(tk), len(tr)
        self._call("gather")
        for k in range(0, n, 4096):
            m = min(4096, n - k)
            linear(key_latent[k:k + m], kv_weight, kv[k:k + m], m)
        self._call("tiles")


def latent_tiles_fit(dtype, D, P, E):
    return bool(H.load().pta_latent_tiles_fit(_CODE[dtype], D, P, E))


class HeadAttention:
    """The calls of attention over cached keys and values of one layer.  `mixer` gives the sizes, the visible positions and what the
    result goes through (engine/hybrid.py HeadMixer); proj rows hold q | k | v (none where the values are the keys) | gate per
    feature (where there is one)."""

    def __init__(self, mixer, eps, q_norm, k_norm, cos_sin, sink, lam, keys, values, proj, rows, slot, pos, head_gate, out, far=None):
        m = mixer
        heads, G, M, D, E = m.heads, m.kv_heads, m.maps, m.stored_dim, m.stored_vdim
        es, ld = proj.element_size(), proj.shape[-1]
        for t, n in ((keys, (G, M, D)), (values, (G, E))):
            _need(t, proj.dtype, "cache")
            if (*t.shape[1:-2], t.shape[-1]) != n or t.shape[-2] != keys.shape[-2]:
                raise ValueError(f"the cache must be [slots, {n[:-1]}, length, {n[-1]}], got {tuple(t.shape)}")
        _need(proj, proj.dtype, "projection", rows * ld)
        _need(slot, I32, "slot", rows)
        _need(pos, I32, "pos", rows)
        _need(out, proj.dtype, "out", rows * heads * E)
        for t, n in ((q_norm, D), (k_norm, D), (sink, heads), (head_gate, rows * heads)):
            if t is not None:
                _need(t, F32, "norms, sinks and gates", n)
        at_k = heads * M * D
        at_v = at_k if m.keys_are_values else at_k + G * M * D
        at_gate = at_k + G * M * D + (0 if m.keys_are_values else G * E)
        if ld < at_gate + (heads * E if m.gate == "feature" else 0):
            raise ValueError("the projection rows do not hold queries, keys, values and gate")
        base = proj.data_ptr()
        a = self.a = H.HeadArgs(_CODE[proj.dtype], rows, heads, G, M, D, E, m.dim, m.vdim, base, base + at_k * es, base + at_v * es, ld)
        a.q_norm, a.k_norm, a.eps, a.scale = _p(q_norm), _p(k_norm), eps, m.scale
        if cos_sin is not None:
            _need(cos_sin, F32, "cos_sin")
            a.cos_sin, a.positions, a.rot = _p(cos_sin), cos_sin.shape[0], cos_sin.shape[1] * 2
        a.window, a.keep, a.chunk = m.window or (1 << 30), m.keep, m.chunk or 0
        a.keys, a.values, a.ring_len, a.slot, a.pos, a.sink = _p(keys), _p(values), keys.shape[-2], _p(slot), _p(pos), _p(sink)
        a.lambda_, a.diff, a.out, a.splits = lam, m.diff or 0.0, _p(out), 1
        a.head_gate = _p(head_gate)
        a.gate = base + at_gate * es if m.gate == "feature" else None
        if far is not None:
            for t in far:
                _need(t, F32, "far", heads)
            a.far1, a.far2 = (_p(t) for t in far)

    def decode(self, splits, workspace, conv=None):
        """One row per sequence: norms, rotation, append and attention; conv = (ShortConv, ring): queries, keys and values go
        through it first."""
        a = self.a
        if conv is not None:
            a.conv = conv[0].args(conv[1])
        a.splits, a.workspace, a.workspace_bytes = splits, _p(workspace), workspace.numel() if workspace is not None else 0
        H.check(H.load().pta_head_decode(ctypes.byref(a), _stream()))

    def prompt(self, tiles):
        """Rows of a pass with several rows per sequence; tiles = (first rows, row counts, how many)."""
        a, lib = self.a, H.load()
        tr, tc, n = tiles
        _need(tr, I32, "tiles", n)
        _need(tc, I32, "tiles", n)
        a.tile_row, a.tile_count, a.tiles = _p(tr), _p(tc), n
        H.check(lib.pta_head_append(ctypes.byref(a), _stream()))
        H.check(lib.pta_head_attention(ctypes.byref(a), _stream()))


def head_workspace(rows, mixer, splits, device):
    n = H.load().pta_head_attention_workspace_bytes(rows, mixer.heads, mixer.maps, mixer.stored_vdim, splits)
    return torch.empty(max(n, 16), dtype=torch.uint8, device=device)


class Routing:
    """Where the routing of up to `rows` rows goes: choice c of row r in chosen[r, c], its weight beside it."""

    def __init__(self, rows, experts, top, shared, scale, device, score=H.SCORE_SOFTMAX, groups=1, keep=1, share=False):
        self.score, self.groups, self.keep, self.share = score, groups, keep, bool(share)
        self.experts, self.top, self.shared, self.scale, self.choices = experts, top, bool(shared), scale, top + bool(shared)
        self.chosen = torch.zeros((rows, self.choices), dtype=I32, device=device)
        self.weights = torch.zeros((rows, self.choices), dtype=F32, device=device)

    def args(self, rows, correction=None):
        _need(self.chosen, I32, "routing", rows * self.choices)
        if correction is not None:
            _need(correction, F32, "correction", self.experts)
        return H.Routing(self.experts, self.top, int(self.shared), self.scale, _p(self.chosen), _p(self.weights), self.score, _p(correction),
                         self.groups, self.keep, int(self.share))

    def __call__(self, logits, rows, correction=None):
        """Routes rows by their logits fp32 [rows, experts + shared]."""
        _need(logits, F32, "router logits", rows * (self.experts + self.shared))
        a = self.args(rows, correction)
        H.check(H.load().pta_route(_p(logits), rows, ctypes.byref(a), _stream()))

    def by_product(self, h, router, rows, correction=None):
        """Routes bf16 rows by their products with the router, a WideWeight."""
        _need(h, torch.bfloat16, "rows", rows * h.shape[-1])
        if (router.dtype, router.K, router.n_main) != (torch.bfloat16, h.shape[-1], self.experts + self.shared):
            raise ValueError("the router does not fit the rows or the routing")
        a = self.args(rows, correction)
        H.check(H.load().pta_route_rows(_p(h), h.shape[-1], rows, _p(router.data), ctypes.byref(a), _stream()))


def result_norm(x, rows, eps, h, weight=None, table=None, embed_scale=1.0, ids=None, ids_index=None, pos_out=None, y=None, y_weight=None,
                parts=None, n_parts=0, parts_ld=None, part_weight=None, final_weight=None, router=None, routing=None):
    """x += norm(result), h = x (pta_result_norm).  The result is y (times y_weight [rows, n][:, c], given as (weights, c)) plus the
    weighted parts [rows, parts_ld, width] (the first n_parts of a row, default: all); with `router` the rows are routed into `routing`."""
    width = x.shape[-1]
    _need(x, F32, "x", rows * width)
    _need(h, h.dtype, "h", rows * h.shape[-1])
    if table is not None:
        _need(table, h.dtype, "table")
        _need(ids, I32, "ids")
    else:
        _need(weight, F32, "weight", width)
    if final_weight is not None:
        _need(final_weight, F32, "final_weight", width)
    if y is not None:
        _need(y, F32, "y", rows * width)
    stride = ids.shape[-1] if ids is not None and ids.dim() == 2 else 1
    a = H.ResultNormArgs(_CODE[h.dtype], rows, width, _p(x), _p(table), table.shape[0] if table is not None else 0, embed_scale, _p(ids), stride,
                         _p(ids_index), _p(pos_out), _p(y))
    if y_weight is not None:
        w, c = y_weight
        _need(w, F32, "y_weight", rows * w.shape[-1])
        a.y_weight, a.weights_ld = w.data_ptr() + 4 * c, w.shape[-1]
    if parts is not None:
        if parts.dtype not in (F32, h.dtype):
            raise ValueError(f"parts must be float32 or {h.dtype}")
        parts_ld = parts_ld or n_parts
        _need(parts, parts.dtype, "parts", rows * parts_ld * width)
        _need(part_weight, F32, "part_weight", rows * part_weight.shape[-1])
        if a.weights_ld not in (0, part_weight.shape[-1]):
            raise ValueError("the weights of y and of the parts belong to one buffer")
        a.parts, a.n_parts, a.parts_ld, a.part_f32 = _p(parts), n_parts, parts_ld, int(parts.dtype == F32)
        a.part_weight, a.weights_ld = _p(part_weight), part_weight.shape[-1]
    a.weight, a.eps, a.final_weight, a.h, a.h_ld = _p(weight), eps, _p(final_weight), _p(h), h.shape[-1]
    if router is not None:
        _need(router, h.dtype, "router", (routing.experts + routing.shared) * h.shape[-1])
        a.router, a.routing = _p(router), routing.args(rows)
    H.check(H.load().pta_result_norm(ctypes.byref(a), _stream()))


def depth_norm(history, depth, rows, eps, h, norm_weight, centred=True, weights=None, y=None, y_weight=None, next=None, table=None, embed_scale=1.0,
               ids=None, ids_index=None, pos_out=None, side_table=None, side=None, router=None, routing=None, correction=None):
    """The end of a layer (pta_depth_norm).  history fp32 [depths, R, width], of which the first `depth` count; next: the index in it
    that gets the average; side_table [vocab, layers, ld], side [layers, R, ld]."""
    width = history.shape[-1]
    _need(history, F32, "history")
    if history.shape[1] < rows or depth > history.shape[0] or (next is not None and not depth <= next < history.shape[0]):
        raise ValueError(f"a history of {tuple(history.shape)} for {rows} rows at depth {depth}")
    _need(h, h.dtype, "h", rows * h.shape[-1])
    _need(norm_weight, F32, "norm_weight", width)
    a = H.DepthNormArgs(_CODE[h.dtype], rows, width, _p(history), history.shape[1] * width, depth)
    if weights is not None:
        _need(weights, F32, "weights", depth)
        a.weights = _p(weights)
    if y is not None:
        _need(y, F32, "y", rows * width)
        _need(y_weight, F32, "y_weight", width)
        a.y, a.y_weight = _p(y), _p(y_weight)
    if next is not None:
        a.next = history[next].data_ptr()
    a.centred, a.norm_weight, a.eps, a.h, a.h_ld = int(centred), _p(norm_weight), eps, _p(h), h.shape[-1]
    if table is not None:
        _need(table, h.dtype, "table")
        _need(ids, I32, "ids")
        a.table, a.vocab, a.embed_scale, a.ids = _p(table), table.shape[0], embed_scale, _p(ids)
        a.ids_stride, a.ids_index, a.pos_out = ids.shape[-1] if ids.dim() == 2 else 1, _p(ids_index), _p(pos_out)
        if side is not None:
            _need(side_table, h.dtype, "side_table")
            _need(side, h.dtype, "side")
            if side_table.shape != (table.shape[0], side.shape[0], side.shape[2]) or side.shape[1] < rows:
                raise ValueError(f"the tokens' own parts {tuple(side_table.shape)} do not fit {tuple(side.shape)}")
            a.side_table, a.side, a.side_layers, a.side_ld, a.side_stride = _p(side_table), _p(side), side.shape[0], side.shape[2], side[0].numel()
    if router is not None:
        _need(router, h.dtype, "router", (routing.experts + routing.shared) * h.shape[-1])
        a.router, a.routing = _p(router), routing.args(rows, correction)
    H.check(H.load().pta_depth_norm(ctypes.byref(a), _stream()))


def add_parts(x, rows, h, parts=None, n_parts=0, parts_ld=None, part_weight=None):
    """x [R, width] fp32 += the weighted parts [rows, parts_ld, width]; h = x (pta_add_parts)."""
    width = x.shape[-1]
    _need(x, F32, "x", rows * width)
    _need(h, h.dtype, "h", rows * h.shape[-1])
    a = H.AddPartsArgs(_CODE[h.dtype], rows, width, _p(x))
    if parts is not None:
        parts_ld = parts_ld or n_parts
        if parts.dtype not in (F32, h.dtype):
            raise ValueError(f"parts must be float32 or {h.dtype}")
        _need(parts, parts.dtype, "parts", rows * parts_ld * width)
        _need(part_weight, F32, "part_weight", rows * part_weight.shape[-1])
        a.parts, a.n_parts, a.parts_ld, a.part_f32 = _p(parts), n_parts, parts_ld, int(parts.dtype == F32)
        a.part_weight, a.weights_ld = _p(part_weight), part_weight.shape[-1]
    a.h, a.h_ld = _p(h), h.shape[-1]
    H.check(H.load().pta_add_parts(ctypes.byref(a), _stream()))


class ExpertWeight:
    """Linear weights of one shape, one per expert, one after the other: bf16 tiled (channels rounded up to 16, many to 128), fp32
    as they are.  main_to: further zero channels, as WideWeight's.  That of a single expert also serves `linear`."""
    tail, tail_bias = 0, None

    def __init__(self, weights, dtype, main_to=None):
        """weights: an iterable of [N, K] tensors"""
        parts = []
        for w in weights:
            n, k = w.shape
            self.n_main, self.K, self.dtype = n if main_to is None else main_to, pad8(k), dtype
            tile = 128 if self.n_main >= 1024 else 16
            self.N = (self.n_main + tile - 1) // tile * tile
            full = torch.zeros((self.N, self.K), dtype=dtype, device=w.device)
            full[:n, :k] = w.to(dtype)
            if dtype == torch.bfloat16:
                lib = H.load()
                data = torch.empty(lib.pta_bf16_tiled_bytes(self.N, self.K), dtype=torch.uint8, device=w.device)
                H.check(lib.pta_bf16_tile(full.data_ptr(), data.data_ptr(), self.N, self.K, _stream()))
                torch.cuda.current_stream().synchronize()      # `full` goes back to the allocator here
                full = data
            parts.append(full)
        self.count, self.data = len(parts), torch.stack(parts)

    @property
    def nbytes(self):
        """Bytes of one expert's."""
        return self.n_main * self.K * (2 if self.dtype == torch.bfloat16 else 4)

    def args(self, up=None, pair=H.PAIR_NONE, limit=0.0, slope=0.0):
        if up is not None and (up.N, up.K, up.count) != (self.N, self.K, self.count):
            raise ValueError("the weights of a pair must be alike")
        return H.ExpertWeights(_p(self.data), _p(up.data) if up is not None else None, self.K, self.N, self.n_main, pair, limit, slope)


def expert_lists(rows, top, experts, tile_rows, device):
    return torch.zeros(H.load().pta_expert_lists_size(rows, top, experts, tile_rows), dtype=I32, device=device)


def group_experts(routing, rows, tile_rows, lists):
    _need(lists, I32, "lists", H.load().pta_expert_lists_size(rows, routing.top, routing.experts, tile_rows))
    H.check(H.load().pta_group_experts(_p(routing.chosen), rows, routing.top, routing.choices, routing.experts, tile_rows, _p(lists), _stream()))


def experts(x, routing, rows, routed, out, shared=None, lists=None, tile_rows=0):
    """One product of every row's experts (pta_experts).  routed, shared: dict(w=ExpertWeight, and of a pair up=, pair=, limit=, slope=);
    x [rows, ld] for a pair, else [rows * choices, ld]; out [rows * choices, ld]."""
    w, dtype, n = routed["w"], routed["w"].dtype, rows * routing.choices
    pair = routed.get("up") is not None
    _need(x, dtype, "x", (rows if pair else n) * x.shape[-1])
    if out.dtype not in (dtype, F32):
        raise ValueError(f"out must be {dtype} or float32")
    _need(out, out.dtype, "out", n * out.shape[-1])
    if w.count != routing.experts or (shared is not None and (shared["w"].dtype != dtype or not routing.shared or (shared.get("up") is not None) != pair)):
        raise ValueError("the experts' weights do not fit the routing")
    pack = lambda d: d["w"].args(**{k: v for k, v in d.items() if k != "w"})
    a = H.ExpertsArgs(_CODE[dtype], rows, routing.experts, routing.top, routing.choices, _p(routing.chosen), _p(x), x.shape[-1], pack(routed))
    if shared is not None:
        a.shared = pack(shared)
    a.Y, a.ld_y, a.out_f32 = _p(out), out.shape[-1], int(out.dtype == F32)
    if lists is not None:
        _need(lists, I32, "lists", H.load().pta_expert_lists_size(rows, routing.top, routing.experts, tile_rows))
        a.lists, a.tile_rows = _p(lists), tile_rows
    H.check(H.load().pta_experts(ctypes.byref(a), _stream()))


def mlstm_state(slots, heads, dim, vdim, device):
    return torch.zeros((slots, H.load().pta_mlstm_state_floats(heads, dim, vdim)), dtype=F32, device=device)


def mlstm(proj, rows, heads, dim, vdim, gates, cap, state, slot, seqs, longest, o, chunked, scratch=None):
    """proj rows hold q | k | v | ...; seqs = (first rows, row counts, how many), longest: the largest count; o [rows, heads *
    vdim] fp32.  scratch(bytes) -> uint8 tensor: memory for passes that are cut into segments (default: allocated here)."""
    es, HD, HE = proj.element_size(), heads * dim, heads * vdim
    seq_row, seq_count, n = seqs
    _need(proj, proj.dtype, "projection", rows * proj.shape[-1])
    _need(gates, F32, "gates", rows * 2 * heads)
    _need(state, F32, "state")
    _need(o, F32, "o", rows * HE)
    if state.shape[1] != H.load().pta_mlstm_state_floats(heads, dim, vdim) or proj.shape[-1] < 2 * HD + 2 * HE:
        raise ValueError("mlstm: the state or the projection does not fit the sizes")
    base = proj.data_ptr()
    a = H.MlstmArgs(_CODE[proj.dtype], rows, heads, dim, vdim, base, base + HD * es, base + 2 * HD * es, proj.shape[-1], _p(gates), cap,
                    _p(state), _p(slot), _p(seq_row), _p(seq_count), n, longest, int(chunked), _p(o), None, 0)
    need = H.load().pta_mlstm_workspace_bytes(ctypes.byref(a))
    if need:
        ws = scratch(need) if scratch is not None else torch.empty(need, dtype=torch.uint8, device=proj.device)
        a.workspace, a.workspace_bytes = _p(ws), ws.numel()
    H.check(H.load().pta_mlstm(ctypes.byref(a), _stream()))


def head_norm_gate(o, weight, proj, gate_at, out, rows, heads, vdim, eps):
    """out = per-head RMS norm of o, times weight, times sigmoid of the projection's channels from gate_at on."""
    _need(o, F32, "o", rows * heads * vdim)
    _need(weight, F32, "weight", heads * vdim)
    _need(out, proj.dtype, "out", rows * out.shape[-1])
    if proj.shape[-1] < gate_at + heads * vdim:
        raise ValueError("the projection does not hold the gate")
    H.check(H.load().pta_head_norm_gate(_CODE[proj.dtype], _p(o), _p(weight), proj.data_ptr() + gate_at * proj.element_size(),
                                        proj.shape[-1], _p(out), out.shape[-1], rows, heads, vdim, eps, _stream()))


def ssd_state(slots, heads, dim, vdim, device):
    return torch.zeros((slots, H.load().pta_ssd_state_floats(heads, dim, vdim)), dtype=F32, device=device)


def ssd(x, x_at, rows, heads, groups, dim, vdim, dt, constants, state, slot, seqs, longest, y, chunked=False, scratch=None, pos=None, conv=None):
    """State-space recurrence (pta_ssd) over columns x_at .. of x, which hold x | b | c; sizes as stored.  dt fp32 [rows, heads];
    constants = (dt_bias, a_log, skip); seqs = (first rows, row counts, how many); y fp32 [rows, heads * vdim].  conv = (ShortConv, ring):
    every sequence has one row, its columns as projected."""
    es, at_b, at_c = x.element_size(), heads * vdim, heads * vdim + groups * dim
    _need(x, x.dtype, "x", rows * x.shape[-1])
    _need(dt, F32, "dt", rows * heads)
    for t in constants:
        _need(t, F32, "dt_bias, a_log and skip", heads)
    _need(state, F32, "state")
    _need(slot, I32, "slot", rows)
    _need(y, F32, "y", rows * heads * vdim)
    if state.shape[1] != H.load().pta_ssd_state_floats(heads, dim, vdim) or x.shape[-1] < x_at + at_c + groups * dim or x_at % 8:
        raise ValueError("ssd: the state or the rows do not fit the sizes")
    base, (seq_row, seq_count, n) = x.data_ptr() + x_at * es, seqs
    a = H.SsdArgs(_CODE[x.dtype], rows, heads, groups, dim, vdim, base, base + at_b * es, base + at_c * es, x.shape[-1], _p(dt),
                  *(_p(t) for t in constants), _p(state), _p(slot), _p(pos), _p(seq_row), _p(seq_count), n, longest, int(chunked), _p(y))
    if conv is not None:
        _need(pos, I32, "pos", rows)
        a.conv = conv[0].args(conv[1])
    else:
        need = H.load().pta_ssd_workspace_bytes(ctypes.byref(a))
        if need:
            ws = scratch(need) if scratch is not None else torch.empty(need, dtype=torch.uint8, device=x.device)
            a.workspace, a.workspace_bytes = _p(ws), ws.numel()
    H.check(H.load().pta_ssd(ctypes.byref(a), _stream()))


def gated_norm(y, z, weight, out, rows, heads, stored, vdim, parts, eps):
    """out = norm in `parts` equal parts of y silu(z), times weight (pta_gated_norm); z: rows whose first columns are the gate."""
    n = heads * stored
    _need(y, F32, "y", rows * n)
    _need(z, z.dtype, "z", rows * z.shape[-1])
    _need(weight, F32, "weight", n)
    _need(out, z.dtype, "out", rows * n)
    a = H.GatedNormArgs(_CODE[z.dtype], rows, heads, stored, vdim, parts, _p(y), _p(z), z.shape[-1], _p(weight), eps, _p(out))
    H.check(H.load().pta_gated_norm(ctypes.byref(a), _stream()))


def argmax(logits, ids):
    _need(logits, F32, "logits")
    _need(ids, I32, "ids")
    n = logits.shape[-1]
    H.check(H.load().pta_argmax_f32(_p(logits), _p(ids), None, logits.numel() // n, n, _stream()))
    return ids


def topk(logits, k, ids, values=None):
    _need(logits, F32, "logits")
    n = logits.shape[-1]
    H.check(H.load().pta_topk_f32(_p(logits), _p(ids), _p(values), logits.numel() // n, n, k, _stream()))
    return ids
