"""Kernels of attention by heads, of the residual that takes normed results, of routing and of expert mixtures, one by one against
oracle/golapel.py."""
import numpy as np
import pytest
import torch

from oracle import golapel as G

pytestmark = pytest.mark.gpu

DTYPES = ["float32", "bfloat16"]


def _dev(a, dtype=torch.float32):
    return torch.from_numpy(np.ascontiguousarray(a)).to("cuda").to(dtype).contiguous()


def _np(t):
    return t.float().cpu().numpy().astype(np.float64)


def _rel(got, want):
    return np.abs(got - want).max() / max(np.abs(want).max(), 1e-30)


def _hk():
    from poptransformer_amd import hybrid_kernels as HK
    return HK, HK.DTYPES


# ---------------------------------------------------------------------------------------------- attention
def _mixer(**kw):
    from poptransformer_amd.engine.hybrid import HeadMixer, Rotation
    rot = kw.pop("rot", None)
    base = dict(heads=4, kv_heads=2, dim=16, vdim=16, scale=0.5)
    return HeadMixer(**{**base, **kw}, rot=Rotation(*rot) if rot is not None else None)


WINDOW = dict(keys_are_values=True, sink=True, gate="head")
MIXERS = {
    "window": _mixer(window=20, keep=5, rot=(100.0, 16), **WINDOW),
    "window no keep, rotated in part": _mixer(heads=3, kv_heads=3, dim=24, vdim=24, window=33, rot=(30.0, 8, False, 2.0), **WINDOW),
    "window of one, five to one": _mixer(heads=5, kv_heads=1, dim=40, vdim=40, window=1, keep=1, rot=(30.0, 40), **WINDOW),
    "all positions": _mixer(heads=2, kv_heads=1, dim=64, vdim=64, rot=(1e4, 64), **WINDOW),
    "more kept than the window": _mixer(dim=8, vdim=8, window=3, keep=70, **WINDOW),
    "wide heads": _mixer(heads=8, kv_heads=2, dim=128, vdim=128, scale=0.1, window=130, keep=4, rot=(1e4, 64), **WINDOW),
    "widest tiles": _mixer(heads=2, kv_heads=1, dim=256, vdim=256, scale=0.06, window=50, keep=2, rot=(1e4, 256), **WINDOW),
    "maps": _mixer(vdim=24, chunk=20, diff=0.3),
    "maps, odd sizes": _mixer(heads=7, kv_heads=1, dim=11, vdim=5, chunk=37, diff=0.7),
    "maps, wide": _mixer(heads=4, kv_heads=2, dim=64, vdim=128, scale=0.15, chunk=100, diff=0.5),
    "maps, widest": _mixer(heads=2, kv_heads=1, dim=136, vdim=200, scale=0.1, chunk=70, diff=0.5),
    "maps, every position": _mixer(heads=2, kv_heads=2, dim=32, vdim=16, diff=0.1),
    "chunks": _mixer(heads=3, kv_heads=3, dim=24, vdim=16, chunk=14, rot=(80.0, 24, True, 3.0, (64.0, 4.0, 1.0)), gate="feature"),
    "chunks of one": _mixer(dim=16, vdim=32, chunk=1, rot=(80.0, 8, True), gate="feature"),
    "chunks, odd sizes": _mixer(heads=6, kv_heads=2, dim=10, vdim=9, chunk=65, rot=(80.0, 6, True), gate="feature"),
    "chunks, beyond the tiles": _mixer(heads=2, kv_heads=1, dim=264, vdim=300, scale=0.06, chunk=40, rot=(1e4, 128, True), gate="feature"),
    "chunks, wide": _mixer(heads=4, kv_heads=4, dim=128, vdim=64, scale=0.1, chunk=128, rot=(1e4, 128, True), gate="feature"),
}


class _Layer:
    """One layer's attention over given projections of some sequences, beside the oracle's."""

    def __init__(self, m, dtype, lengths, seed, standout=(), portion=64, max_len=400):
        HK, T = _hk()
        self.m, self.dtype, self.HK = m, T[dtype], HK
        rng = np.random.default_rng(seed)
        self.M, self.D, self.E = m.maps, m.stored_dim, m.stored_vdim
        round_ = lambda a: _np(_dev(a, self.dtype))
        self.wq, self.wk = (1 + 0.2 * rng.standard_normal(m.dim) for _ in range(2))
        self.sink = rng.standard_normal(m.heads) + 1 if m.sink else None
        self.lam = 0.63 if m.diff is not None else 0.0
        self.eps = 1e-3
        self.q, self.k, self.v, self.gate, self.want = {}, {}, {}, {}, {}
        f, amplitude = m.rot.frequencies() if m.rot is not None else (None, 1.0)
        for s, n in lengths.items():
            q = round_(rng.standard_normal((n, m.heads, self.M, m.dim)))
            k = round_(rng.standard_normal((n, m.kv_heads, self.M, m.dim)))
            for i, j in standout:                                    # query i's score of key j towers over the others
                if i < n:
                    k[j] = q[i, ::m.heads // m.kv_heads] = round_(rng.standard_normal(k[j].shape))
            v = k[:, :, 0] if m.keys_are_values else round_(rng.standard_normal((n, m.kv_heads, m.vdim)))
            g = rng.standard_normal((n, m.heads) if m.gate == "head" else (n, m.heads, m.vdim))
            g = g if m.gate != "feature" else round_(g)
            qn, kn = G.rms_norm(q, self.wq, self.eps), G.rms_norm(k, self.wk, self.eps)
            if m.rot is not None:
                qn, kn = (G.rotate(x, f, amplitude, m.rot.neighbours) for x in (qn, kn))
            kn = round_(kn)
            mask = G.chunk_mask(n, m.chunk) if m.chunk else G.window_mask(n, m.window, m.keep)
            a = [G.attend(qn[:, :, t], kn[:, :, t], v, m.scale, mask, self.sink) for t in range(self.M)]
            o = a[0] if self.M == 1 else G.differential_combine(*a, self.lam, m.diff, self.eps)
            if m.gate is not None:
                o = o * G.sigmoid(g[..., None] if m.gate == "head" else g)
            self.q[s], self.k[s], self.v[s], self.gate[s], self.want[s] = q, k, v, g, o
        n = max(min(max_len, m.keep + m.span - 1 + portion), m.keep + 1)
        slots = max(lengths) + 1
        self.keys = torch.full((slots, m.kv_heads, self.M, n, self.D), 9.0, dtype=self.dtype, device="cuda")
        self.values = torch.full((slots, m.kv_heads, n, self.E), 9.0, dtype=self.dtype, device="cuda")
        self.cos_sin = _dev(m.rot.angles(max_len)) if m.rot is not None else None
        self.at = dict.fromkeys(lengths, 0)

    def _packed(self, t, size, stored, paired):
        """heads of `size` features, in pairs' order where they are turned, padded with zeros"""
        m = self.m
        if paired and m.rot is not None:
            t = t[..., m.rot.pairs(m.dim)]
        out = np.zeros((*t.shape[:-1], stored))
        out[..., :size] = t
        return out.reshape(t.shape[0], -1)

    def run(self, counts, splits=None):
        """The next tokens of the sequences as one pass; compares every row."""
        from poptransformer_amd import _hybrid_lib as H
        HK, m = self.HK, self.m
        sel = [(s, slice(self.at[s], self.at[s] + c)) for s, c in counts.items()]
        cat = lambda d: np.concatenate([d[s][k] for s, k in sel])
        parts = [self._packed(cat(self.q), m.dim, self.D, True), self._packed(cat(self.k), m.dim, self.D, True)]
        if not m.keys_are_values:
            parts.append(self._packed(cat(self.v), m.vdim, self.E, False))
        if m.gate == "feature":
            parts.append(self._packed(cat(self.gate), m.vdim, self.E, False))
        proj = _dev(np.concatenate(parts, 1), self.dtype)
        rows = len(proj)
        head_gate = _dev(cat(self.gate)) if m.gate == "head" else None
        slot = _dev(np.repeat(list(counts), list(counts.values())), torch.int32)
        pos = _dev(np.concatenate([np.arange(k.start, k.stop) for _, k in sel]), torch.int32)
        out = torch.full((rows, m.heads * self.E), 7.0, dtype=self.dtype, device="cuda")
        norms = [_dev(self._packed(w[None], m.dim, self.D, True)[0]) for w in (self.wq, self.wk)]
        sink = _dev(self.sink) if m.sink else None
        att = HK.HeadAttention(m, self.eps, *norms, self.cos_sin, sink, self.lam, self.keys, self.values,
                               proj, rows, slot, pos, head_gate, out)
        if splits is not None:
            att.decode(splits, HK.head_workspace(rows, m, splits, "cuda") if splits > 1 else None)
        else:
            tiles, first = [], 0
            for c in counts.values():
                tiles += [(first + a, min(H.HEAD_TILE, c - a)) for a in range(0, c, H.HEAD_TILE)]
                first += c
            att.prompt((_dev([t[0] for t in tiles], torch.int32), _dev([t[1] for t in tiles], torch.int32), len(tiles)))
        for s, c in counts.items():
            self.at[s] += c
        got = _np(out).reshape(rows, m.heads, self.E)
        if m.keys_are_values and m.rot is not None:
            back = np.argsort(m.rot.pairs(m.dim))
            got[..., :m.dim] = got[..., :m.dim][..., back]
        assert (got[..., m.vdim:] == 0).all()
        want = cat(self.want)
        err = np.abs(got[..., :m.vdim] - want).max((1, 2)) / max(np.abs(want).max(), 1e-3)
        assert err.max() < (2e-5 if self.dtype == torch.float32 else 2.5e-2), (counts, int(err.argmax()), err.max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MIXERS))
def test_attention_in_portions_and_decoding(name, dtype):
    """Sequences of unequal length in one pass, portions down to two tokens, single tokens in one to many parts, rings that wrap."""
    m = MIXERS[name]
    layer = _Layer(m, dtype, {2: 330, 0: 150}, 1)
    for counts, splits in (({2: 1, 0: 1}, 1), ({2: 64, 0: 2}, None), ({2: 1}, 3), ({2: 1, 0: 1}, 2), ({0: 33, 2: 64}, None), ({0: 1}, 1), ({2: 2}, None),
                           ({2: 1, 0: 1}, 64), ({0: 50, 2: 1}, None), ({2: 64, 0: 61}, None), ({2: 1}, 1), ({2: 1}, 5), ({2: 64}, None)):
        print(f"heads {name} {dtype} {counts} splits {splits}", flush=True)
        layer.run(counts, splits)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["window", "all positions", "wide heads", "maps, wide", "chunks, wide"])
def test_attention_of_long_portions(name, dtype):
    layer = _Layer(MIXERS[name], dtype, {1: 390, 0: 300}, 2, portion=300, max_len=400)
    for counts in ({1: 290, 0: 1}, {0: 299, 1: 100}):
        print(f"heads {name} {dtype} {counts}", flush=True)
        layer.run(counts)


def _edges(m):
    """(query, key) just inside and just outside everything that limits what is seen"""
    if m.chunk:
        c = m.chunk
        return [(3 * c - 1, 2 * c), (2 * c, 2 * c - 1), (4 * c, 4 * c), (4 * c + 1, 3 * c)] if c > 1 else [(5, 4), (9, 9)]
    w, k = m.window, m.keep
    far = k + w + 60
    pairs = [(far, far - w + 1), (far + 1, far - w + 1), (far + 7, k), (far + 8, far + 8 - w)]
    return pairs + ([(far + 9, 0), (far + 10, k - 1)] if k else [])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["window", "window no keep, rotated in part", "window of one, five to one", "more kept than the window", "wide heads",
                                  "maps", "maps, odd sizes", "chunks", "chunks of one", "chunks, odd sizes", "chunks, wide"])
def test_attention_at_the_edges_of_what_is_seen(name, dtype):
    """One key's score towers over the others, once where it is just seen and once where it just is not."""
    m = MIXERS[name]
    n = max(i for i, _ in _edges(m)) + 3
    for cuts in ([n], [1] * n, [2] * (n // 2)):
        layer = _Layer(m, dtype, {0: n}, 3, _edges(m), portion=n, max_len=n)
        print(f"edges {name} {dtype} {len(cuts)} cuts", flush=True)
        for c in cuts:
            layer.run({0: c}, 1 if c == 1 else None)


def test_attention_checks_its_arguments():
    HK, _ = _hk()
    layer = _Layer(MIXERS["window"], "float32", {0: 10}, 0)
    layer.keys = layer.keys[:, :, :, :5].contiguous()
    with pytest.raises(ValueError):
        layer.run({0: 1}, 1)                                         # values of another length
    layer.values = layer.values[:, :, :5].contiguous()
    with pytest.raises(ValueError):
        layer.run({0: 1}, 1)                                         # no rows besides those that are kept
    layer = _Layer(MIXERS["maps"], "float32", {0: 10}, 0)
    with pytest.raises(ValueError):
        layer.run({0: 1}, 65)


# ---------------------------------------------------------------------------------------------- residual and routing
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 53), (3, 84), (17, 1032), (2, 4096), (70, 2048), (5, 8200)])
def test_result_norm(dtype, rows, width):
    HK, T = _hk()
    rng = np.random.default_rng(width)
    ld, tol = HK.pad8(width), 5e-6 if dtype == "float32" else 6e-3
    ids, table = rng.integers(0, 19, (rows, 3)), _np(_dev(rng.standard_normal((19, width)), T[dtype]))
    x, h = torch.full((rows, width), 7.0, device="cuda"), torch.full((rows, ld), 7.0, dtype=T[dtype], device="cuda")
    pos = torch.zeros(rows, dtype=torch.int32, device="cuda")
    HK.result_norm(x, rows, 1e-5, h, table=_dev(table, T[dtype]), embed_scale=2.5, ids=_dev(ids, torch.int32), ids_index=_dev(np.array(2), torch.int32),
                   pos_out=pos)
    want = 2.5 * table[ids[:, 2]]
    assert _rel(_np(x), want) < 1e-6 and _rel(_np(h)[:, :width], want) < tol and (_np(h)[:, width:] == 0).all() and (pos == 2).all()
    w, wf = rng.standard_normal(width), rng.standard_normal(width)
    experts, top = 9, 3
    router = _np(_dev(rng.standard_normal((experts + 1, width)) / np.sqrt(width), T[dtype]))
    padded = np.zeros((experts + 1, ld))
    padded[:, :width] = router
    for variant in range(5):
        print(f"result {dtype} {rows}x{width} {variant}", flush=True)
        y, parts = rng.standard_normal((rows, width)), rng.standard_normal((rows, 4, width))
        weights = _dev(rng.random((rows, 4)))
        part_type = T[dtype] if variant == 2 else torch.float32
        before, wts, pv = _np(x), _np(weights), _np(_dev(parts, part_type))
        kw, u = [(dict(y=_dev(y)), y),
                 (dict(parts=_dev(parts), n_parts=4, part_weight=weights), (wts[..., None] * pv).sum(1)),
                 (dict(parts=_dev(parts, part_type), n_parts=3, parts_ld=4, part_weight=weights, y=_dev(y), y_weight=(weights, 3)),
                  (wts[:, :3, None] * pv[:, :3]).sum(1) + wts[:, 3:] * y),
                 (dict(y=_dev(y), final_weight=_dev(wf)), y), (dict(y=_dev(y)), y)][variant]
        routing = HK.Routing(rows, experts, top, variant == 4, 1.3, "cuda")
        if variant in (0, 4):
            kw.update(router=_dev(padded[:experts + routing.shared], T[dtype]), routing=routing)
        HK.result_norm(x, rows, 1e-5, h, weight=_dev(w), **kw)
        want = before + G.rms_norm(u, w, 1e-5)
        assert _rel(_np(x), want) < 3e-6
        assert _rel(_np(h)[:, :width], G.rms_norm(want, wf, 1e-5) if variant == 3 else want) < tol
        assert (_np(h)[:, width:] == 0).all()
        if variant in (0, 4):
            z = _np(h)[:, :width] @ router.T
            chosen, weight = G.route(z[:, :experts], top, 1.3)
            assert np.array_equal(routing.chosen.cpu().numpy()[:, :top], chosen)
            assert _rel(_np(routing.weights)[:, :top], weight) < 1e-4
            if variant == 4:
                assert (routing.chosen[:, top] == experts).all() and _rel(_np(routing.weights)[:, top], G.sigmoid(z[:, experts])) < 1e-4


@pytest.mark.parametrize("rows,experts,top", [(1, 1, 1), (5, 8, 3), (300, 64, 6), (2, 65, 65), (7, 1000, 8)])
@pytest.mark.parametrize("shared", [False, True])
def test_routing(rows, experts, top, shared):
    HK, _ = _hk()
    z = np.random.default_rng(experts).standard_normal((rows, experts + shared)) * 3
    z[0, :experts // 2] = z[0, 0]                                    # equal scores: the first ones
    r = HK.Routing(rows + 2, experts, top, shared, 0.8, "cuda")
    r(_dev(z), rows)
    chosen, weight = G.route(z[:, :experts].astype(np.float32).astype(np.float64), top, 0.8)
    assert np.array_equal(r.chosen.cpu().numpy()[:rows, :top], chosen) and _rel(_np(r.weights)[:rows, :top], weight) < 1e-5
    if shared:
        assert (r.chosen[:rows, top] == experts).all() and _rel(_np(r.weights)[:rows, top], G.sigmoid(z[:, experts])) < 1e-5


@pytest.mark.parametrize("rows,experts,top,shared,d", [(17, 8, 3, True, 84), (1, 5, 1, False, 53), (300, 64, 6, False, 1032), (40, 33, 2, True, 256),
                                                       (16, 130, 4, True, 2100), (33, 1000, 8, True, 72)])
def test_routing_by_product(rows, experts, top, shared, d):
    HK, T = _hk()
    rng = np.random.default_rng(rows)
    h, w = (torch.zeros((n, HK.pad8(d)), dtype=torch.bfloat16, device="cuda") for n in (rows, experts + shared))
    h[:, :d], w[:, :d] = _dev(rng.standard_normal((rows, d))), _dev(rng.standard_normal((experts + shared, d)) * 2 / np.sqrt(d))
    r = HK.Routing(rows + 2, experts, top, shared, 0.8, "cuda")
    r.chosen.fill_(-7)
    r.by_product(h, HK.WideWeight(w[:, :d].float(), T["bfloat16"]), rows)
    z = _np(h) @ _np(w).T
    chosen, weight = G.route(z[:, :experts], top, 0.8)
    assert np.array_equal(r.chosen.cpu().numpy()[:rows, :top], chosen) and _rel(_np(r.weights)[:rows, :top], weight) < 1e-4
    assert (r.chosen[rows:] == -7).all()
    if shared:
        assert (r.chosen[:rows, top] == experts).all() and _rel(_np(r.weights)[:rows, top], G.sigmoid(z[:, experts])) < 1e-4


# ---------------------------------------------------------------------------------------------- experts
def _choices(rng, rows, experts, top, how):
    if how == "all the same":
        return np.tile(np.arange(top)[::-1], (rows, 1))
    return np.stack([rng.permutation(experts)[:top] for _ in range(rows)])


@pytest.mark.parametrize("tile", [128, 256])
def test_lists_of_the_experts_rows(tile):
    HK, _ = _hk()
    rng = np.random.default_rng(0)
    for rows, experts, top, shared, how in ((1, 4, 2, False, ""), (700, 5, 2, True, ""), (2048, 64, 8, False, ""), (300, 1000, 3, True, ""),
                                            (513, 9, 1, False, "all the same")):
        r = HK.Routing(rows, experts, top, shared, 1.0, "cuda")
        chosen = _choices(rng, rows, experts, top, how)
        r.chosen[:, :top] = _dev(chosen, torch.int32)
        if shared:
            r.chosen[:, top] = experts
        lists = HK.expert_lists(rows, top, experts, tile, "cuda")
        HK.group_experts(r, rows, tile, lists)
        got = lists.cpu().numpy()
        begin = got[4:4 + experts + 1]
        counts = np.bincount(chosen.reshape(-1), minlength=experts)
        assert np.array_equal(np.diff(begin), counts) and begin[0] == 0
        order_at = 4 + (experts + 4) // 4 * 4
        order = got[order_at:order_at + rows * top]
        flat = r.chosen.cpu().numpy().reshape(-1)
        for e in range(experts):
            assert sorted(order[begin[e]:begin[e + 1]]) == list(np.flatnonzero(flat == e))
        n = got[0]
        tiles = got[order_at + (rows * top + 3) // 4 * 4:][:4 * n].reshape(n, 4)
        assert n == (-(-counts // tile)).sum()
        for e in range(experts):
            mine = tiles[tiles[:, 0] == e]
            assert mine[:, 2].sum() == counts[e] and (mine[:, 2] <= tile).all()
            assert np.array_equal(mine[:, 1], begin[e] + tile * np.arange(len(mine)))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 2, 7, 16, 17, 130, 600])
def test_experts(dtype, rows):
    """Both products of a mixture, directly and over lists, some experts without rows, with and without a shared expert."""
    HK, T = _hk()
    from poptransformer_amd import _hybrid_lib as H
    rng = np.random.default_rng(rows)
    for experts, top, d, ff, shared_ff, how in ((6, 2, 84, 40, 24, ""), (5, 1, 53, 18, None, ""), (33, 4, 200, 72, 136, ""), (3, 3, 136, 1040, 56, ""),
                                                (7, 2, 2100, 100, 300, "all the same")):
        shared = shared_ff is not None
        r = HK.Routing(rows, experts, top, shared, 1.0, "cuda")
        chosen = _choices(rng, rows, experts, top, how)
        r.chosen[:, :top] = _dev(chosen, torch.int32)
        if shared:
            r.chosen[:, top] = experts
        x = torch.zeros((rows, HK.pad8(d)), dtype=T[dtype], device="cuda")
        x[:, :d] = _dev(rng.standard_normal((rows, d)), T[dtype])

        def weights(count, n):
            make = lambda a, b: [_dev(rng.standard_normal((a, b)) * 1.5 / np.sqrt(b), T[dtype]) for _ in range(count)]
            return make(n, d), make(n, d), make(d, n)
        routed, extra = weights(experts, ff), weights(1, shared_ff) if shared else None

        def packed(w, n, limit):
            g, u = (HK.ExpertWeight(t, T[dtype], main_to=HK.pad8(n)) for t in w[:2])
            return dict(w=g, up=u, pair=H.PAIR_CLAMPED, limit=limit, slope=1.702), dict(w=HK.ExpertWeight(w[2], T[dtype]))

        def expert(w, e, row, limit):
            sd = {n: _np(t[e]) for n, t in zip(("gate", "up", "down"), w)}
            return G.clamped_expert(sd, "", _np(x)[row, :d], limit, lambda a: _np(_dev(a, T[dtype])))
        pair, down = packed(routed, ff, 1.1)
        ways = ["lists 128", "lists 256"] + (["direct"] if dtype == "bfloat16" and rows <= 16 else [])
        want = np.zeros((rows, r.choices, d))
        for i in range(rows):
            for c in range(top):
                want[i, c] = expert(routed, chosen[i, c], i, 1.1)
            if shared:
                want[i, top] = expert(extra, 0, i, 0.7)
        for way in ways:
            print(f"experts {dtype} rows {rows} {experts} of {d}x{ff} {way}", flush=True)
            direct = way == "direct"
            ld = max(HK.pad8(ff), HK.pad8(shared_ff or 0)) if direct else HK.pad8(ff)
            act = torch.full((rows * r.choices, ld), 7.0, dtype=T[dtype], device="cuda")
            out = torch.full((rows * r.choices, d), 7.0, dtype=T[dtype] if way == "lists 256" else torch.float32, device="cuda")
            kw, shared_pair, shared_down = {}, None, None
            if direct and shared:
                shared_pair, shared_down = packed(extra, shared_ff, 0.7)
            if not direct:
                tile = int(way.split()[1])
                lists = HK.expert_lists(rows, top, experts, tile, "cuda")
                HK.group_experts(r, rows, tile, lists)
                kw = dict(lists=lists, tile_rows=tile)
            HK.experts(x, r, rows, pair, act, shared_pair, **kw)
            HK.experts(act, r, rows, down, out, shared_down, **kw)
            got = _np(out).reshape(rows, r.choices, d)
            done = r.choices if direct else top
            assert (got[:, done:] == 7.0).all()
            tol = 1e-5 if dtype == "float32" else 2e-2
            assert _rel(got[:, :done], want[:, :done]) < tol
        if shared:                                                   # the weight of a single expert in a plain product
            g, u = extra[:2]
            act = torch.empty((rows, HK.pad8(shared_ff)), dtype=T[dtype], device="cuda")
            first = packed(extra, shared_ff, 0.7)[0]
            HK.linear(x, first["w"], act, rows, **{k: v for k, v in first.items() if k != "w"})
            a, b = _np(x)[:, :d] @ _np(g[0]).T, _np(x)[:, :d] @ _np(u[0]).T
            a, b = np.minimum(a, 0.7), np.clip(b, -0.7, 0.7)
            assert _rel(_np(act)[:, :shared_ff], a * G.sigmoid(1.702 * a) * (b + 1)) < (1e-5 if dtype == "float32" else 1e-2)
            assert (_np(act)[:, shared_ff:] == 0).all()
