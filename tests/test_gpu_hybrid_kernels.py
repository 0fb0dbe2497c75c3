"""Kernels of poptransformer_hybrid.h one by one against the plain mechanisms of oracle/zekilix.py (float64)."""
import numpy as np
import pytest
import torch

from oracle import zekilix as Z

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


# ---------------------------------------------------------------------------------------------- Linear
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 3, 5, 8, 16, 17, 40, 64, 65, 130, 300])
def test_linear(dtype, rows):
    HK, T = _hk()
    rng = np.random.default_rng(rows)
    for n, k, tail in ((24, 40, 0), (50, 72, 6), (1160, 136, 8), (640, 1100, 0)):
        print(f"linear {dtype} rows {rows} n {n} k {k} tail {tail}", flush=True)
        w = _dev(rng.standard_normal((n, k)) / np.sqrt(k)).to(T[dtype])
        x = torch.zeros((rows, HK.pad8(k)), dtype=T[dtype], device="cuda")
        x[:, :k] = _dev(rng.standard_normal((rows, k))).to(T[dtype])
        bias = _dev(rng.standard_normal(tail)) if tail else None
        ww = HK.WideWeight(w.float(), T[dtype], tail=tail, tail_bias=bias)
        want = _np(x)[:, :k] @ _np(w).T
        ld = HK.pad8(n - tail)
        out = torch.full((rows, ld), 7.0, dtype=T[dtype], device="cuda")
        gates = torch.full((rows, max(tail, 1)), 7.0, device="cuda")
        ws = HK.linear_workspace(rows, ww.N, "cuda")
        HK.linear(x, ww, out, rows, ld=ld, tail=gates if tail else None, workspace=ws)
        tol = 2e-6 if dtype == "float32" else 6e-3
        assert _rel(_np(out)[:, :n - tail], want[:, :n - tail]) < tol
        assert (_np(out)[:, n - tail:] == 7.0).all()          # padding channels and padding columns are left alone
        if tail:
            assert _rel(_np(gates), want[:, n - tail:] + _np(bias)) < 1e-5
        else:
            f32 = torch.empty((rows, n), device="cuda")
            HK.linear(x, ww, f32, rows, ld=n, cap=1.5)
            assert _rel(_np(f32), Z.softcap(want, 1.5)) < 1e-5


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 4, 9, 16, 33, 64, 100, 260])
def test_gate_up_pair(dtype, rows):
    HK, T = _hk()
    from poptransformer_amd import _hybrid_lib as H
    rng = np.random.default_rng(rows)
    for n, k in ((20, 48), (1030, 520)):
        print(f"pair {dtype} rows {rows} n {n} k {k}", flush=True)
        g, u = (_dev(rng.standard_normal((n, k)) * 2 / np.sqrt(k)).to(T[dtype]) for _ in range(2))
        x = _dev(rng.standard_normal((rows, k))).to(T[dtype])
        wg, wu = (HK.WideWeight(w.float(), T[dtype], main_to=HK.pad8(n)) for w in (g, u))
        out = torch.full((rows, HK.pad8(n)), 7.0, dtype=T[dtype], device="cuda")
        G, U = _np(x) @ _np(g).T, _np(x) @ _np(u).T
        tol = 1e-5 if dtype == "float32" else 6e-3
        HK.linear(x, wg, out, rows, up=wu, pair=H.PAIR_CLAMPED, limit=0.8, slope=1.702)
        assert _rel(_np(out)[:, :n], Z.clamped_glu(G, U, 0.8)) < tol
        assert (_np(out)[:, n:] == 0).all()
        HK.linear(x, wg, out, rows, up=wu, pair=H.PAIR_SWIGLU)
        assert _rel(_np(out)[:, :n], U * G * Z.sigmoid(G)) < tol


def test_argument_checks():
    HK, T = _hk()
    w = HK.WideWeight(torch.zeros((8, 16), device="cuda"), torch.float32)
    x = torch.zeros((2, 16), device="cuda")
    with pytest.raises(ValueError):
        HK.linear(x.double(), w, torch.zeros((2, 8), device="cuda"), 2)
    with pytest.raises(ValueError):
        HK.linear(torch.zeros((2, 24), device="cuda"), w, torch.zeros((2, 8), device="cuda"), 2)
    with pytest.raises(ValueError):
        HK.linear(x, w, torch.zeros((2, 4), device="cuda"), 2)


# ---------------------------------------------------------------------------------------------- streams
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("S", [1, 2, 3, 4, 8])
def test_streams_and_norm(dtype, S):
    HK, T = _hk()
    rng = np.random.default_rng(S)
    for rows, d in ((1, 36), (5, 75), (70, 1028), (3, 4096)):
        print(f"streams {dtype} S {S} rows {rows} width {d}", flush=True)
        x = rng.standard_normal((rows, S, d))
        y, w = rng.standard_normal((rows, d)), rng.standard_normal(d)
        win, wout, mix, nxt = (rng.standard_normal(s) for s in (S, S, (S, S), S))
        st, h = _dev(x), torch.full((rows, HK.pad8(d)), 7.0, dtype=T[dtype], device="cuda")
        total = torch.empty((rows, d), device="cuda")
        HK.streams_norm(st, rows, 1e-5, weight=_dev(w), h=h, y=_dev(y), connect=(_dev(wout), _dev(mix)), mult=0.6, next_in=_dev(nxt),
                        sum_out=total)
        new = Z.connect(np.moveaxis(x, 1, 0), win, wout, mix, 0.6, lambda u: y)
        tol = 1e-5 if dtype == "float32" else 6e-3
        assert _rel(_np(st), np.moveaxis(new, 0, 1)) < 5e-6
        assert _rel(_np(total), new.sum(0)) < 5e-6
        assert _rel(_np(h)[:, :d], Z.layer_norm(np.tensordot(nxt, new, axes=1), w, 1e-5)) < tol
        assert (_np(h)[:, d:] == 0).all()
        # gathered rows, plain sum, streams left alone
        pick = np.array([rows - 1, 0, rows // 2], np.int32)
        before = st.clone()
        h3 = torch.empty((3, HK.pad8(d)), dtype=T[dtype], device="cuda")
        HK.streams_norm(st, 3, 1e-5, weight=_dev(w), h=h3, y=_dev(y), connect=(_dev(wout), _dev(mix)), mult=0.6, write=False,
                        gather=_dev(pick, torch.int32))
        again = Z.connect(np.moveaxis(_np(before), 1, 0), win, wout, mix, 0.6, lambda u: y).sum(0)
        assert torch.equal(st, before)
        assert _rel(_np(h3)[:, :d], Z.layer_norm(again, w, 1e-5)[pick]) < tol
        # from the embedding, ids out of a container's column
        table = _dev(rng.standard_normal((11, d))).to(T[dtype])
        ids = rng.integers(0, 11, (rows, 6)).astype(np.int32)
        at, pos = torch.tensor(4, dtype=torch.int32, device="cuda"), torch.zeros(rows, dtype=torch.int32, device="cuda")
        HK.streams_norm(st, rows, 1e-5, weight=_dev(w), h=h, table=table, embed_scale=2.5, ids=_dev(ids, torch.int32), ids_index=at,
                        pos_out=pos, next_in=_dev(nxt))
        e = _np(table)[ids[:, 4]] * 2.5
        assert _rel(_np(st), np.repeat(e[:, None], S, 1)) < 1e-6
        assert _rel(_np(h)[:, :d], Z.layer_norm(e * nxt.sum(), w, 1e-5)) < tol
        assert (pos == 4).all()


# ---------------------------------------------------------------------------------------------- attention
class Attention:
    """One attention layer's cache, fed in portions; the projection rows are given."""

    def __init__(self, dtype, H, G, D, window, slots, ring_len, seed, scale=None):
        HK, T = _hk()
        rng = np.random.default_rng(seed)
        self.HK, self.dtype, self.H, self.G, self.D, self.window = HK, T[dtype], H, G, D, window
        self.qn, self.kn = 1 + 0.3 * rng.standard_normal(H * D), 1 + 0.3 * rng.standard_normal(G * D)
        self.scale = D ** -0.5 if scale is None else scale
        self.slopes = Z.head_slopes(H)
        self.ring = torch.zeros((slots, G, ring_len, HK.pad8(D)), dtype=self.dtype, device="cuda")
        self.rinv = torch.zeros((slots, ring_len), device="cuda")
        self.att = HK.WindowAttention(H, G, D, self.scale, window, 1e-5, _dev(self.qn), _dev(self.kn), _dev(self.slopes), self.ring, self.rinv)

    def project(self, q, k, gate):
        n = q.shape[1] + k.shape[1] + gate.shape[1]
        rows = torch.zeros((q.shape[0], self.HK.pad8(n)), dtype=self.dtype, device="cuda")
        rows[:, :n] = _dev(np.concatenate([q, k, gate], 1)).to(self.dtype)
        return rows

    def run(self, proj, spans, splits=1, tile=128):
        """spans [(slot, first position, rows)]: rows of proj in order."""
        HK, i32 = self.HK, torch.int32
        n = proj.shape[0]
        slot = np.concatenate([np.full(c, s) for s, _, c in spans]).astype(np.int32)
        pos = np.concatenate([p + np.arange(c) for _, p, c in spans]).astype(np.int32)
        out = torch.full((n, HK.pad8(self.H * self.D)), 7.0, dtype=self.dtype, device="cuda")
        if all(c == 1 for _, _, c in spans):
            ws = HK.window_workspace(n, self.H, self.D, splits, "cuda")
            self.att.decode(proj, n, _dev(slot, i32), _dev(pos, i32), out, splits, ws)
        else:
            starts = np.concatenate([[0], np.cumsum([c for _, _, c in spans])[:-1]])
            tiles = [(a + k, min(tile, c - k)) for a, (_, _, c) in zip(starts, spans) for k in range(0, c, tile)]
            t = (_dev(np.array([x for x, _ in tiles]), i32), _dev(np.array([x for _, x in tiles]), i32), len(tiles))
            self.att.prompt(proj, n, _dev(slot, i32), _dev(pos, i32), out, torch.zeros(n, device="cuda"), t)
        assert (_np(out)[:, self.H * self.D:] == 0).all()
        return _np(out)[:, :self.H * self.D]

    def want(self, proj):
        H, G, D = self.H, self.G, self.D
        p = _np(proj)
        q, k, gate = p[:, :H * D], p[:, H * D:(H + G) * D], p[:, (H + G) * D:(2 * H + G) * D]
        T = q.shape[0]
        o = Z.windowed_attention((Z.rms_norm(q, 1e-5) * self.qn).reshape(T, H, D), (Z.rms_norm(k, 1e-5) * self.kn).reshape(T, G, D),
                                 k.reshape(T, G, D), self.scale, self.slopes, self.window)
        return o.reshape(T, H * D) * Z.sigmoid(gate)

    def tol(self):
        return 2e-5 if self.dtype == torch.float32 else 2e-2        # bf16: queries, weights and results are rounded


SHAPES = [(4, 2, 8, 5), (6, 2, 20, 33), (2, 2, 48, 64), (8, 1, 64, 65), (5, 1, 72, 63), (4, 1, 128, 100), (3, 3, 136, 40),
          (2, 1, 256, 1), (2, 1, 300, 50), (4, 4, 16, None)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,D,window", SHAPES)
def test_attention_prompt_decode_and_portions(dtype, H, G, D, window):
    """A whole prompt; the same in portions (down to one and two tokens) through a ring that wraps; token by token with
    the window in one and in several parts."""
    rng = np.random.default_rng(D)
    T = 150
    q, k, gate = rng.standard_normal((T, H * D)), rng.standard_normal((T, G * D)), rng.standard_normal((T, H * D))
    for how in ("whole", "portions", "decode", "decode split"):
        print(f"attention {dtype} H {H} G {G} D {D} window {window}: {how}", flush=True)
        most = {"whole": T, "portions": 70}.get(how, 1)
        ring = T if window is None else min(T, window - 1 + most)
        a = Attention(dtype, H, G, D, window, 2, ring, seed=D)
        proj = a.project(q, k, gate)
        want = a.want(proj)
        if how == "whole":
            got = a.run(proj, [(1, 0, T)])
        elif how == "portions":
            parts, p = [], 0
            for c in (2, 1, 70, 2, 3, 64, 8):
                parts.append(a.run(proj[p:p + c].contiguous(), [(1, p, c)]))
                p += c
            got = np.concatenate(parts)
        else:
            got = np.concatenate([a.run(proj[t:t + 1].contiguous(), [(1, t, 1)], splits=1 if how == "decode" else 3) for t in range(T)])
        assert _rel(got, want) < a.tol(), how


@pytest.mark.parametrize("dtype", DTYPES)
def test_attention_batch_of_unequal_sequences(dtype):
    rng = np.random.default_rng(3)
    H, G, D, window = 6, 3, 40, 37
    a = Attention(dtype, H, G, D, window, 4, 256, seed=1)
    lens, slots = [1, 200, 64, 129], [2, 0, 3, 1]
    projs = [a.project(*(rng.standard_normal((n, c)) for c in (H * D, G * D, H * D))) for n in lens]
    got = a.run(torch.cat(projs), [(s, 0, n) for s, n in zip(slots, lens)])
    want = np.concatenate([a.want(p) for p in projs])
    assert _rel(got, want) < a.tol()
    # one more token each, in another order, together
    more = [torch.cat([p, a.project(*(rng.standard_normal((1, c)) for c in (H * D, G * D, H * D)))]) for p in projs]
    order = [3, 0, 2, 1]
    got = a.run(torch.cat([more[i][-1:] for i in order]), [(slots[i], lens[i], 1) for i in order], splits=2)
    assert _rel(got, np.concatenate([a.want(more[i])[-1:] for i in order])) < a.tol()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [16, 48, 128])
def test_one_key_stands_out_at_the_edge_of_the_window(dtype, D):
    """A query and one key that are strongly alike: the key is found while it is the window's oldest, and not one position
    later - in a prompt, in a portion that starts there, and decoded; near and at multiples of the ring and tile length."""
    H, G, window, T, scale = 2, 1, 64, 260, 4.0
    rng = np.random.default_rng(D)
    for at in (0, 1, 63, 64, 127, 130):
        q, k, gate = (0.3 * rng.standard_normal((T, c)) for c in (H * D, G * D, H * D))
        mark = rng.standard_normal(D)
        k[at] = 3 * mark
        for i in (at + window - 1, at + window):
            q[i] = np.tile(3 * mark, H)
        a = Attention(dtype, H, G, D, window, 1, window - 1 + T, seed=D, scale=scale)
        a.slopes = a.slopes * 0 + 0.01
        a.att.slopes = _dev(a.slopes)
        proj = a.project(q, k, gate)
        want = a.want(proj)
        seen, gone = at + window - 1, at + window
        assert np.abs(want[seen]).max() > 1.5 * np.abs(want[gone]).max()          # the edge shows in what is expected
        assert _rel(a.run(proj, [(0, 0, T)]), want) < a.tol()
        b = Attention(dtype, H, G, D, window, 1, window - 1 + T, seed=D, scale=scale)
        b.slopes, b.att.slopes = a.slopes, a.att.slopes
        b.run(proj[:seen].contiguous(), [(0, 0, seen)])
        got = b.run(proj[seen:seen + 2].contiguous(), [(0, seen, 2)])
        assert _rel(got, want[seen:seen + 2]) < a.tol()
        c = Attention(dtype, H, G, D, window, 1, window + seen, seed=D, scale=scale)
        c.slopes, c.att.slopes = a.slopes, a.att.slopes
        c.run(proj[:seen].contiguous(), [(0, 0, seen)])
        for t, splits in ((seen, 1), (gone, 2)):
            assert _rel(c.run(proj[t:t + 1].contiguous(), [(0, t, 1)], splits=splits), want[t:t + 1]) < a.tol()


# ---------------------------------------------------------------------------------------------- matrix memory
class Memory:
    def __init__(self, dtype, H, D, E, cap, slots):
        HK, T = _hk()
        self.HK, self.dtype, self.H, self.D, self.E, self.cap = HK, T[dtype], H, D, E, cap
        self.state = HK.mlstm_state(slots, H, D, E, "cuda")

    def project(self, q, k, v):
        H, D, E = self.H, self.D, self.E
        n = 2 * H * D + 2 * H * E
        rows = torch.zeros((q.shape[0], self.HK.pad8(n)), dtype=self.dtype, device="cuda")
        rows[:, :2 * H * D + H * E] = _dev(np.concatenate([q, k, v], 1)).to(self.dtype)
        return rows

    def run(self, proj, gates, spans, chunked):
        i32 = torch.int32
        n = proj.shape[0]
        slot = np.concatenate([np.full(c, s) for s, c in spans]).astype(np.int32)
        counts = np.array([c for _, c in spans])
        starts = np.concatenate([[0], np.cumsum(counts)[:-1]])
        o = torch.full((n, self.H * self.E), 7.0, device="cuda")
        self.HK.mlstm(proj, n, self.H, self.D, self.E, _dev(gates), self.cap, self.state, _dev(slot, i32),
                      (_dev(starts, i32), _dev(counts, i32), len(spans)), int(counts.max()), o, chunked)
        return _np(o).reshape(n, self.H, self.E)

    def want(self, proj, gates):
        H, D, E = self.H, self.D, self.E
        p, T = _np(proj), proj.shape[0]
        i, f = Z.softcap(gates[:, :H], self.cap), Z.log_sigmoid(Z.softcap(gates[:, H:], self.cap))
        return Z.mlstm_recurrence(p[:, :H * D].reshape(T, H, D) * D ** -0.5, p[:, H * D:2 * H * D].reshape(T, H, D),
                                  p[:, 2 * H * D:2 * H * D + H * E].reshape(T, H, E), i, f)


def _gates(rng, T, H, kind):
    i, f = rng.standard_normal((T, H)), rng.standard_normal((T, H))
    if kind == "long":                       # keeps nearly everything
        return np.concatenate([i, 6 + f], 1)
    if kind == "short":                      # forgets at once: log forget gates far below zero
        return np.concatenate([i, -20 + f], 1)
    if kind == "spikes":                     # single tokens that outweigh all others
        i[T // 3::17] += 12
        return np.concatenate([i, 3 + f], 1)
    return np.concatenate([4 * i, 3 * f], 1)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,E", [(3, 16, 32), (2, 24, 40), (1, 40, 8), (2, 64, 100), (2, 100, 64), (1, 256, 96), (1, 300, 33)])
@pytest.mark.parametrize("kind", ["mixed", "long", "short", "spikes"])
def test_mlstm(dtype, H, D, E, kind):
    """Whole, in portions (down to two tokens, at and around multiples of the chunk), token by token, and a batch of
    unequal sequences; the state carried from one to the next."""
    rng = np.random.default_rng(D + E)
    T = 330                                  # chunked: three segments of up to 128 tokens
    m = Memory(dtype, H, D, E, 7.0, 4)
    proj = m.project(*(rng.standard_normal((T, c)) for c in (H * D, H * D, H * E)))
    gates = _gates(rng, T, H, kind)
    want = m.want(proj, gates)

    def close(got, ref):
        # per token and head, against its own size: a token that reads almost nothing is not hidden by one that reads much
        size = np.abs(ref).max(-1, keepdims=True) + 1e-3 * np.abs(want).max()
        return (np.abs(got - ref) / size).max() < (2e-4 if dtype == "float32" else 2e-3)
    for chunked in ((False, True) if dtype == "bfloat16" else (False,)):
        print(f"mlstm {dtype} H {H} D {D} E {E} {kind} chunked {chunked}", flush=True)
        m.state.zero_()
        assert close(m.run(proj, gates, [(1, T)], chunked), want)
        for cuts in ((64, 64, 202), (2, 63, 65, 2, 198), (129, 127, 74), (329, 1)):
            m.state.zero_()
            parts, p = [], 0
            for c in cuts:
                parts.append(m.run(proj[p:p + c].contiguous(), gates[p:p + c], [(2, c)], chunked))
                p += c
            assert close(np.concatenate(parts), want), cuts
        m.state.zero_()
        got = [m.run(proj[:130].contiguous(), gates[:130], [(3, 130)], chunked)]
        got += [m.run(proj[t:t + 1].contiguous(), gates[t:t + 1], [(3, 1)], False) for t in range(130, T)]
        assert close(np.concatenate(got), want)
        m.state.zero_()
        lens, slots = [70, 1, 330, 129], [3, 0, 2, 1]
        got = m.run(torch.cat([proj[:n] for n in lens]), np.concatenate([gates[:n] for n in lens]), list(zip(slots, lens)), chunked)
        assert close(got, np.concatenate([want[:n] for n in lens]))


@pytest.mark.parametrize("dtype", DTYPES)
def test_head_norm_and_gate(dtype):
    HK, T = _hk()
    rng = np.random.default_rng(0)
    for rows, H, E, at in ((1, 3, 20, 8), (9, 2, 128, 0), (5, 1, 7, 3)):
        o, w = rng.standard_normal((rows, H * E)) * 10.0 ** rng.integers(-4, 2, (rows, 1)), rng.standard_normal(H * E)
        proj = _dev(rng.standard_normal((rows, HK.pad8(at + H * E)))).to(T[dtype])
        out = torch.full((rows, HK.pad8(H * E)), 7.0, dtype=T[dtype], device="cuda")
        HK.head_norm_gate(_dev(o), _dev(w), proj, at, out, rows, H, E, 1e-5)
        want = Z.rms_norm(o.reshape(rows, H, E), 1e-5).reshape(rows, -1) * w * Z.sigmoid(_np(proj)[:, at:at + H * E])
        assert _rel(_np(out)[:, :H * E], want) < (3e-6 if dtype == "float32" else 6e-3)
        assert (_np(out)[:, H * E:] == 0).all()


# ---------------------------------------------------------------------------------------------- selection
def test_selection_over_fp32_logits():
    HK, _ = _hk()
    rng = np.random.default_rng(0)
    x = rng.integers(-20, 20, (5, 3001)).astype(np.float32)              # many ties
    x[2, :] = np.nan
    x[3, 100] = np.nan
    ids = torch.zeros(5, dtype=torch.int32, device="cuda")
    HK.argmax(_dev(x), ids)
    clean = np.where(np.isnan(x), -np.inf, x)
    assert ids.cpu().tolist() == [int(r.argmax()) for r in clean[:2]] + [0] + [int(r.argmax()) for r in clean[3:]]
    y = rng.integers(-20, 20, (3, 40000)).astype(np.float32)              # whole vectors, several per thread
    HK.argmax(_dev(y), ids)
    assert ids[:3].cpu().tolist() == [int(r.argmax()) for r in y]
    top = torch.zeros((5, 7), dtype=torch.int32, device="cuda")
    HK.topk(_dev(x), 7, top)
    for r in (0, 1, 3, 4):
        order = sorted(range(x.shape[1]), key=lambda c: (-clean[r, c], c))[:7]
        assert top[r].cpu().tolist() == order
