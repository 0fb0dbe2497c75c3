"""Kernels of latent attention, grouped norm with token shift and the gated epilogues, one by one against oracle/ruperax.py."""
import numpy as np
import pytest
import torch

from oracle import ruperax as R
from poptransformer_amd import _hybrid_lib as H

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


# ---------------------------------------------------------------------------------------------- Linear epilogues
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 4, 7, 16, 33, 64, 100, 300])
def test_linear_bias_gate_and_accumulation(dtype, rows):
    """The residual's update: y += mul * (x W^T + b); and sigmoid(x W^T + b)."""
    HK, T = _hk()
    rng = np.random.default_rng(rows)
    for n, k in ((24, 40), (50, 72), (1160, 136), (640, 1100)):
        print(f"epilogue {dtype} rows {rows} n {n} k {k}", flush=True)
        w = _dev(rng.standard_normal((n, k)) / np.sqrt(k)).to(T[dtype])
        x = torch.zeros((rows, HK.pad8(k)), dtype=T[dtype], device="cuda")
        x[:, :k] = _dev(rng.standard_normal((rows, k))).to(T[dtype])
        bias, mul, y = _dev(rng.standard_normal(n)), _dev(rng.random((rows, n)), T[dtype]), _dev(rng.standard_normal((rows, n)))
        ww = HK.WideWeight(w.float(), T[dtype])
        z = _np(x)[:, :k] @ _np(w).T + _np(bias)
        want = _np(y) + _np(mul) * z
        HK.linear(x, ww, y, rows, ld=n, bias=bias, mul=mul, accumulate=True, workspace=HK.linear_workspace(rows, ww.N, "cuda"))
        assert _rel(_np(y), want) < 1e-5
        out = torch.empty((rows, n), dtype=T[dtype], device="cuda")
        HK.linear(x, ww, out, rows, ld=n, bias=bias, act=H.ACT_SIGMOID)
        assert _rel(_np(out), R.sigmoid(z)) < (1e-5 if dtype == "float32" else 6e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 5, 16, 40, 130])
def test_linears_with_inputs_of_their_own(dtype, rows):
    HK, T = _hk()
    rng = np.random.default_rng(rows)
    for k, sizes in ((48, (30, 16, 100)), (1032, (1032, 700, 1032)), (1032, (1032, 1100, 1150))):
        print(f"group {dtype} rows {rows} k {k}", flush=True)
        calls, want, tail = [], [], torch.empty((rows, 5), device="cuda")
        for i, n in enumerate(sizes):
            w, x = _dev(rng.standard_normal((n, k)) / np.sqrt(k)).to(T[dtype]), _dev(rng.standard_normal((rows, k)), T[dtype])
            ww = HK.WideWeight(w.float(), T[dtype], tail=5 if i == 1 else 0)
            out = torch.full((rows, ww.n_main), 7.0, dtype=T[dtype], device="cuda")
            calls.append((x, ww, out, dict(tail=tail if i == 1 else None, act=H.ACT_SIGMOID if i == 2 else H.ACT_NONE)))
            want.append(_np(x) @ _np(w).T)
        HK.linear_group(rows, *calls)
        tol = 1e-5 if dtype == "float32" else 6e-3
        assert _rel(_np(calls[0][2]), want[0]) < tol
        assert _rel(_np(calls[1][2]), want[1][:, :-5]) < tol and _rel(_np(tail), want[1][:, -5:]) < 1e-5
        assert _rel(_np(calls[2][2]), R.sigmoid(want[2])) < tol


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 6, 16, 50, 140])
def test_swiglu_with_biases(dtype, rows):
    HK, T = _hk()
    from poptransformer_amd import _hybrid_lib as H
    rng = np.random.default_rng(rows)
    for n, k in ((24, 48), (1032, 520)):
        g, u = (_dev(rng.standard_normal((n, k)) * 2 / np.sqrt(k)).to(T[dtype]) for _ in range(2))
        x, bg, bu = _dev(rng.standard_normal((rows, k)), T[dtype]), _dev(rng.standard_normal(n)), _dev(rng.standard_normal(n))
        out = torch.empty((rows, n), dtype=T[dtype], device="cuda")
        HK.linear(x, HK.WideWeight(g.float(), T[dtype]), out, rows, up=HK.WideWeight(u.float(), T[dtype]), pair=H.PAIR_SWIGLU, bias=bg, bias2=bu)
        want = R.silu(_np(x) @ _np(g).T + _np(bg)) * (_np(x) @ _np(u).T + _np(bu))
        assert _rel(_np(out), want) < (1e-5 if dtype == "float32" else 6e-3)


# ---------------------------------------------------------------------------------------------- norm and shift
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,groups", [(36, 3), (75, 5), (75, 1), (130, 26), (1028, 2), (1024, 4), (2048, 1), (4096, 4), (5120, 2), (8448, 3)])
def test_grouped_norm_and_token_shift(dtype, width, groups):
    """Sequences of unequal length in one pass; one of them goes on where an earlier pass left it, one is in a used slot."""
    HK, T = _hk()
    rng = np.random.default_rng(width)
    tol = 5e-6 if dtype == "float32" else 6e-3
    w1, w2, mix = (rng.standard_normal(width) for _ in range(3))
    state = torch.full((8, width), 9.0, device="cuda")
    many = 2100 if width <= 2048 else 300                        # (a workgroup walks through several rows)
    seqs = {s: rng.standard_normal((many + 320, width)) for s in (5, 0, 3)}
    want = {s: R.group_rms_norm(x, w1, groups, 1e-5) for s, x in seqs.items()}
    shifted = {s: R.token_shift(h, mix) for s, h in want.items()}
    at = dict.fromkeys(seqs, 0)
    for counts in ({5: 1, 0: 1, 3: 1}, {5: 7, 3: many}, {0: 2, 5: 3}, {5: 1, 3: 1}, {3: 2}, {0: 9, 5: 4, 3: 5}, {0: 300, 5: 299}):
        print(f"shift {dtype} width {width} counts {counts}", flush=True)
        rows = sum(counts.values())
        x = np.concatenate([seqs[s][at[s]:at[s] + c] for s, c in counts.items()])
        slot = np.repeat(list(counts), list(counts.values()))
        pos = np.concatenate([np.arange(at[s], at[s] + c) for s, c in counts.items()])
        last, first = np.full(rows, -1), 0
        for c in counts.values():
            last[first] = first + c - 1
            first += c
        ld = HK.pad8(width)
        h1, h2, hm = (torch.full((rows, ld), 7.0, dtype=T[dtype], device="cuda") for _ in range(3))
        single = all(c == 1 for c in counts.values())
        HK.shift_norm(_dev(x), rows, groups, 1e-5, _dev(w1), h1, _dev(w2), h2, _dev(mix), hm, state, _dev(slot, torch.int32),
                      None if single else _dev(last, torch.int32), _dev(pos, torch.int32), 4000)
        sel = [(s, slice(at[s], at[s] + c)) for s, c in counts.items()]
        assert _rel(_np(h1)[:, :width], np.concatenate([want[s][k] for s, k in sel])) < tol
        assert _rel(_np(h2)[:, :width], np.concatenate([R.group_rms_norm(seqs[s][k], w2, groups, 1e-5) for s, k in sel])) < tol
        assert _rel(_np(hm)[:, :width], np.concatenate([shifted[s][k] for s, k in sel])) < tol
        assert all((_np(h)[:, width:] == 0).all() for h in (h1, h2, hm))
        for s, c in counts.items():
            at[s] += c
            assert _rel(_np(state[s]), want[s][at[s] - 1]) < 5e-6
    assert (state[[1, 2, 4, 6, 7]] == 9).all()


@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding_with_positions_and_gathered_rows(dtype):
    HK, T = _hk()
    rng = np.random.default_rng(0)
    d, V, P, n = 60, 50, 40, 30
    table, places = _dev(rng.standard_normal((V, d)), T[dtype]), _dev(rng.standard_normal((P, d)), T[dtype])
    w, mix = rng.standard_normal(d), rng.standard_normal(d)
    ids, state = rng.integers(0, V, n), torch.full((1, d), 5.0, device="cuda")
    x = torch.full((n, d), 7.0, device="cuda")
    h1, hm = (torch.empty((n, 64), dtype=T[dtype], device="cuda") for _ in range(2))
    last = np.full(n, -1)
    last[0] = n - 1
    zero = torch.zeros(n, dtype=torch.int32, device="cuda")
    HK.shift_norm(x, n, 2, 1e-5, _dev(w), h1, shift=_dev(mix), hm=hm, state=state, slot=zero, last=_dev(last, torch.int32),
                  pos=_dev(np.arange(n), torch.int32), positions=P, table=table, pos_table=places, embed_scale=2.5, ids=_dev(ids, torch.int32))
    want = _np(table)[ids] * 2.5 + _np(places)[:n]
    h = R.group_rms_norm(want, w, 2, 1e-5)
    tol = 5e-6 if dtype == "float32" else 6e-3
    assert _rel(_np(x), want) < 1e-6 and _rel(_np(h1)[:, :d], h) < tol and _rel(_np(hm)[:, :d], R.token_shift(h, mix)) < tol
    pick = np.array([29, 3, 3, 0])
    out = torch.empty((4, 64), dtype=T[dtype], device="cuda")
    HK.shift_norm(x, 4, 2, 1e-5, _dev(w), out, gather=_dev(pick, torch.int32))
    assert _rel(_np(out)[:, :d], h[pick]) < tol
    # a decode iteration: ids and position from the loop's counter, which may run past the table
    grid = _dev(np.arange(3 * 45).reshape(3, 45) % V, torch.int32)
    for step in (0, 12, 44):
        pos_out = torch.full((3,), -1, dtype=torch.int32, device="cuda")
        x3, h3 = torch.empty((3, d), device="cuda"), torch.empty((3, 64), dtype=T[dtype], device="cuda")
        HK.shift_norm(x3, 3, 2, 1e-5, _dev(w), h3, positions=P, table=table, pos_table=places, embed_scale=2.5, ids=grid,
                      ids_index=_dev(np.array(step), torch.int32), pos_out=pos_out)
        p = min(step, P - 1)
        assert _rel(_np(x3), _np(table)[_np(grid)[:, step].astype(int)] * 2.5 + _np(places)[p]) < 1e-6 and (pos_out == p).all()


# ---------------------------------------------------------------------------------------------- latent attention
class Case:
    """One layer's attention over sequences in slots of a ring: inputs, and the oracle's attention over everything each
    sequence holds."""

    def __init__(self, dtype, heads, dim, rot, vdim, kv_rank, window, ring_len, lens, seed=0, plant=()):
        from poptransformer_amd.engine.hybrid import LatentMixer, Rotation
        self.HK, self.T = _hk()
        T = self.dtype = self.T[dtype]
        rng = np.random.default_rng(seed)
        self.m = m = LatentMixer(heads, dim, rot, vdim, 24, kv_rank, (dim + rot) ** -0.5 * 2, window, Rotation(20.0, rot))
        _, D, P, E, Rp, _, _ = m.sizes
        self.lens, self.ring_len, self.slots = lens, ring_len, [2 * i + 1 for i in range(len(lens))]
        total = max(lens)
        self.cs = _dev(m.angles(total))
        pairs = m.pairs()

        def rounded(a):
            return _np(_dev(a, T))
        self.uk, self.uv = (rounded(rng.standard_normal((heads, n, kv_rank)) / np.sqrt(kv_rank)) for n in (dim, vdim))
        self.gate = rng.standard_normal((len(lens), total, heads))
        self.q = rounded(rng.standard_normal((len(lens), total, heads, dim + rot)))
        self.c = rounded(rng.standard_normal((len(lens), total, kv_rank)))
        k_rot = rounded(R.rotate_half(rng.standard_normal((len(lens), total, rot)).swapaxes(0, 1), 20.0, rot).swapaxes(0, 1))
        for s, i, j in plant:                    # query i of sequence s finds key j with a score that outweighs all others
            q_rot = R.rotate_half(self.q[s][..., dim:], 20.0, rot)[i]
            k_rot[s, j] = rounded(np.linalg.pinv(q_rot) @ np.full(heads, 100.0))
        q_rot = np.stack([R.rotate_half(x[..., dim:], 20.0, rot) for x in self.q])
        self.want = []
        for s in range(len(lens)):
            k = np.concatenate([np.einsum("tr,hdr->thd", self.c[s], self.uk), np.repeat(k_rot[s][:, None], heads, 1)], -1)
            o = R.sliding_softmax_attention(np.concatenate([self.q[s][..., :dim], q_rot[s]], -1), k,
                                            np.einsum("tr,her->the", self.c[s], self.uv), m.scale, window)
            self.want.append(o * R.sigmoid(self.gate[s])[..., None])
        # as stored: padded, the two of a rotated pair side by side
        self.q_stored = np.zeros((len(lens), total, heads, D + P))
        self.q_stored[..., :dim], self.q_stored[..., D:D + rot] = self.q[..., :dim], self.q[..., dim:][..., pairs]
        self.rows = np.zeros((len(lens), total, Rp + P))
        self.rows[..., :kv_rank], self.rows[..., Rp:Rp + rot] = self.c, k_rot[..., pairs]
        uk, uv = np.zeros((heads, D, Rp)), np.zeros((heads, E, Rp))
        uk[:, :dim, :kv_rank], uv[:, :vdim, :kv_rank] = self.uk, self.uv
        self.uk_t, self.uv_s = _dev(uk.transpose(0, 2, 1), T), _dev(uv, T)
        self.kv_weight = self.HK.WideWeight(_dev(np.concatenate([uk.reshape(-1, Rp), uv.reshape(-1, Rp)])), T)

    def run(self, portions, absorbed, splits=1):
        """portions [(sequence, first position, rows)] -> (got, wanted) [rows, heads, vdim]"""
        m, HK = self.m, self.HK
        H, D, P, E, Rp = m.sizes[:5]
        ring = torch.full((2 * len(self.lens) + 1, self.ring_len, Rp + P), 3.0, dtype=self.dtype, device="cuda")
        for s, p0, n in portions:                # what a sequence has left behind by then, newest rows over older ones
            for p in range(max(0, p0 + n - self.ring_len), p0 + n):
                ring[self.slots[s], p % self.ring_len] = _dev(self.rows[s, p], self.dtype)
        sel = [(s, slice(p0, p0 + n)) for s, p0, n in portions]
        rows = sum(n for _, _, n in portions)
        slot = _dev(np.concatenate([np.full(n, self.slots[s]) for s, _, n in portions]), torch.int32)
        pos = _dev(np.concatenate([np.arange(p0, p0 + n) for _, p0, n in portions]), torch.int32)
        q = _dev(np.concatenate([self.q_stored[s][k] for s, k in sel]), self.dtype)
        gate = _dev(np.concatenate([self.gate[s][k] for s, k in sel]))
        out = torch.full((rows, H * E), 7.0, dtype=self.dtype, device="cuda")
        att = HK.LatentAttention(m.sizes, m.scale, m.window, 1e-5, torch.ones(m.q_rank, device="cuda"), None, self.cs, ring, rows, slot, pos)
        if absorbed:
            att.absorbed(q, self.uk_t, torch.empty((rows * H, Rp + P), dtype=self.dtype, device="cuda"), splits,
                         torch.full((rows * H * splits, Rp), float("nan"), device="cuda"), torch.empty((rows * H * splits, 2), device="cuda"),
                         self.uv_s, gate, out)
        else:
            ks, kp, tr, tc, tk, at, r = [], [], [], [], [], 0, 0
            for s, p0, n in portions:
                first = max(0, p0 - m.window + 1) if m.window else 0
                ks.append(np.full(p0 + n - first, self.slots[s]))
                kp.append(np.arange(first, p0 + n))
                for k in range(0, n, 128):
                    tr.append(r + k)
                    tc.append(min(128, n - k))
                    tk.append(at - first)
                at += p0 + n - first
                r += n
            keys = [_dev(np.concatenate(a), torch.int32) for a in (ks, kp)]
            bufs = [torch.empty((at, c), dtype=self.dtype, device="cuda") for c in (Rp, P, self.kv_weight.n_main)]
            att.over_heads(q, keys, bufs[0], bufs[1], self.kv_weight, bufs[2], [_dev(np.array(a), torch.int32) for a in (tr, tc, tk)], gate, out)
        got = _np(out).reshape(rows, H, E)
        assert (got[..., m.vdim:] == 0).all()
        return got[..., :m.vdim], np.concatenate([self.want[s][k] for s, k in sel])


SIZES = [(3, 20, 6, 28, 44), (21, 9, 10, 17, 70), (16, 128, 64, 128, 512), (5, 72, 24, 88, 200), (2, 100, 64, 256, 800), (1, 180, 60, 16, 64)]


@pytest.mark.parametrize("dtype,absorbed", [("float32", True), ("bfloat16", True), ("bfloat16", False)])
@pytest.mark.parametrize("sizes", SIZES, ids=lambda s: "-".join(map(str, s)))
def test_latent_attention(sizes, dtype, absorbed):
    """Rows of several sequences at once, rings that wrap, windows of one token up to all of them, windows in parts."""
    lens = (300, 3, 131)
    for window, ring_len in ((1, 160), (63, 256), (64, 256), (65, 256), (None, 320)):
        case = Case(dtype, *sizes, window, ring_len, lens, seed=window or 0)
        for portions in ([(0, 0, 150), (1, 0, 3), (2, 0, 131)], [(0, 150, 150), (1, 2, 1), (2, 129, 2)], [(0, 299, 1), (2, 130, 1)],
                         [(0, 63, 1), (1, 0, 1), (2, 64, 1)]):
            for splits in ((1, 3) if absorbed else (1,)):
                print(f"latent {sizes} {dtype} absorbed {absorbed} window {window} {portions} splits {splits}", flush=True)
                got, want = case.run(portions, absorbed, splits)
                assert _rel(got, want) < (2e-5 if dtype == "float32" else 1.5e-2)


def test_latents_and_sizes_beyond_the_matrix_unit():
    """bf16 on the vector unit."""
    for sizes in ((2, 40, 160, 24, 100), (1, 16, 8, 16, 1200)):
        got, want = Case("bfloat16", *sizes, 30, 128, (90,)).run([(0, 0, 90)], True, 2)
        assert _rel(got, want) < 1.5e-2
    HK, T = _hk()
    assert HK.latent_tiles_fit(torch.bfloat16, 192, 64, 256) and not HK.latent_tiles_fit(torch.bfloat16, 224, 64, 64)
    assert not HK.latent_tiles_fit(torch.float32, 32, 32, 32)
    with pytest.raises(ValueError):
        Case("bfloat16", 1, 250, 64, 16, 32, 30, 128, (90,)).run([(0, 0, 90)], False)


@pytest.mark.parametrize("dtype,absorbed", [("float32", True), ("bfloat16", True), ("bfloat16", False)])
@pytest.mark.parametrize("window", [2, 64, 65, 100])
def test_one_key_at_the_edge_of_the_window(window, dtype, absorbed):
    """A single key outweighs all others: just inside the window it is the result, just outside it is nothing."""
    for i in (window, 127, 128, 191):
        inside, outside = i - window + 1, i - window
        for j in (inside, outside):
            if j < 0:
                continue
            case = Case(dtype, 4, 32, 32, 32, 64, window, 192 + 128, (192,), seed=i, plant=((0, i, j),))
            for portion in ((0, i, 1), (0, max(0, i - 30), min(i, 30) + 1)):
                print(f"edge {dtype} absorbed {absorbed} window {window} query {i} key {j} {portion}", flush=True)
                got, want = case.run([portion], absorbed, 2 if absorbed else 1)
                assert _rel(got, want) < (1e-4 if dtype == "float32" else 3e-2)
                value = np.einsum("r,her->he", case.c[0, j], case.uv) * R.sigmoid(case.gate[0, i])[:, None]
                assert (np.abs(want[-1] - value).max() < 0.05 * np.abs(value).max()) == (j == inside)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("own", [True, False])
def test_latent_norms_and_cache_entries(dtype, own):
    from poptransformer_amd.engine.hybrid import LatentMixer, Rotation
    HK, T = _hk()
    rng = np.random.default_rng(0)
    for q_rank, kv_rank, rot in ((30, 44, 6), (300, 512, 64), (9, 32, 32)):
        m = LatentMixer(2, 16, rot, 16, q_rank, kv_rank, 1.0, 10, Rotation(7.0, rot))
        _, D, P, E, Rp, _, _ = m.sizes
        Qp, pairs, n, slots, ring_len = HK.pad8(q_rank), m.pairs(), 40, 3, 64
        cq, c, k = (rng.standard_normal((n, w)) for w in (q_rank, kv_rank, rot))
        proj = np.zeros((n, Qp + (Rp + P if own else 0)))
        proj[:, :q_rank] = cq
        if own:
            proj[:, Qp:Qp + kv_rank], proj[:, Qp + Rp:Qp + Rp + rot] = c, k[:, pairs]
        proj = _dev(proj, T[dtype])
        wq, wc = rng.standard_normal(q_rank), rng.standard_normal(kv_rank)
        ring = torch.full((slots, ring_len, Rp + P), 7.0, dtype=T[dtype], device="cuda")
        slot, pos = rng.integers(0, slots, n), rng.permutation(600)[:n]
        pos = pos - pos % ring_len + np.arange(n)                # rows of their own, far positions
        cs = _dev(m.angles(700))
        out = torch.full((n, Qp), 7.0, dtype=T[dtype], device="cuda")
        att = HK.LatentAttention(m.sizes, 1.0, 10, 1e-5, _dev(wq), _dev(wc) if own else None, cs, ring, n, _dev(slot, torch.int32),
                                 _dev(pos, torch.int32))
        att.append(proj, out)
        tol = 1e-5 if dtype == "float32" else 6e-3
        stored = _np(proj)
        assert _rel(_np(out)[:, :q_rank], R.rms_norm(stored[:, :q_rank], wq, 1e-5)) < tol and (_np(out)[:, q_rank:] == 0).all()
        got = _np(ring)[slot, pos % ring_len]
        if not own:
            assert (_np(ring) == 7).all()
            continue
        full = np.zeros((700, rot))
        back = np.argsort(pairs)
        full[pos] = stored[:, Qp + Rp:Qp + Rp + rot][:, back]
        assert _rel(got[:, :kv_rank], R.rms_norm(stored[:, Qp:Qp + kv_rank], wc, 1e-5)) < tol
        assert _rel(got[:, Rp:Rp + rot][:, back], R.rotate_half(full, 7.0, rot)[pos]) < tol
        assert (got[:, kv_rank:Rp] == 0).all() and (got[:, Rp + rot:] == 0).all()
        used = np.zeros((slots, ring_len), bool)
        used[slot, pos % ring_len] = True
        assert (_np(ring)[~used] == 7).all()
