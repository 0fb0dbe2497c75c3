"""Kernels of short convolutions, the state-space recurrence, distance penalties, corrected routing and the end of a layer whose result
is averaged over the depths, one by one against oracle/sabolorn.py."""
import numpy as np
import pytest
import torch

from oracle import sabolorn as S
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


class Pass:
    """Rows of a pass: `counts` {slot: rows} after `at` {slot: rows so far}."""

    def __init__(self, counts, at):
        sel = [(s, np.arange(at[s], at[s] + c)) for s, c in counts.items()]
        n = sum(counts.values())
        first = np.concatenate([[0], np.cumsum(list(counts.values()))[:-1]])
        last = np.full(n, -1)
        last[first] = first + np.array(list(counts.values())) - 1
        tiles = [(f + k, min(128, c - k)) for f, c in zip(first, counts.values()) for k in range(0, c, 128)]
        i32 = lambda a: _dev(np.asarray(a), torch.int32)
        self.n, self.sel, self.longest = n, sel, max(counts.values())
        self.slot, self.pos, self.last = i32(np.repeat(list(counts), list(counts.values()))), i32(np.concatenate([p for _, p in sel])), i32(last)
        self.tiles = (i32([t[0] for t in tiles]), i32([t[1] for t in tiles]), len(tiles))
        self.seqs = (i32(first), i32(list(counts.values())), len(counts))

    def rows(self, d):
        return np.concatenate([d[s][p] for s, p in self.sel])


# ---------------------------------------------------------------------------------------------- Linear epilogues
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows", [1, 5, 16, 33, 100, 300])
def test_linear_activations(dtype, rows):
    """gelu(x W^T) * e, and relu(x W^T)^2, the second beside another weight."""
    HK, T = _hk()
    rng = np.random.default_rng(rows)
    for n, k in ((24, 40), (50, 1032), (1160, 136)):
        print(f"activations {dtype} rows {rows} n {n} k {k}", flush=True)
        w, w2 = (_dev(rng.standard_normal((n, k)) * 1.5 / np.sqrt(k)).to(T[dtype]) for _ in range(2))
        x = torch.zeros((rows, HK.pad8(k)), dtype=T[dtype], device="cuda")
        x[:, :k] = _dev(rng.standard_normal((rows, k)))
        ld = HK.pad8(n)
        mul, out, out2 = _dev(rng.standard_normal((rows, ld)), T[dtype]), *(torch.full((rows, ld), 7.0, dtype=T[dtype], device="cuda") for _ in range(2))
        ww, ww2 = (HK.WideWeight(t.float(), T[dtype], main_to=ld) for t in (w, w2))
        z, z2 = (_np(x)[:, :k] @ _np(t).T for t in (w, w2))
        HK.linear(x, ww, out, rows, act=H.ACT_GELU_TANH, mul=mul)
        tol = 1e-5 if dtype == "float32" else 6e-3
        assert _rel(_np(out)[:, :n], S.gelu_tanh(z) * _np(mul)[:, :n]) < tol and (_np(out)[:, n:] == 0).all()
        HK.linear_group(rows, (x, ww, out, {}), (x, ww2, out2, dict(act=H.ACT_RELU_SQUARE)))
        assert _rel(_np(out)[:, :n], z) < tol and _rel(_np(out2)[:, :n], np.maximum(z2, 0) ** 2) < tol
    with pytest.raises(ValueError):
        HK.linear(x, ww, out, rows, act=4)


# ---------------------------------------------------------------------------------------------- short convolutions
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps,channels,bias", [(4, 48, True), (1, 8, False), (2, 1040, False), (3, 520, True), (6, 16, True), (17, 24, False), (40, 8, True)])
def test_short_convolution_in_portions(dtype, taps, channels, bias):
    """Portions of any size, down to single rows beside long ones; columns beside the convolved ones; slots used again."""
    HK, T = _hk()
    rng = np.random.default_rng(taps)
    lens = {0: 300, 2: 420}
    u = {s: _np(_dev(rng.standard_normal((n, channels)), T[dtype])) for s, n in lens.items()}
    w, b = rng.standard_normal((channels, taps)), rng.standard_normal(channels) if bias else None
    want = {s: S.short_convolution(x, w, b) for s, x in u.items()}
    conv = HK.ShortConv(_dev(w.T), _dev(b) if bias else None, silu=bias)
    ring = torch.full((3, taps, channels), float("nan"), dtype=T[dtype], device="cuda")
    at = {0: 0, 2: 0}
    for counts in ({2: 1, 0: 1}, {0: 130}, {2: 2, 0: 2}, {0: 1}, {2: 260, 0: 17}, {2: 1}, {2: 1, 0: 3}, {2: 16}, {2: 3, 0: 146}, {2: 120}):
        print(f"conv {dtype} taps {taps} channels {channels} {counts}", flush=True)
        p = Pass(counts, at)
        x = torch.full((p.n, channels + 24), float("nan"), dtype=T[dtype], device="cuda")
        x[:, 16:16 + channels] = _dev(p.rows(u))
        y = torch.full((p.n, channels + 8), 7.0, dtype=T[dtype], device="cuda")
        conv(x, 16, y, ring, p.n, p.slot, p.pos, p.last, p.tiles)
        z = p.rows(want)
        assert _rel(_np(y)[:, :channels], S.silu(z) if bias else z) < (5e-6 if dtype == "float32" else 6e-3) and (_np(y)[:, channels:] == 7).all()
        for s, c in counts.items():
            at[s] += c


def test_short_convolution_checks_its_arguments():
    HK, _ = _hk()
    conv = HK.ShortConv(torch.zeros((4, 16), device="cuda"))
    p, x = Pass({0: 3}, {0: 0}), torch.zeros((3, 16), device="cuda")
    for ring in (torch.zeros((1, 3, 16), device="cuda"), torch.zeros((1, 4, 24), device="cuda")):
        with pytest.raises(ValueError):
            conv(x, 0, x.clone(), ring, 3, p.slot, p.pos, p.last, p.tiles)
    ring = torch.zeros((1, 4, 16), device="cuda")
    for bad in (lambda: conv(x, 8, x.clone(), ring, 3, p.slot, p.pos, p.last, p.tiles), lambda: conv(x, 0, x, ring, 3, p.slot, p.pos, p.last, p.tiles)):
        with pytest.raises(ValueError):
            bad()


# ---------------------------------------------------------------------------------------------- state space
class _Memory:
    """One layer's recurrence over given projections of some sequences, beside the oracle's."""

    def __init__(self, dtype, heads, groups, dim, vdim, lens, seed=0, taps=4, rate=(-3.0, 0.5), step=0.2):
        HK, T = _hk()
        self.HK, self.dtype, self.sizes = HK, T[dtype], (heads, groups, dim, vdim)
        rng = np.random.default_rng(seed)
        n, C = heads * vdim, heads * vdim + 2 * groups * dim
        round_ = lambda a: _np(_dev(a, self.dtype))
        self.w, self.b = rng.standard_normal((C, taps)) * 0.5, rng.standard_normal(C) * 0.3
        self.dt_bias, self.a_log, self.skip = np.log(np.expm1(rng.uniform(0.2, 1, heads) * step)), rng.uniform(*rate, heads), rng.standard_normal(heads)
        self.u, self.dt, self.conv, self.want, self.at = {}, {}, {}, {}, dict.fromkeys(lens, 0)
        for s, T_ in lens.items():
            self.u[s], self.dt[s] = round_(rng.standard_normal((T_, C))), rng.standard_normal((T_, heads))
            c = self.conv[s] = round_(S.silu(S.short_convolution(self.u[s], self.w, self.b)))
            x, bb, cc = c[:, :n].reshape(T_, heads, vdim), c[:, n:n + groups * dim].reshape(T_, groups, dim), c[:, n + groups * dim:].reshape(T_, groups, dim)
            self.want[s] = S.state_space(x, bb, cc, S.softplus(self.dt[s] + self.dt_bias), self.a_log, self.skip).reshape(T_, n)
        slots = max(lens) + 1
        self.state = HK.ssd_state(slots, heads, dim, vdim, "cuda")
        self.short = HK.ShortConv(_dev(self.w.T), _dev(self.b), silu=True)
        self.ring = torch.full((slots, taps, C), float("nan"), dtype=self.dtype, device="cuda")

    def run(self, counts, chunked):
        """The next tokens as one pass, through the convolution's launch, or within the recurrence's where all counts are 1."""
        heads, groups, dim, vdim = self.sizes
        p = Pass(counts, self.at)
        x = torch.full((p.n, 8 + self.w.shape[0]), float("nan"), dtype=self.dtype, device="cuda")
        x[:, 8:] = _dev(p.rows(self.u))
        x_at, conv = 8, (self.short, self.ring)
        if p.longest > 1:
            y = torch.empty((p.n, self.w.shape[0]), dtype=self.dtype, device="cuda")
            self.short(x, 8, y, self.ring, p.n, p.slot, p.pos, p.last, p.tiles)
            x, x_at, conv = y, 0, None
        out = torch.full((p.n, heads * vdim), 7.0, device="cuda")
        constants = [_dev(t) for t in (self.dt_bias, self.a_log, self.skip)]
        self.HK.ssd(x, x_at, p.n, heads, groups, dim, vdim, _dev(p.rows(self.dt)), constants, self.state, p.slot, p.seqs, p.longest, out, chunked,
                    pos=p.pos, conv=conv)
        for s, c in counts.items():
            self.at[s] += c
        want = p.rows(self.want)
        # (bf16: a rounding of a convolved value that falls the other way beside the oracle's)
        err = np.abs(_np(out) - want).max(1) / max(np.abs(want).max(), 1e-3)
        assert err.max() < (2e-5 if self.dtype == torch.float32 else 8e-3), (counts, chunked, int(err.argmax()), err.max())


SSD_SIZES = [(4, 2, 24, 24), (3, 3, 8, 16), (2, 1, 128, 64), (5, 1, 40, 104), (2, 2, 256, 40), (1, 1, 64, 8), (8, 2, 120, 32)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", SSD_SIZES, ids=lambda s: "-".join(map(str, s)))
def test_state_space_in_portions_and_decoding(sizes, dtype):
    """Sequences of unequal length in one pass, portions down to two tokens around single ones, with and without chunks."""
    layer = _Memory(dtype, *sizes, {2: 500, 0: 300})
    for counts, chunked in (({2: 1, 0: 1}, False), ({2: 64, 0: 2}, True), ({2: 1}, False), ({0: 65, 2: 63}, True), ({2: 2, 0: 3}, False), ({2: 1, 0: 1}, False),
                            ({0: 150, 2: 8}, True), ({2: 2}, True), ({2: 1, 0: 1}, False), ({2: 300, 0: 1}, True), ({2: 5, 0: 1}, False), ({2: 1}, False)):
        print(f"ssd {sizes} {dtype} {counts} chunked {chunked}", flush=True)
        layer.run(counts, chunked)


def test_state_space_of_long_portions_in_segments():
    """Sequences long enough to be cut into segments that run side by side, of unequal lengths."""
    for sizes, lens in (((2, 1, 64, 64), {0: 2000, 1: 700}), ((3, 3, 128, 40), {1: 1500})):
        layer = _Memory("bfloat16", *sizes, lens, seed=3, rate=(-6.0, -1.0))
        for counts in ([{0: 1300, 1: 2}, {0: 699, 1: 690}, {0: 1, 1: 1}] if len(lens) == 2 else [{1: 1}, {1: 1400}, {1: 99}]):
            print(f"ssd segments {sizes} {counts}", flush=True)
            layer.run(counts, True)


@pytest.mark.parametrize("rate,step", [((-9.0, -7.0), 0.05), ((1.5, 3.0), 2.0)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_states_that_hardly_fade_and_that_fade_at_once(dtype, rate, step):
    layer = _Memory(dtype, 3, 1, 32, 16, {0: 700}, seed=4, rate=rate, step=step)
    for counts, chunked in (({0: 260}, True), ({0: 1}, False), ({0: 7}, False), ({0: 300}, True), ({0: 1}, False)):
        layer.run(counts, chunked)


def test_a_larger_state_than_the_chunks_take():
    layer = _Memory("bfloat16", 2, 1, 320, 16, {0: 60}, seed=5)
    layer.run({0: 40}, True)
    layer.run({0: 1}, False)


def test_state_space_checks_its_arguments():
    layer = _Memory("float32", 2, 1, 16, 16, {0: 8})
    layer.state = layer.state[:, :-1].contiguous()
    with pytest.raises(ValueError):
        layer.run({0: 2}, False)
    layer = _Memory("float32", 2, 1, 512 + 8, 16, {0: 4})
    with pytest.raises(ValueError):
        layer.run({0: 1}, False)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,vdim,parts", [(4, 20, 2), (3, 10, 2), (2, 64, 1), (5, 7, 5), (6, 24, 4), (1, 6, 3), (32, 64, 1), (80, 128, 8), (3, 5, 15), (300, 64, 2)])
def test_gated_norm(dtype, heads, vdim, parts):
    HK, T = _hk()
    rng = np.random.default_rng(heads)
    for rows in (1, 3, 70):
        E = HK.pad8(vdim)
        y, z, w = rng.standard_normal((rows, heads, E)), rng.standard_normal((rows, heads, E)), np.zeros((heads, E))
        y[..., vdim:], z[..., vdim:] = 0, 0
        w[:, :vdim] = rng.standard_normal((heads, vdim))
        z = _np(_dev(z, T[dtype]))
        rows_z = torch.full((rows, heads * E + 16), 5.0, dtype=T[dtype], device="cuda")
        rows_z[:, :heads * E] = _dev(z.reshape(rows, -1))
        out = torch.full((rows, heads * E), 7.0, dtype=T[dtype], device="cuda")
        HK.gated_norm(_dev(y.reshape(rows, -1)), rows_z, _dev(w.reshape(-1)), out, rows, heads, E, vdim, parts, 1e-3)
        true = lambda a: a[..., :vdim].reshape(*a.shape[:-2], -1)
        got = _np(out).reshape(rows, heads, E)
        want = S.gated_group_norm(true(y), true(z), true(w), parts, 1e-3)
        assert _rel(true(got), want) < (1e-5 if dtype == "float32" else 6e-3) and (got[..., vdim:] == 0).all(), rows


# ---------------------------------------------------------------------------------------------- attention
class _Heads:
    """One layer's attention over given projections of some sequences: convolutions and the penalty of the distance."""

    def __init__(self, dtype, heads, kv_heads, dim, vdim, taps, lens, seed=0, standout=(), far=None, max_len=400):
        from poptransformer_amd.engine.hybrid import HeadMixer
        HK, T = _hk()
        self.HK, self.dtype = HK, T[dtype]
        m = self.m = HeadMixer(heads, kv_heads, dim, vdim, 0.5 * dim ** -0.5 * 3, biases="qkv", norms=False, far=True, taps=taps)
        rng = np.random.default_rng(seed)
        round_ = lambda a: _np(_dev(a, self.dtype))
        self.r = far or (rng.uniform(0.1, 1.5, heads), rng.uniform(0.02, 0.5, heads))
        self.parts = [(heads, dim, m.stored_dim), (kv_heads, dim, m.stored_dim), (kv_heads, vdim, m.stored_vdim)]
        self.w = [rng.standard_normal((h * n, taps)) * 0.4 + (np.arange(taps) == taps - 1) * 0.7 for h, n, _ in self.parts]
        self.u, self.want, self.at = {}, {}, dict.fromkeys(lens, 0)
        for s, n in lens.items():
            u = [round_(rng.standard_normal((n, h * c))) for h, c, _ in self.parts]
            for i, j in standout:                                     # (one tap: what is planted is what is scored)
                if i < n:
                    k = round_(rng.standard_normal((kv_heads, dim)) * 2.5)
                    u[1][j], u[0][i] = k.reshape(-1), np.repeat(k, heads // kv_heads, 0).reshape(-1)
            self.u[s] = u
            q, k, v = (round_(S.short_convolution(a, w)).reshape(n, h, c) for a, w, (h, c, _) in zip(u, self.w, self.parts))
            self.want[s] = S.softmax_attention(q, k, v, m.scale, S.log_distance(*self.r))
        slots = max(lens) + 1
        n = (max_len + 63) // 64 * 64
        self.keys = torch.full((slots, kv_heads, 1, n, m.stored_dim), 9.0, dtype=self.dtype, device="cuda")
        self.values = torch.full((slots, kv_heads, n, m.stored_vdim), 9.0, dtype=self.dtype, device="cuda")
        weights = np.concatenate([self._stored(w.reshape(h, c, taps).transpose(2, 0, 1), c, st) for w, (h, c, st) in zip(self.w, self.parts)], 1)
        self.conv = HK.ShortConv(_dev(weights))
        self.ring = torch.full((slots, taps, m.conv_channels), float("nan"), dtype=self.dtype, device="cuda")

    def _stored(self, a, size, stored):
        out = np.zeros((*a.shape[:-1], stored))
        out[..., :size] = a
        return out.reshape(a.shape[0], -1)

    def run(self, counts, splits=None):
        HK, m = self.HK, self.m
        p = Pass(counts, self.at)
        rows = [np.concatenate([self.u[s][k][q] for s, q in p.sel]) for k in range(3)]
        proj = _dev(np.concatenate([self._stored(a.reshape(p.n, h, c), c, st) for a, (h, c, st) in zip(rows, self.parts)], 1), self.dtype)
        if splits is None:
            raw, proj = proj, torch.empty_like(proj)
            self.conv(raw, 0, proj, self.ring, p.n, p.slot, p.pos, p.last, p.tiles)
        out, far = torch.full((p.n, m.heads * m.stored_vdim), 7.0, dtype=self.dtype, device="cuda"), tuple(_dev(t) for t in self.r)
        att = HK.HeadAttention(m, 1e-5, None, None, None, None, 0.0, self.keys, self.values, proj, p.n, p.slot, p.pos, None, out, far)
        if splits is None:
            att.prompt(p.tiles)
        else:
            att.decode(splits, HK.head_workspace(p.n, m, splits, "cuda") if splits > 1 else None, (self.conv, self.ring))
        for s, c in counts.items():
            self.at[s] += c
        got = _np(out).reshape(p.n, m.heads, m.stored_vdim)
        assert (got[..., m.vdim:] == 0).all()
        want = p.rows(self.want)
        err = np.abs(got[..., :m.vdim] - want).max((1, 2)) / np.abs(want).max()
        assert err.max() < (2e-5 if self.dtype == torch.float32 else 2.5e-2), (counts, splits, int(err.argmax()), err.max())


HEAD_SIZES = [(6, 2, 16, 24, 4), (3, 1, 10, 7, 2), (2, 2, 64, 64, 1), (8, 1, 128, 128, 4), (5, 5, 40, 72, 3), (2, 1, 136, 200, 6), (3, 3, 264, 40, 4)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", HEAD_SIZES, ids=lambda s: "-".join(map(str, s)))
def test_attention_with_convolutions_and_distances(sizes, dtype):
    layer = _Heads(dtype, *sizes, {2: 390, 0: 200}, 1)
    for counts, splits in (({2: 1, 0: 1}, 1), ({2: 64, 0: 2}, None), ({2: 1}, 3), ({2: 1, 0: 1}, 2), ({0: 33, 2: 64}, None), ({0: 1}, 1), ({2: 2}, None),
                           ({2: 1, 0: 1}, 64), ({0: 150, 2: 1}, None), ({2: 200, 0: 3}, None), ({2: 1}, 1), ({2: 1}, 5), ({2: 50}, None)):
        print(f"far {sizes} {dtype} {counts} splits {splits}", flush=True)
        layer.run(counts, splits)


@pytest.mark.parametrize("dtype", DTYPES)
def test_one_key_far_away_against_its_distance(dtype):
    """A key whose score towers over the others is found from far away by a head with a small penalty, and lost by one with a large one."""
    far = (np.array([0.02, 6.0]), np.array([0.1, 0.5]))
    pairs = [(255, 0), (300, 1), (320, 63), (330, 64), (389, 127)]
    for cuts in ([390], [1] * 390, [130, 126, 134], [200] + [1] * 190):
        layer = _Heads(dtype, 2, 1, 32, 16, 1, {0: 390}, 2, pairs, far)
        print(f"far key {dtype} {len(cuts)} cuts", flush=True)
        i, j = pairs[-1]
        # the oracle's: head 0 gives the far key's value, head 1 hardly any of it
        v = layer.u[0][2][j] * layer.w[2][:, -1]
        assert np.abs(layer.want[0][i, 0] - v).max() < 0.05 * np.abs(v).max() < np.abs(layer.want[0][i, 1] - v).max()
        for c in cuts:
            layer.run({0: c}, 1 if c == 1 else None)


def test_latent_attention_with_a_gate_per_feature():
    """The same results as with the gate per head, feature by feature times another gate."""
    from poptransformer_amd.engine.hybrid import LatentMixer, Rotation
    HK, T = _hk()
    rng = np.random.default_rng(0)
    for heads, dim, rot, vdim, R in ((3, 32, 32, 28, 64), (16, 128, 64, 128, 512), (2, 64, 32, 250, 96)):
        for dtype, absorbed in (("float32", True), ("bfloat16", True), ("bfloat16", False)):
            print(f"feature gate {heads} {dim} {vdim} {dtype} {absorbed}", flush=True)
            m = LatentMixer(heads, dim, rot, vdim, 24, R, 0.1, None, Rotation(50.0, rot, True))
            E, n, t = m.sizes[3], 70, T[dtype]
            rand = lambda *s: _dev(rng.standard_normal(s), t)
            ring, q, uk_t, uv = rand(1, 128, R + rot), rand(n, heads * (dim + rot)), rand(heads, R, dim) / R ** 0.5, rand(heads, E, R) / R ** 0.5
            uk_t, uv = uk_t.contiguous(), uv.contiguous()
            slot, pos = torch.zeros(n, dtype=torch.int32, device="cuda"), torch.arange(n, dtype=torch.int32, device="cuda")
            gate, norm, angles = rand(n, heads * E + 16), torch.ones(24, device="cuda"), _dev(m.angles(128))
            out = []
            for g in (torch.zeros((n, heads), device="cuda"), (gate, 8)):
                o = torch.empty((n, heads * E), dtype=t, device="cuda")
                att = HK.LatentAttention(m.sizes, m.scale, None, 1e-5, norm, None, angles, ring, n, slot, pos)
                if absorbed:
                    att.absorbed(q, uk_t, torch.empty((n * heads, R + rot), dtype=t, device="cuda"), 2, torch.empty((n * heads * 2, R), device="cuda"),
                                 torch.empty((n * heads * 2, 2), device="cuda"), uv, g, o)
                else:
                    kv = HK.WideWeight(torch.cat([uk_t.transpose(1, 2).reshape(-1, R), uv.reshape(-1, R)]), t)
                    i32 = lambda *a: torch.tensor(a, dtype=torch.int32, device="cuda")
                    bufs = [torch.empty((n, c), dtype=t, device="cuda") for c in (R, rot, kv.n_main)]
                    att.over_heads(q, (slot, pos), bufs[0], bufs[1], kv, bufs[2], (i32(0), i32(n), i32(0)), g, o)
                out.append(_np(o))
            want = out[0] * 2 * S.sigmoid(_np(gate)[:, 8:8 + heads * E])
            assert _rel(out[1], want) < (1e-5 if dtype == "float32" else 1e-2)


# ---------------------------------------------------------------------------------------------- routing
def _routes(z, c, top, groups, keep):
    got = [S.route(a, c, top, groups, keep) for a in z]
    return np.stack([g[0] for g in got]), np.stack([g[1] for g in got])


ROUTERS = [(8, 3, 1, 1), (16, 4, 4, 2), (64, 6, 8, 3), (6, 2, 6, 4), (5, 5, 1, 1), (1, 1, 1, 1), (256, 8, 8, 4), (40, 3, 8, 3), (1000, 8, 10, 2), (12, 2, 2, 1)]


@pytest.mark.parametrize("experts,top,groups,keep", ROUTERS)
def test_routing_by_corrected_scores(experts, top, groups, keep):
    """From logits, and from rows of many sizes by the product with the router."""
    HK, T = _hk()
    rng = np.random.default_rng(experts)
    c = np.where(rng.random(experts) < 0.2, -2.5, -1.25) + 0.05 * rng.standard_normal(experts)
    c = _np(_dev(c))
    r = HK.Routing(310, experts, top, False, 1.0, "cuda", H.SCORE_SIGMOID, groups, keep, True)
    for rows in (1, 33, 300):
        z = _np(_dev(rng.standard_normal((rows, experts)) * 2))
        r(_dev(z), rows, _dev(c))
        chosen, weight = _routes(z, c, top, groups, keep)
        assert np.array_equal(r.chosen.cpu().numpy()[:rows], chosen) and _rel(_np(r.weights)[:rows], weight) < 1e-5
    for rows, d in ((17, 84), (300, 1032)):
        h, w = (torch.zeros((n, HK.pad8(d)), dtype=torch.bfloat16, device="cuda") for n in (rows, experts))
        h[:, :d], w[:, :d] = _dev(rng.standard_normal((rows, d))), _dev(rng.standard_normal((experts, d)) * 2 / np.sqrt(d))
        r.by_product(h, HK.WideWeight(w[:, :d].float(), T["bfloat16"]), rows, _dev(c))
        chosen, weight = _routes(_np(h) @ _np(w).T, c, top, groups, keep)
        same = (r.chosen.cpu().numpy()[:rows] == chosen).all(1)
        assert same.mean() > 0.98 and _rel(_np(r.weights)[:rows][same], weight[same]) < 1e-4         # (a close call may fall the other way)


def test_routing_without_shares_corrections_or_groups():
    HK, _ = _hk()
    z = _np(_dev(np.random.default_rng(0).standard_normal((20, 9))))
    r = HK.Routing(20, 9, 2, True, 1.5, "cuda", H.SCORE_SIGMOID)
    r(_dev(np.concatenate([z, z[:, :1]], 1)), 20)
    order = np.argsort(-z, 1)[:, :2]
    assert np.array_equal(r.chosen.cpu().numpy(), np.concatenate([order, np.full((20, 1), 9)], 1))
    assert _rel(_np(r.weights), np.concatenate([1.5 * S.sigmoid(np.take_along_axis(z, order, 1)), S.sigmoid(z[:, :1])], 1)) < 1e-5
    for bad in (dict(groups=2), dict(groups=3, keep=4), dict(groups=9, keep=1)):
        with pytest.raises(ValueError):
            HK.Routing(20, 9, 2, False, 1.0, "cuda", H.SCORE_SIGMOID, **bad)(_dev(z), 20)
    with pytest.raises(ValueError):
        HK.Routing(20, 9, 2, False, 1.0, "cuda", groups=3)(_dev(z), 20)


# ---------------------------------------------------------------------------------------------- the end of a layer
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 53), (3, 84), (17, 1032), (2, 4096), (70, 2048), (5, 8200)])
def test_depth_norm(dtype, rows, width):
    HK, T = _hk()
    rng = np.random.default_rng(width)
    ld, tol, layers, side_ld, eps = HK.pad8(width), 5e-6 if dtype == "float32" else 6e-3, 11, 24, 1e-3
    R = (rows + 3) // 4 * 4
    history = torch.full((layers + 2, R, width), 7.0, device="cuda")
    h = torch.full((rows, ld), 7.0, dtype=T[dtype], device="cuda")
    ids, table, side_table = rng.integers(0, 19, (rows, 3)), *(_np(_dev(rng.standard_normal(s), T[dtype])) for s in ((19, width), (19, layers, side_ld)))
    w, wy = rng.standard_normal(width), rng.standard_normal(width)
    experts, top = 12, 3
    router = np.zeros((experts, ld))
    router[:, :width] = rng.standard_normal((experts, width)) * 2 / np.sqrt(width)
    router, correction = _dev(router, T[dtype]), _dev(rng.standard_normal(experts) * 0.3)
    routing = HK.Routing(rows, experts, top, False, 1.0, "cuda", H.SCORE_SIGMOID, 3, 2, True)
    pos, side = torch.zeros(rows, dtype=torch.int32, device="cuda"), torch.full((layers, R, side_ld), 7.0, dtype=T[dtype], device="cuda")
    HK.depth_norm(history, 0, rows, eps, h, _dev(w), table=_dev(table, T[dtype]), embed_scale=2.5, ids=_dev(ids, torch.int32),
                  ids_index=_dev(np.array(2), torch.int32), pos_out=pos, side_table=_dev(side_table, T[dtype]), side=side, next=1)
    want = 2.5 * table[ids[:, 2]]
    assert _rel(_np(history)[0, :rows], want) < 1e-6 and _rel(_np(history)[1, :rows], want) < 1e-6 and (pos == 2).all()
    assert _rel(_np(h)[:, :width], S.layer_norm(want, w, eps)) < tol and (_np(h)[:, width:] == 0).all()
    assert np.array_equal(_np(side)[:, :rows], side_table[ids[:, 2]].transpose(1, 0, 2)) and (_np(side)[:, rows:] == 7).all()
    for depth in (2, 3, 9, 10, layers + 1):
        print(f"depth {dtype} {rows}x{width} depth {depth}", flush=True)
        history[:depth, :rows] = _dev(rng.standard_normal((depth, rows, width)))
        before, y, a = _np(history)[:depth, :rows], rng.standard_normal((rows, width)) * 3, rng.standard_normal(depth)
        last = depth == layers + 1
        centred = depth != 3
        HK.depth_norm(history, depth, rows, eps, h, _dev(w), centred, _dev(a), _dev(y), _dev(wy), next=None if last else depth, router=router,
                      routing=routing, correction=correction)
        newest = before[-1] + S.rms_norm(y, wy, eps)
        u = S.depth_average([*before[:-1], newest], a)
        assert _rel(_np(history)[depth - 1, :rows], newest) < 3e-6 and np.array_equal(_np(history)[:depth - 1, :rows], before[:-1])
        assert last or _rel(_np(history)[depth, :rows], u) < 5e-6
        assert _rel(_np(h)[:, :width], (S.layer_norm if centred else S.rms_norm)(u, w, eps)) < tol and (_np(h)[:, width:] == 0).all()
        chosen, weight = _routes(_np(h) @ _np(router).T, _np(correction), top, 3, 2)
        same = (routing.chosen.cpu().numpy() == chosen).all(1)
        assert same.mean() > 0.9 and _rel(_np(routing.weights)[same], weight[same]) < 1e-4
    assert (_np(history)[0, rows:] == 7).all()
    for bad in (dict(depth=layers + 3), dict(depth=2, next=1), dict(depth=2, next=layers + 2)):
        with pytest.raises(ValueError):
            HK.depth_norm(history, rows=rows, eps=eps, h=h, norm_weight=_dev(w), weights=_dev(np.ones(20)), **bad)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(1, 53), (3, 84), (17, 1032), (300, 4096)])
def test_parts_added_to_the_residual(dtype, rows, width):
    HK, T = _hk()
    rng = np.random.default_rng(width)
    x, h = _dev(rng.standard_normal((rows, width))), torch.full((rows, HK.pad8(width)), 7.0, dtype=T[dtype], device="cuda")
    tol = 2e-6 if dtype == "float32" else 6e-3
    for part_type, n in ((None, 0), (torch.float32, 3), (T[dtype], 8), (torch.float32, 1)):
        before = want = _np(x)
        kw = {}
        if n:
            parts, weight = _dev(rng.standard_normal((rows, n + 1, width)), part_type), _dev(rng.standard_normal((rows, n + 1)))
            kw = dict(parts=parts, n_parts=n, parts_ld=n + 1, part_weight=weight)
            want = before + (_np(weight)[:, :n, None] * _np(parts)[:, :n]).sum(1)
        HK.add_parts(x, rows, h, **kw)
        assert _rel(_np(x), want) < 2e-6 and _rel(_np(h)[:, :width], want) < tol and (_np(h)[:, width:] == 0).all()
