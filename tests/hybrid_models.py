"""Small configurations and random tensors of hybrid decoders for the tests, and what the tests of whole decoders share."""
import numpy as np


def attention(heads=4, kv_heads=2, dim=16, window=12, scale=None, mlp=None, of=None):
    c = {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim,
                                        "scale": dim ** -0.5 if scale is None else scale}, "mlp": mlp}
    if window is not None:
        c["mixer"]["mask"] = {"size": window}
    if of is not None:
        c["weights_of"] = of
    return c


def mlstm(heads=3, dim=24, vdim=40, cap=7.0, mlp=None, of=None):
    c = {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": mlp}
    if of is not None:
        c["weights_of"] = of
    return c


def dense(ff=56, limit=0.9):
    return {"kind": "dense", "ff": ff, "limit": limit}


def config(layers, width=80, vocab=112, streams=3, eps=1e-5, mult=0.35, embed=3.0, cap=9.0):
    c = {"architecture": "Zekilix", "embedding": {"scale": embed}, "layers": layers, "logit_softcap": cap, "norm": {"eps": eps},
         "residual_mult": mult, "vocab": vocab, "width": width}
    if streams is not None:
        c["streams"] = streams
    return c


def small_config(**kw):
    """Both mixers, a layer without a feed-forward, and both kinds used a second time."""
    return config([mlstm(mlp=dense()), attention(mlp=dense(ff=64, limit=1.3)), mlstm(heads=2, dim=16, vdim=32, mlp=None),
                   attention(mlp=dense(ff=64, limit=1.3), of=1), mlstm(mlp=dense(), of=0)], **kw)


def bf16(a):
    """fp32 values that bf16 holds exactly (round to nearest even)."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(np.uint32).view(np.float32)


def random_tensors(cfg, seed, forget_bias=2.0):
    rng = np.random.default_rng(seed)
    d, V, S = cfg["width"], cfg["vocab"], cfg.get("streams")
    sd = {}

    def lin(name, n, k, gain=1.0):
        sd[name] = bf16(rng.standard_normal((n, k)) * gain / np.sqrt(k))

    def vec(name, n, mean=1.0, spread=0.2):
        sd[name] = bf16(mean + spread * rng.standard_normal(n))

    def connect(name):
        vec(name + ".in", S, 0.6, 0.2)
        vec(name + ".out", S, 0.8, 0.2)
        sd[name + ".mix"] = bf16(np.eye(S) * 0.8 + 0.15 * rng.standard_normal((S, S)))

    sd["embed"] = bf16(rng.standard_normal((V, d)))
    for i, lay in enumerate(cfg["layers"]):
        if lay.get("weights_of") is not None:
            continue
        p, m = f"l{i}.", lay["mixer"]
        vec(p + "norm1", d)
        if S is not None:
            connect(p + "hc1")
        if lay["type"] == "attention":
            N, KD = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
            for n, c in (("q", N), ("k", KD), ("g", N)):
                lin(p + "mix." + n, c, d)
            vec(p + "mix.q.norm", N, 1.3)
            vec(p + "mix.k.norm", KD, 1.3)
        else:
            N, QD = m["heads"] * m["vdim"], m["heads"] * m["dim"]
            for n, c in (("q", QD), ("k", QD), ("v", N), ("g", N), ("i", m["heads"]), ("f", m["heads"])):
                lin(p + "mix." + n, c, d)
            vec(p + "mix.i.b", m["heads"], -0.5, 0.5)
            vec(p + "mix.f.b", m["heads"], forget_bias, 0.5)
            vec(p + "mix.norm", N)
        lin(p + "mix.o", d, N)
        if lay.get("mlp") is not None:
            ff = lay["mlp"]["ff"]
            vec(p + "norm2", d)
            if S is not None:
                connect(p + "hc2")
            lin(p + "mlp.gate", ff, d)
            lin(p + "mlp.up", ff, d)
            lin(p + "mlp.down", d, ff)
    vec("final.norm", d)
    lin("head", V, d, 2.0)
    return sd


def token_ids(seed, n, cfg):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], n).tolist()


class Reference:
    """The oracle's logits of one sequence, and per number format how far from them a result may be: the rms of the
    difference over the rms of all logits is compared with what rounding alone does to this very sequence (fp32 accumulates
    in another order: a floor)."""

    def __init__(self, forward, sd, cfg, ids, dtype):
        self.logits = forward(sd, cfg, ids)
        self.scale = np.sqrt((self.logits ** 2).mean())
        if dtype == "float32":
            self.limit = 2e-5
        else:
            # (three roundings: one sample of what rounding does says little about a single position)
            draws = [self.error(forward(sd, cfg, ids, rnd=lambda a, k=k: bf16(a * (1 + k)) / (1 + k))).max() for k in (0, 0.13, 0.31)]
            self.limit = 2.0 * max(draws) + 0.01

    def error(self, got, at=slice(None)):
        return np.sqrt(((got - self.logits[at]) ** 2).mean(-1)) / self.scale

    def check(self, got, at=slice(None)):
        got = got.float().cpu().numpy() if hasattr(got, "cpu") else got
        err = self.error(got, at)
        assert err.max() < self.limit, f"place {int(err.argmax())}: {err.max():.2e}, limit {self.limit:.2e}"


def feed(dec, slot, ids, cuts):
    """The tokens in portions of the given sizes (the rest one by one); logits of all positions."""
    out, p, cuts = [], 0, list(cuts)
    while p < len(ids):
        c = min(cuts.pop(0) if cuts else 1, len(ids) - p)
        out.append(dec.advance([(slot, ids[p:p + c], list(range(c)))]).cpu().numpy())
        p += c
    return np.concatenate(out)


def greedy(forward, cfg, sd, ids, steps, pad, tie):
    """The loop by the oracle: container after `steps` iterations, and per row the number of comparable columns (up to the
    first place where two logits are closer than `tie` of the largest)."""
    out = ids.copy()
    B, L = ids.shape
    cols = np.full(B, min(steps + 1, L))
    for b in range(B):
        for t in range(min(steps, L - 1)):
            if out[b, t + 1] != pad:
                continue
            logits = forward(sd, cfg, out[b, :t + 1])[-1]
            top = np.sort(logits)[-2:]
            if top[1] - top[0] < tie * np.abs(logits).max():
                cols[b] = min(cols[b], t + 1)
            out[b, t + 1] = int(logits.argmax())
    return out, cols
