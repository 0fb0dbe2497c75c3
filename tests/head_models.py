"""Small configurations and random tensors of decoders with attention by heads and mixtures of experts for the tests."""
import numpy as np

from tests.hybrid_models import bf16


def _scaled(dim, scale):
    return 2.0 * dim ** -0.5 if scale is None else scale


def windowed(heads=4, kv_heads=2, dim=16, window=12, keep=3, base=50.0, turned=8, factor=2.0, scale=None, mlp=None):
    """Sliding window with kept first positions, sinks, values that are the keys, a gate per head."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": _scaled(dim, scale), "rot": {"base": base, "dims": turned}}
    if factor is not None:
        m["rot"]["scaling"] = {"factor": factor}
    if window is not None:
        m["mask"] = {"size": window, "keep_first": keep}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def differential(heads=4, kv_heads=2, dim=16, vdim=24, chunk=20, diff=0.3, scale=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": _scaled(dim, scale), "diff": diff, "mask": {"size": chunk}}
    return {"type": "attention_2", "mixer": m, "mlp": mlp}


def chunked(heads=3, kv_heads=3, dim=24, vdim=16, chunk=14, base=80.0, turned=24, scaling=(3.0, 64, 4.0, 1.0), scale=None, mlp=None):
    """Within chunks, neighbours rotated with stretched frequencies, a gate per feature."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": _scaled(dim, scale), "rot": {"base": base, "dims": turned}}
    if scaling is not None:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if chunk is not None:
        m["mask"] = {"size": chunk}
    return {"type": "attention_3", "mixer": m, "mlp": mlp}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=6, top=2, ff=40, limit=1.2, scale=1.7, shared=24, shared_limit=0.9):
    c = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "scale": scale, "top": top}}
    if shared is not None:
        c["shared"] = {"ff": shared, "limit": shared_limit}
    return c


def config(layers, width=84, vocab=112, eps=1e-5, embed=3.0):
    return {"architecture": "Golapel", "embedding": {"scale": embed}, "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}


HEADS = {
    # every mixer with and without experts, and a last layer without a feed-forward
    "small": config([windowed(mlp=moe()), chunked(mlp=dense()), differential(mlp=moe(ff=24, shared=40)), windowed(window=5, keep=1, mlp=dense(40)),
                     differential(heads=2, kv_heads=2, chunk=9), chunked(chunk=31)]),
    # sizes that are multiples of nothing, part of a head rotated, one expert of one, all of three, masks of one token
    "odd": config([windowed(heads=3, kv_heads=1, dim=20, window=7, keep=2, turned=6, mlp=moe(experts=5, top=1, ff=18, shared=None)),
                   chunked(heads=5, kv_heads=5, dim=9, vdim=13, chunk=6, turned=2, base=3.0, mlp=moe(experts=3, top=3, ff=10, shared=9)),
                   differential(heads=7, kv_heads=1, dim=11, vdim=5, chunk=8, diff=0.8, mlp=dense(20)),
                   windowed(heads=1, kv_heads=1, dim=44, window=1, keep=0, turned=44, factor=None, mlp=moe(experts=1, top=1, ff=12, shared=30)),
                   differential(heads=1, kv_heads=1, dim=2, vdim=1, chunk=1), windowed(heads=6, kv_heads=3, dim=10, window=None, turned=2)],
                  width=53, vocab=91, embed=1.0),
    # everything as large as everything else; factors of one
    "alike": config([windowed(heads=2, kv_heads=2, dim=32, window=64, keep=64, turned=32, factor=1.0, scale=1.0 / 16, mlp=dense(64)),
                     differential(heads=2, kv_heads=2, dim=32, vdim=32, chunk=64, diff=0.5, scale=1.0 / 16, mlp=moe(2, 2, 64, 1.0, 1.0, 64, 1.0)),
                     chunked(heads=2, kv_heads=2, dim=32, vdim=32, chunk=64, turned=32, scaling=(1.0, 64, 2.0, 2.0), scale=1.0 / 16, mlp=dense(64))],
                    width=64, vocab=64, embed=1.0),
    # rotation and chunks left out
    "plain": config([dict(windowed(mlp=moe(shared=None))), chunked(chunk=None, scaling=None, mlp=dense()), windowed(window=3, keep=40)]),
    # sizes of larger models: every kind of tile, whole tiles of channels, heads beyond the tiles
    "wide": config([windowed(heads=10, kv_heads=2, dim=136, window=90, keep=5, turned=64, base=1e4, mlp=moe(experts=24, top=4, ff=300, shared=1100)),
                    differential(heads=4, kv_heads=2, dim=72, vdim=136, chunk=70, mlp=moe(experts=40, top=3, ff=130, shared=None)),
                    chunked(heads=3, kv_heads=1, dim=264, vdim=40, chunk=50, turned=128, base=1e4, mlp=dense(1100)),
                    differential(heads=2, kv_heads=1, dim=40, vdim=260, chunk=33), chunked(heads=2, kv_heads=2, dim=128, vdim=128, chunk=80, turned=128)],
                   width=1032, vocab=300),
}
HEADS["plain"]["layers"][0]["mixer"]["rot"] = None


def random_heads(cfg, seed):
    """Tokens carry a code in which their experts stand well apart from the others, so that no rounding changes a choice; the final
    norm's weights have both signs, so that a token does not predict itself."""
    rng = np.random.default_rng(seed)
    d, V, emb = cfg["width"], cfg["vocab"], cfg["embedding"]["scale"]
    sd = {}

    def lin(name, n, k, gain=1.0):
        sd[name] = bf16(rng.standard_normal((n, k)) * gain / np.sqrt(k))

    def vec(name, n, mean=1.0, spread=0.2):
        sd[name] = bf16(mean + spread * rng.standard_normal(n))

    mixtures = [(i, lay["mlp"]["router"]) for i, lay in enumerate(cfg["layers"]) if (lay["mlp"] or {}).get("kind") == "moe"]
    axes = np.linalg.qr(rng.standard_normal((d, d)))[0].T
    x = rng.standard_normal((V, d)) * 1.5
    for i, r in mixtures:
        mine, axes = axes[:r["experts"]], axes[r["experts"]:]
        code = np.sort(rng.standard_normal((V, r["experts"])), 1)[:, ::-1] + np.where(np.arange(r["experts"]) < r["top"], 6.0, -6.0)
        code = rng.permuted(code, axis=1)
        x += (code - x @ mine.T) @ mine
        sd[f"l{i}.mlp.router"] = bf16(mine * 0.5)
    sd["embed"] = bf16(x / emb)
    for i, lay in enumerate(cfg["layers"]):
        p, m, f = f"l{i}.", lay["mixer"], lay["mlp"]
        H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        maps = 2 if lay["type"] == "attention_2" else 1
        vec(p + "norm1", d, 0.8)
        for n, c in [("q", H * maps * D), ("k", G * maps * D)] + ([("v", G * E)] if lay["type"] != "attention" else []):
            lin(p + "mix." + n, c, d, 0.3)
            if lay["type"] != "attention_2":
                vec(p + f"mix.{n}.b", c, 0.0, 0.5)
        vec(p + "mix.q.norm", D)
        vec(p + "mix.k.norm", D)
        if lay["type"] == "attention":
            vec(p + "mix.sink", H, 1.0, 1.0)
            lin(p + "mix.g", H, d, 0.3)
        elif lay["type"] == "attention_2":
            for n in ("lq1", "lk1", "lq2", "lk2"):
                vec(p + "mix." + n, D, 0.0, 0.6 / D ** 0.5)
        else:
            lin(p + "mix.g", H * E, d, 0.3)
        lin(p + "mix.o", d, H * E)
        if f is None:
            continue
        vec(p + "norm2", d, 0.8)
        parts = [("", f["ff"])] if f["kind"] == "dense" else [(f"e{e}.", f["expert"]["ff"]) for e in range(f["router"]["experts"])]
        if f.get("shared") is not None:
            parts.append(("shared.", f["shared"]["ff"]))
            lin(p + "mlp.shared.sg", 1, d, 0.3)
        for q, ff in parts:
            for n, shape in (("gate", (ff, d)), ("up", (ff, d)), ("down", (d, ff))):
                lin(p + "mlp." + q + n, *shape, 1.0 if n == "down" else 0.3)
    vec("final.norm", d, 0.0, 1.0)
    return sd
