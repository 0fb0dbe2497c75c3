"""Small configurations and random tensors of decoders whose results are averaged over the depths for the tests."""
import numpy as np

from tests.hybrid_models import bf16


def latent(heads=4, dim=16, rot_dim=8, vdim=12, q_rank=20, kv_rank=24, base=60.0, scaling=(3.0, 64, 4.0, 1.0), scale=None, of=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "scale": 2.0 * (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"base": base, "dims": rot_dim}}
    if scaling is not None:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if of is not None:
        m["kv_from"] = of
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def attention(heads=6, kv_heads=2, dim=16, vdim=24, taps=4, scale=None, mlp=None):
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": taps,
                                                       "scale": 2.0 * dim ** -0.5 if scale is None else scale}}


def mamba(heads=4, groups=2, state=24, vdim=20, taps=4, norm_groups=2, mlp=None):
    return {"type": "mamba2", "mlp": mlp, "mixer": {"heads": heads, "groups": groups, "state": state, "vdim": vdim, "conv": taps,
                                                    "norm_groups": norm_groups}}


def dense(ff=56):
    return {"kind": "dense", "ff": ff}


def moe(experts=8, top=3, ff=40, groups=(2, 1)):
    r = {"experts": experts, "top": top}
    if groups is not None:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def config(layers, width=84, vocab=112, eps=1e-5, embed=3.0, cap=9.0, side=20):
    return {"architecture": "Sabolorn", "embedding": {"scale": embed}, "layers": layers, "logit_softcap": cap, "norm": {"eps": eps},
            "token_side": {"dim": side}, "vocab": vocab, "width": width}


DEPTH = {
    # every mixer with and without experts, a cache read by two others, a layer without a feed-forward
    "small": config([mamba(mlp=moe()), latent(mlp=dense()), attention(mlp=moe(top=2, ff=24)), latent(of=1, mlp=moe()), mamba(heads=2, groups=1, mlp=None),
                     latent(heads=2, of=1, dim=8, vdim=16, q_rank=9, scale=0.4, mlp=dense(40))]),
    # sizes that are multiples of nothing, other numbers of taps, one group and as many as heads, norms across heads, one expert of one
    "odd": config([attention(heads=3, kv_heads=1, dim=10, vdim=7, taps=2, mlp=moe(experts=5, top=1, ff=18, groups=None)),
                   mamba(heads=3, groups=3, state=9, vdim=10, taps=3, norm_groups=2, mlp=dense(20)), attention(heads=2, kv_heads=2, dim=9, vdim=13, taps=6),
                   latent(heads=5, dim=7, rot_dim=6, vdim=9, q_rank=11, kv_rank=13, scaling=None, base=7.0, mlp=moe(experts=6, top=2, ff=10, groups=(3, 2))),
                   mamba(heads=1, groups=1, state=5, vdim=6, taps=1, norm_groups=3, mlp=moe(experts=1, top=1, ff=12, groups=None)),
                   attention(heads=5, kv_heads=5, dim=4, vdim=3, taps=1, mlp=dense(9))], width=53, vocab=91, embed=1.0, cap=None, side=7),
    # everything as large as everything else; factors of one
    "alike": config([latent(heads=2, dim=32, rot_dim=32, vdim=32, q_rank=32, kv_rank=32, scaling=(1.0, 64, 2.0, 2.0), scale=0.125, mlp=dense(64)),
                     mamba(heads=2, groups=2, state=32, vdim=32, norm_groups=1, mlp=moe(4, 2, 64, (1, 1))),
                     attention(heads=2, kv_heads=2, dim=32, vdim=32, scale=0.125, mlp=dense(64))], width=64, vocab=64, embed=1.0, side=32),
    # sizes of larger models: every kind of tile, whole tiles of channels, heads beyond the tiles
    "wide": config([latent(heads=10, dim=96, rot_dim=32, vdim=72, q_rank=200, kv_rank=160, base=1e4, scaling=(4.0, 256, 16.0, 1.0), mlp=moe(24, 4, 300, (4, 2))),
                    mamba(heads=10, groups=2, state=120, vdim=64, norm_groups=2, mlp=dense(1100)),
                    attention(heads=10, kv_heads=2, dim=136, vdim=72, mlp=moe(40, 3, 130, (8, 3))), latent(heads=3, dim=240, rot_dim=32, vdim=40, of=None),
                    mamba(heads=3, groups=1, state=200, vdim=104, norm_groups=1), attention(heads=3, kv_heads=1, dim=40, vdim=264)],
                   width=1032, vocab=300, side=136),
}


def _codes(rng, V, r, banned):
    """Router coordinates of every token: `top` experts stand out in the groups that are kept, one in every other group stands out further,
    as does the one that the correction keeps away."""
    E, top = r["experts"], r["top"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    size = E // g["count"]
    code = np.full((V, E), -5.0)
    for t in range(V):
        kept = rng.permutation(g["count"])[:g["keep"]]
        lists = [[e for e in rng.permutation(np.arange(k * size, (k + 1) * size)) if e != banned] for k in kept]
        order = [e for k in range(size) for mine in lists for e in mine[k:k + 1]]
        high = order[:top]
        for mine in lists if g["keep"] < g["count"] else ():        # two that count in every kept group
            for e in mine[:2]:
                code[t, e] = 1.0
        code[t, high] = 7.0
        for k in set(range(g["count"])) - set(kept):
            code[t, rng.integers(k * size, (k + 1) * size)] = 9.0
        if banned is not None:
            code[t, banned] = 9.0
    return 0.4 * (code + 0.3 * rng.standard_normal(code.shape))


def random_depth(cfg, seed):
    """Tokens carry a code in which their experts stand well apart from the others, so that no rounding changes a choice; the final
    norm's weights have both signs, so that a token does not predict itself."""
    rng = np.random.default_rng(seed)
    d, V, n_side, layers = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"], cfg["layers"]
    sd = {}

    def lin(name, n, k, gain=1.0):
        sd[name] = bf16(rng.standard_normal((n, k)) * gain / np.sqrt(k))

    def vec(name, n, mean=1.0, spread=0.2):
        sd[name] = bf16(mean + spread * rng.standard_normal(n))

    def taps(name, channels, n):
        sd[name] = bf16(rng.standard_normal((channels, n)) * 0.35 + (np.arange(n) == n - 1) * 0.8)

    def out(name, k, gain=1.0):
        """what a sublayer adds to the residual, which leaves the codes alone"""
        w = rng.standard_normal((d, k)) * gain / np.sqrt(k)
        sd[name] = bf16(w - used.T @ (used @ w))

    axes = np.linalg.qr(rng.standard_normal((d, d)))[0].T
    used = axes[:sum(lay["mlp"]["router"]["experts"] for lay in layers if (lay["mlp"] or {}).get("kind") == "moe")]
    x = rng.standard_normal((V, d)) * 0.6
    for i, lay in enumerate(layers):
        if (lay["mlp"] or {}).get("kind") != "moe":
            continue
        r = lay["mlp"]["router"]
        g = r.get("groups") or {"count": 1, "keep": 1}
        size = r["experts"] // g["count"]
        banned = int(rng.integers(r["experts"])) if size * g["keep"] > r["top"] and size > 3 else None
        mine, axes = axes[:r["experts"]], axes[r["experts"]:]
        x += (_codes(rng, V, r, banned) - x @ mine.T) @ mine
        sd[f"l{i}.mlp.router"] = bf16(mine)
        sd[f"l{i}.mlp.correction"] = bf16(np.where(np.arange(r["experts"]) == banned, -2.5, -1.25))
    scale = np.sqrt((x ** 2).mean())
    for i, lay in enumerate(layers):                 # (behind a norm the code is divided by this)
        if f"l{i}.mlp.router" in sd:
            sd[f"l{i}.mlp.router"] = bf16(sd[f"l{i}.mlp.router"] * scale * 1.4)
    sd["embed"] = bf16(x / cfg["embedding"]["scale"])
    sd["side.embed"] = bf16(rng.standard_normal((V, len(layers) * n_side)))
    for i, lay in enumerate(layers):
        p, m, f = f"l{i}.", lay["mixer"], lay["mlp"]
        mix = p + "mix."
        H, E = m["heads"], m["vdim"]
        vec(p + "norm1", d, 1.0, 0.1)
        if lay["type"] == "latent_attention":
            D, P, R, Q = m["dim"], m["rot_dim"], m["kv_rank"], m["q_rank"]
            lin(mix + "dq", Q, d)
            vec(mix + "dq.norm", Q)
            lin(mix + "uq", H * (D + P), Q)
            if m.get("kv_from") is None:
                lin(mix + "dkv", R + P, d)
                vec(mix + "dkv.norm", R)
            lin(mix + "uk", H * D, R)
            lin(mix + "uv", H * E, R)
            lin(mix + "g", H * E, d, 1.5)
        elif lay["type"] == "attention":
            G, D = m["kv_heads"], m["dim"]
            for n, c in (("q", H * D), ("k", G * D), ("v", G * E)):
                lin(mix + n, c, d)
                vec(mix + n + ".b", c, 0.0, 0.4)
                taps(mix + n + ".conv", c, m["conv"])
            sd[mix + "r1"] = bf16(rng.uniform(0.2, 2.0, H) * np.where(np.arange(H) % 3 == 1, 0.02, 1.0))
            sd[mix + "r2"] = bf16(rng.uniform(0.05, 0.5, H))
        else:
            inner, states = H * E, m["groups"] * m["state"]
            lin(mix + "in", 2 * inner + 2 * states + H, d)
            taps(mix + "conv", inner + 2 * states, m["conv"])
            vec(mix + "conv.b", inner + 2 * states, 0.0, 0.3)
            sd[mix + "dt_bias"] = bf16(np.log(np.expm1(rng.uniform(0.02, 0.5, H))))
            sd[mix + "A_log"] = bf16(rng.uniform(-4.0, 0.5, H))
            vec(mix + "D", H, 0.8, 0.3)
            vec(mix + "norm", inner)
        out(mix + "o", H * E, 1.4)
        parts = [] if f is None else [("", f["ff"])] if f["kind"] == "dense" else [(f"e{e}.", f["expert"]["ff"]) for e in range(f["router"]["experts"])]
        for q, ff in parts:
            if f["kind"] == "moe":
                lin(p + "mlp." + q + "gate", ff, d)
            lin(p + "mlp." + q + "up", ff, d)
            out(p + "mlp." + q + "down", ff, 0.6 if f["kind"] == "dense" else 1.0)
        lin(p + "side.gate", n_side, d)
        out(p + "side.proj", n_side)
        vec(p + "side.norm", d, 0.5, 0.2)
        w = rng.uniform(-0.15, 0.15, i + 2)
        w[0], w[-1] = 0.4, 0.6
        sd[p + "dwa"] = bf16(w)
    vec("final.norm", d, 0.0, 1.0)
    return sd
