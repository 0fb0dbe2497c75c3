"""Small configurations and random tensors of decoders with latent attention and parallel sublayers for the tests."""
import numpy as np

from tests.hybrid_models import bf16


def latent(heads=4, dim=16, rot_dim=8, vdim=24, q_rank=40, kv_rank=32, window=12, scale=None, base=50.0, ff=56, of=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
         "scale": (dim + rot_dim) ** -0.5 * 3 if scale is None else scale, "rot": {"base": base, "dims": rot_dim}}
    if window is not None:
        m["mask"] = {"size": window}
    if of is not None:
        m["kv_from"] = of
    return {"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def parallel_config(layers, width=84, vocab=112, groups=3, eps=1e-5, embed=3.0, positions=720):
    return {"architecture": "Ruperax", "embedding": {"scale": embed}, "layers": layers, "max_positions": positions,
            "norm": {"eps": eps, "groups": groups}, "vocab": vocab, "width": width}


def small_parallel():
    """A cache of its own, the same cache under a wider window and other heads, a layer without a feed-forward, all positions."""
    return parallel_config([latent(), latent(window=30, heads=3, vdim=20, q_rank=28, of=0), latent(window=None, kv_rank=48, ff=None, base=1e4),
                            latent(window=9, kv_rank=48, base=1e4, of=2, ff=40)])


PARALLEL = {
    "small": small_parallel(),
    # sizes that are multiples of nothing, a window of one token, more than 16 heads
    "odd": parallel_config([latent(heads=3, dim=20, rot_dim=6, vdim=28, q_rank=30, kv_rank=44, window=7, ff=36),
                            latent(heads=1, dim=5, rot_dim=2, vdim=3, q_rank=9, kv_rank=10, window=1, base=2.5, ff=None),
                            latent(heads=21, dim=9, rot_dim=10, vdim=17, q_rank=50, kv_rank=70, window=65, ff=20),
                            latent(heads=2, dim=33, rot_dim=6, vdim=40, q_rank=11, kv_rank=44, window=64, of=0, ff=12)],
                           width=54, vocab=91, groups=9, embed=1.0),
    # one group, everything as large as everything else
    "alike": parallel_config([latent(heads=2, dim=32, rot_dim=32, vdim=32, q_rank=64, kv_rank=64, window=64, scale=1.0, ff=64),
                              latent(heads=2, dim=32, rot_dim=32, vdim=32, q_rank=64, kv_rank=64, window=64, scale=1.0, ff=64, of=0)],
                             width=64, vocab=64, groups=1, embed=1.0),
    # sizes of larger models: every kind of tile, a latent beyond the matrix unit's, heads beyond the tiles
    "wide": parallel_config([latent(heads=18, dim=128, rot_dim=64, vdim=128, q_rank=192, kv_rank=512, window=90, ff=1100),
                             latent(heads=2, dim=200, rot_dim=64, vdim=72, q_rank=192, kv_rank=600, window=20, ff=72),
                             latent(heads=1, dim=64, rot_dim=160, vdim=260, q_rank=64, kv_rank=1100, window=33, ff=None)],
                            width=1032, vocab=300, groups=4),
}


def random_parallel(cfg, seed):
    rng = np.random.default_rng(seed)
    d, V = cfg["width"], cfg["vocab"]
    sd = {}

    def lin(name, n, k, gain=1.0):
        sd[name] = bf16(rng.standard_normal((n, k)) * gain / np.sqrt(k))

    def vec(name, n, mean=1.0, spread=0.2):
        sd[name] = bf16(mean + spread * rng.standard_normal(n))

    sd["embed"] = bf16(rng.standard_normal((V, d)))
    sd["pos"] = bf16(rng.standard_normal((cfg["max_positions"], d)))
    for i, lay in enumerate(cfg["layers"]):
        p, m = f"l{i}.", lay["mixer"]
        H = m["heads"]
        vec(p + "norm1", d)
        vec(p + "shift", d, 0.5, 0.3)
        lin(p + "rg1", d, d)
        vec(p + "rg1.b", d, 0.0, 0.5)
        lin(p + "mix.dq", m["q_rank"], d)
        vec(p + "mix.dq.norm", m["q_rank"])
        lin(p + "mix.uq", H * (m["dim"] + m["rot_dim"]), m["q_rank"])
        if m.get("kv_from") is None:
            lin(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], d)
            vec(p + "mix.dkv.norm", m["kv_rank"])
        lin(p + "mix.uk", H * m["dim"], m["kv_rank"])
        lin(p + "mix.uv", H * m["vdim"], m["kv_rank"])
        lin(p + "mix.g", H, d, 2.0)
        lin(p + "mix.o", d, H * m["vdim"], 2.0)
        if lay["mlp"] is not None:
            ff = lay["mlp"]["ff"]
            vec(p + "norm2", d)
            lin(p + "rg2", d, d)
            vec(p + "rg2.b", d, 0.0, 0.5)
            for n, (a, b) in (("gate", (ff, d)), ("up", (ff, d)), ("down", (d, ff))):
                lin(p + "mlp." + n, a, b)
                vec(p + f"mlp.{n}.b", a, 0.0, 0.5)
    vec("final.norm", d)
    lin("head", V, d, 2.0)
    return sd
