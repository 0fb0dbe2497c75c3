"""Plain, slow restatement of the Zekilix decoder in float64 numpy, one function per mechanism.

Test infrastructure only.  Arrays are [tokens, features] of ONE sequence, positions count from 0, `cfg` is the
model's configuration (the dictionary of its config.json) and `sd` its tensors by name.  Nothing here is shared with the
product path: a sequence is always evaluated as a whole and from scratch.

`rnd` (default: nothing) is applied where a 16-bit evaluation rounds - what enters a matrix product and what a projection
gives - so that tests can measure how much of a difference rounding alone explains.
"""
import numpy as np

SIGMOID_SLOPE = 1.702           # of the feed-forward's gate


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def softcap(z, cap):
    return cap * np.tanh(z / cap)


def rms_norm(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def layer_norm(x, w, eps):
    c = x - np.mean(x, axis=-1, keepdims=True)
    return c / np.sqrt(np.mean(c * c, axis=-1, keepdims=True) + eps) * w


def head_slopes(n_head):
    return 2.0 ** (-8.0 * (np.arange(n_head) + 1) / n_head)


def windowed_attention(q, k, v, scale, slopes, window):
    """q [T, H, D], k and v [T, G, D]: causal attention over the last `window` positions (None: all of them) with the
    score lowered by slope * distance.  Returns [T, H, D]."""
    T, H, _ = q.shape
    group = H // k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        dist = i - np.arange(lo, i + 1)
        for h in range(H):
            g = h // group
            s = k[lo:i + 1, g] @ q[i, h] * scale - slopes[h] * dist
            p = np.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[lo:i + 1, g]
    return out


def exact(a):
    return a


def attention_mixer(sd, p, mixer, h, eps, rnd=exact):
    H, G, D = mixer["heads"], mixer["kv_heads"], mixer["dim"]
    T = h.shape[0]
    q, k = rnd(h @ sd[p + "q"].T), rnd(h @ sd[p + "k"].T)
    v = k.reshape(T, G, D)
    q = (rms_norm(q, eps) * sd[p + "q.norm"]).reshape(T, H, D)
    k = (rms_norm(k, eps) * sd[p + "k.norm"]).reshape(T, G, D)
    window = (mixer.get("mask") or {}).get("size")
    o = windowed_attention(q, k, v, mixer["scale"], head_slopes(H), window).reshape(T, H * D)
    return rnd(o * sigmoid(rnd(h @ sd[p + "g"].T))) @ sd[p + "o"].T


def mlstm_recurrence(q, k, v, i, f):
    """q, k [T, H, D], v [T, H, E], log gates i and f [T, H]; token by token.  Returns [T, H, E]."""
    T, H, D = q.shape
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        S, n, m = np.zeros((D, v.shape[2])), np.zeros(D), 0.0
        for t in range(T):
            m_new = max(f[t, h] + m, i[t, h])
            keep, take = np.exp(f[t, h] + m - m_new), np.exp(i[t, h] - m_new)
            S = keep * S + take * np.outer(k[t, h], v[t, h])
            n = keep * n + take * k[t, h]
            m = m_new
            out[t, h] = (S.T @ q[t, h]) / (max(abs(n @ q[t, h]), np.exp(-m)) + 1e-6)
    return out


def mlstm_gates(sd, p, h, cap):
    i = softcap(h @ sd[p + "i"].T + sd[p + "i.b"], cap)
    f = log_sigmoid(softcap(h @ sd[p + "f"].T + sd[p + "f.b"], cap))
    return i, f


def mlstm_mixer(sd, p, mixer, h, eps, rnd=exact):
    H, D, E = mixer["heads"], mixer["dim"], mixer["vdim"]
    T = h.shape[0]
    q = rnd(h @ sd[p + "q"].T).reshape(T, H, D) * D ** -0.5
    k = rnd(h @ sd[p + "k"].T).reshape(T, H, D)
    v = rnd(h @ sd[p + "v"].T).reshape(T, H, E)
    i, f = mlstm_gates(sd, p, h, mixer["gate_cap"])
    o = rms_norm(mlstm_recurrence(q, k, v, i, f), eps).reshape(T, H * E)
    return rnd(o * sd[p + "norm"] * sigmoid(rnd(h @ sd[p + "g"].T))) @ sd[p + "o"].T


MIXERS = {"attention": attention_mixer, "mlstm": mlstm_mixer}


def clamped_glu(gate, up, limit):
    g, u = np.minimum(gate, limit), np.clip(up, -limit, limit)
    return g * sigmoid(SIGMOID_SLOPE * g) * (u + 1.0)


def feed_forward(sd, p, mlp, h, rnd=exact):
    return rnd(clamped_glu(h @ sd[p + "gate"].T, h @ sd[p + "up"].T, mlp["limit"])) @ sd[p + "down"].T


def connect(streams, weights_in, weights_out, mix, mult, sublayer):
    """One sublayer between `streams` [S, T, d] (weights None: a single plain residual): read with weights_in, write with weights_out, mix from -> to."""
    if weights_in is None:
        return streams + mult * sublayer(streams[0])[None]
    y = sublayer(np.tensordot(weights_in, streams, axes=1))
    return np.einsum("st,sxd->txd", mix, streams) + mult * weights_out[:, None, None] * y[None]


def owner(cfg, i):
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


def forward(sd, cfg, ids, collect=None, rnd=exact):
    """Logits [T, vocab] of one sequence.  `collect` (a list) receives the sum of the streams after every layer."""
    sd = {k: np.asarray(v, np.float64) for k, v in sd.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = sd["embed"][np.asarray(ids)] * cfg["embedding"]["scale"]
    streams = np.stack([x] * (cfg.get("streams") or 1))
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{owner(cfg, i)}."

        def run(q, norm, fn):
            hc = p + f"hc{q}."
            return connect(streams, *(sd.get(hc + n) for n in ("in", "out", "mix")), mult,
                           lambda u: fn(rnd(layer_norm(u, sd[p + norm], eps))))

        streams = run(1, "norm1", lambda h: MIXERS[layer["type"]](sd, p + "mix.", layer["mixer"], h, eps, rnd))
        if layer.get("mlp") is not None:
            streams = run(2, "norm2", lambda h: feed_forward(sd, p + "mlp.", layer["mlp"], h, rnd))
        if collect is not None:
            collect.append(streams.sum(0))
    logits = rnd(layer_norm(streams.sum(0), sd["final.norm"], eps)) @ sd["head"].T
    return softcap(logits, cfg["logit_softcap"]) if cfg.get("logit_softcap") else logits
