"""Plain, slow restatement of the Ruperax decoder in float64 numpy, one function per mechanism.

Test infrastructure only.  Arrays are [tokens, features] of ONE sequence from its first token on, `cfg` is the
model's configuration (the dictionary of its config.json) and `sd` its tensors by name.  Nothing here is shared with the
product path: a sequence is always evaluated as a whole and from scratch, keys and values are made for every head, and
nothing is cached.

`rnd` (default: nothing) is applied where a 16-bit evaluation rounds - what enters a matrix product and what a projection
gives - so that tests can measure how much of a difference rounding alone explains.
"""
import numpy as np


def exact(a):
    return a


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def group_rms_norm(x, w, groups, eps):
    """Every one of `groups` equal consecutive parts over its own root mean square."""
    parts = x.reshape(x.shape[:-1] + (groups, -1))
    parts = parts / np.sqrt(np.mean(parts * parts, axis=-1, keepdims=True) + eps)
    return parts.reshape(x.shape) * w


def token_shift(h, mix):
    """h_t + (h_{t-1} - h_t) * mix, with zeros before the first token."""
    before = np.zeros_like(h)
    before[1:] = h[:-1]
    return h + (before - h) * mix


def rotate_half(x, base, dims):
    """x [T, ..., n]: the first `dims` features rotated by the token's position, feature i together with i + dims / 2."""
    half = dims // 2
    angle = np.arange(x.shape[0])[:, None] * float(base) ** (-2.0 * np.arange(half) / dims)
    c, s = (f(angle).reshape((x.shape[0],) + (1,) * (x.ndim - 2) + (half,)) for f in (np.cos, np.sin))
    u, v = x[..., :half], x[..., half:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], axis=-1)


def sliding_softmax_attention(q, k, v, scale, window):
    """q, k [T, H, D], v [T, H, E]: causal attention over the last `window` positions (None: all of them)."""
    T = q.shape[0]
    out = np.zeros((T,) + v.shape[1:])
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        s = np.einsum("jhd,hd->hj", k[lo:i + 1], q[i]) * scale
        p = np.exp(s - s.max(1, keepdims=True))
        out[i] = np.einsum("hj,jhe->he", p / p.sum(1, keepdims=True), v[lo:i + 1])
    return out


def latent_of(sd, p, mixer, h, eps, rnd=exact):
    """What a layer caches of every token: the normed latent [T, kv_rank] and the rotated key part [T, rot_dim]."""
    R = mixer["kv_rank"]
    d = rnd(h @ sd[p + "dkv"].T)
    return rnd(rms_norm(d[:, :R], sd[p + "dkv.norm"], eps)), rnd(rotate_half(d[:, R:], mixer["rot"]["base"], mixer["rot"]["dims"]))


def latent_attention(sd, p, mixer, h, latent, eps, rnd=exact):
    H, D, P, E = mixer["heads"], mixer["dim"], mixer["rot_dim"], mixer["vdim"]
    T = h.shape[0]
    c, k_rot = latent
    c_q = rnd(rms_norm(rnd(h @ sd[p + "dq"].T), sd[p + "dq.norm"], eps))
    q = rnd(c_q @ sd[p + "uq"].T).reshape(T, H, D + P)
    q_rot = rotate_half(q[..., D:], mixer["rot"]["base"], mixer["rot"]["dims"])
    k = rnd(c @ sd[p + "uk"].T).reshape(T, H, D)
    v = rnd(c @ sd[p + "uv"].T).reshape(T, H, E)
    full_q = rnd(np.concatenate([q[..., :D], q_rot], -1))
    full_k = np.concatenate([k, np.repeat(k_rot[:, None], H, 1)], -1)
    o = sliding_softmax_attention(full_q, full_k, v, mixer["scale"], (mixer.get("mask") or {}).get("size"))
    o = o * sigmoid(h @ sd[p + "g"].T)[..., None]
    return rnd(o.reshape(T, H * E)) @ sd[p + "o"].T


def feed_forward(sd, p, h, rnd=exact):
    gate = h @ sd[p + "gate"].T + sd[p + "gate.b"]
    up = h @ sd[p + "up"].T + sd[p + "up.b"]
    return rnd(silu(gate) * up) @ sd[p + "down"].T + sd[p + "down.b"]


def residual_gate(sd, name, h, rnd=exact):
    return rnd(sigmoid(h @ sd[name].T + sd[name + ".b"]))


def forward(sd, cfg, ids, collect=None, rnd=exact):
    """Logits [T, vocab] of one sequence.  `collect` (a list) receives the residual after every layer."""
    sd = {k: np.asarray(v, np.float64) for k, v in sd.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    ids = np.asarray(ids)
    x = sd["embed"][ids] * cfg["embedding"]["scale"] + sd["pos"][:len(ids)]
    latents = {}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        h1 = group_rms_norm(x, sd[p + "norm1"], groups, eps)
        h = rnd(token_shift(h1, sd[p + "shift"]))
        j = m.get("kv_from")
        if j is None:
            j = i
            latents[i] = latent_of(sd, p + "mix.", m, h, eps, rnd)
        new = x + residual_gate(sd, p + "rg1", rnd(h1), rnd) * latent_attention(sd, p + "mix.", m, h, latents[j], eps, rnd)
        if layer.get("mlp") is not None:
            h2 = rnd(group_rms_norm(x, sd[p + "norm2"], groups, eps))
            new = new + residual_gate(sd, p + "rg2", h2, rnd) * feed_forward(sd, p + "mlp.", h2, rnd)
        x = new
        if collect is not None:
            collect.append(x)
    return rnd(group_rms_norm(x, sd["final.norm"], groups, eps)) @ sd["head"].T
