"""Plain, slow restatement of the Golapel decoder in float64 numpy, one function per mechanism.

Test infrastructure only.  Arrays are [tokens, features] of ONE sequence from its first token on, `cfg` is the
model's configuration (the dictionary of its config.json) and `sd` its tensors by name.  Nothing here is shared with the
product path: a sequence is always evaluated as a whole and from scratch, every token runs its experts one by one, and
nothing is cached.

`rnd` (default: nothing) is applied where a 16-bit evaluation rounds - what enters a matrix product and what a projection
gives - so that tests can measure how much of a difference rounding alone explains.
"""
import math

import numpy as np


def exact(a):
    return a


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def rms_norm(x, w, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


# ------------------------------------------------------------------------------------------- rotation
def plain_frequencies(base, dims):
    return float(base) ** (-2.0 * np.arange(dims // 2) / dims)


def linear_frequencies(base, dims, factor):
    return plain_frequencies(base, dims) / factor


def yarn_frequencies(base, dims, factor, original, fast, slow):
    """Slow features are interpolated, fast ones kept, a linear ramp between them; (frequencies, factor of cos and sin)."""
    def turns(t):                            # the feature that makes t turns within `original` positions
        return dims * math.log(original / (2 * math.pi * t)) / (2 * math.log(base))
    lo, hi = max(math.floor(turns(fast)), 0), min(math.ceil(turns(slow)), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    f = plain_frequencies(base, dims)
    return f / factor * ramp + f * (1 - ramp), 0.1 * math.log(factor) + 1.0


def rotate(x, frequencies, amplitude=1.0, interleaved=False):
    """x [T, ..., n]: feature pairs of the first 2 * len(frequencies) turned by position * frequency; the pairs are (i, i + half)
    or (2 i, 2 i + 1)."""
    half = len(frequencies)
    angle = (np.arange(x.shape[0])[:, None] * frequencies).reshape((x.shape[0],) + (1,) * (x.ndim - 2) + (half,))
    c, s = np.cos(angle) * amplitude, np.sin(angle) * amplitude
    y = np.array(x, np.float64)
    first, second = (slice(0, 2 * half, 2), slice(1, 2 * half, 2)) if interleaved else (slice(0, half), slice(half, 2 * half))
    u, v = x[..., first], x[..., second]
    y[..., first], y[..., second] = u * c - v * s, v * c + u * s
    return y


# ------------------------------------------------------------------------------------------- attention
def window_mask(T, size=None, keep_first=0):
    """[query, key]: the newest `size` positions (None: all of them) and the first `keep_first`."""
    i, j = np.arange(T)[:, None], np.arange(T)[None]
    near = j <= i if size is None else (j <= i) & (i - j < size)
    return near | ((j <= i) & (j < keep_first))


def chunk_mask(T, size=None):
    i, j = np.arange(T)[:, None], np.arange(T)[None]
    return j <= i if size is None else (j <= i) & (i // size == j // size)


def attend(q, k, v, scale, mask, sink=None):
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]; sink [H]: a score in the denominator that has no value."""
    T, H = q.shape[:2]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // k.shape[1])
        for i in range(T):
            js = np.flatnonzero(mask[i])
            s = k[js, g] @ q[i, h] * scale
            top = s.max() if sink is None else max(s.max(), sink[h])
            p = np.exp(s - top)
            z = p.sum() + (0.0 if sink is None else np.exp(sink[h] - top))
            out[i, h] = p @ v[js, g] / z
    return out


def project(sd, name, h):
    y = h @ sd[name].T
    return y + sd[name + ".b"] if name + ".b" in sd else y


def sink_attention(sd, p, m, h, eps, rnd=exact):
    """Values that are the projected keys, rotation in halves, a window that keeps the first tokens, sinks, a gate per head."""
    H, G, D, T = m["heads"], m["kv_heads"], m["dim"], h.shape[0]
    q, v = rnd(project(sd, p + "q", h)).reshape(T, H, D), rnd(project(sd, p + "k", h)).reshape(T, G, D)
    q, k = rms_norm(q, sd[p + "q.norm"], eps), rms_norm(v, sd[p + "k.norm"], eps)
    if m.get("rot") is not None:
        r = m["rot"]
        f = linear_frequencies(r["base"], r["dims"], r["scaling"]["factor"]) if r.get("scaling") else plain_frequencies(r["base"], r["dims"])
        q, k = rotate(q, f), rotate(k, f)
    mask = m.get("mask") or {}
    o = attend(rnd(q), rnd(k), v, m["scale"], window_mask(T, mask.get("size"), mask.get("keep_first") or 0), sd[p + "sink"])
    o = o * sigmoid(h @ sd[p + "g"].T)[..., None]
    return rnd(o.reshape(T, -1)) @ sd[p + "o"].T


def differential_combine(a1, a2, lam, diff, eps):
    o = a1 - lam * a2
    return o / np.sqrt(np.mean(o * o, axis=-1, keepdims=True) + eps) * (1.0 - diff)


def differential_lambda(sd, p, diff):
    return np.exp(np.sum(sd[p + "lq1"] * sd[p + "lk1"])) - np.exp(np.sum(sd[p + "lq2"] * sd[p + "lk2"])) + diff


def differential_attention(sd, p, m, h, eps, rnd=exact):
    """Two attentions over the same values within chunks, one subtracted from the other; no positions in the scores."""
    H, G, D, E, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q, k = rnd(project(sd, p + "q", h)).reshape(T, H, 2, D), rnd(project(sd, p + "k", h)).reshape(T, G, 2, D)
    v = rnd(project(sd, p + "v", h)).reshape(T, G, E)
    q, k = rnd(rms_norm(q, sd[p + "q.norm"], eps)), rnd(rms_norm(k, sd[p + "k.norm"], eps))
    mask = chunk_mask(T, (m.get("mask") or {}).get("size"))
    a1, a2 = (attend(q[:, :, t], k[:, :, t], v, m["scale"], mask) for t in (0, 1))
    o = differential_combine(a1, a2, differential_lambda(sd, p, m["diff"]), m["diff"], eps)
    return rnd(o.reshape(T, -1)) @ sd[p + "o"].T


def chunk_attention(sd, p, m, h, eps, rnd=exact):
    """Attention within chunks, rotation of neighbours with stretched frequencies, a gate per feature."""
    H, G, D, E, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q, k = rnd(project(sd, p + "q", h)).reshape(T, H, D), rnd(project(sd, p + "k", h)).reshape(T, G, D)
    v = rnd(project(sd, p + "v", h)).reshape(T, G, E)
    q, k = rms_norm(q, sd[p + "q.norm"], eps), rms_norm(k, sd[p + "k.norm"], eps)
    if m.get("rot") is not None:
        r = m["rot"]
        f, amp = yarn_frequencies(r["base"], r["dims"], **r["scaling"]) if r.get("scaling") else (plain_frequencies(r["base"], r["dims"]), 1.0)
        q, k = rotate(q, f, amp, True), rotate(k, f, amp, True)
    o = attend(rnd(q), rnd(k), v, m["scale"], chunk_mask(T, (m.get("mask") or {}).get("size")))
    o = o.reshape(T, -1) * sigmoid(rnd(h @ sd[p + "g"].T))
    return rnd(o) @ sd[p + "o"].T


MIXERS = {"attention": sink_attention, "attention_2": differential_attention, "attention_3": chunk_attention}


# ------------------------------------------------------------------------------------------- feed-forward
def dense(sd, p, h, rnd=exact):
    g = h @ sd[p + "gate"].T
    return rnd(g * sigmoid(g) * (h @ sd[p + "up"].T)) @ sd[p + "down"].T


def clamped_expert(sd, p, h, limit, rnd=exact):
    g, u = np.minimum(h @ sd[p + "gate"].T, limit), np.clip(h @ sd[p + "up"].T, -limit, limit)
    return rnd(g * sigmoid(1.702 * g) * (u + 1.0)) @ sd[p + "down"].T


def route(z, top, scale):
    """Router logits z [T, experts] -> (chosen experts [T, top], their weights): softmax scores, not renormalised."""
    s = np.exp(z - z.max(-1, keepdims=True))
    s /= s.sum(-1, keepdims=True)
    chosen = np.argsort(-s, axis=-1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, -1) * scale


def experts(sd, p, f, h, rnd=exact):
    chosen, weight = route(h @ sd[p + "router"].T, f["router"]["top"], f["router"]["scale"])
    y = np.zeros((h.shape[0], h.shape[1]))
    for t in range(h.shape[0]):
        for e, w in zip(chosen[t], weight[t]):
            y[t] += w * clamped_expert(sd, f"{p}e{e}.", h[t], f["expert"]["limit"], rnd)
    if f.get("shared") is not None:
        y += sigmoid(h @ sd[p + "shared.sg"].T) * clamped_expert(sd, p + "shared.", h, f["shared"]["limit"], rnd)
    return y


def forward(sd, cfg, ids, collect=None, rnd=exact):
    """Logits [T, vocab] of one sequence.  `collect` (a list) receives the residual after every layer."""
    sd = {k: np.asarray(v, np.float64) for k, v in sd.items()}
    eps = cfg["norm"]["eps"]
    x = sd["embed"][np.asarray(ids)] * cfg["embedding"]["scale"]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + rms_norm(MIXERS[layer["type"]](sd, p + "mix.", layer["mixer"], rnd(x), eps, rnd), sd[p + "norm1"], eps)
        f = layer.get("mlp")
        if f is not None:
            y = dense(sd, p + "mlp.", rnd(x), rnd) if f["kind"] == "dense" else experts(sd, p + "mlp.", f, rnd(x), rnd)
            x = x + rms_norm(y, sd[p + "norm2"], eps)
        if collect is not None:
            collect.append(x)
    return rnd(rms_norm(x, sd["final.norm"], eps)) @ sd["embed"].T
