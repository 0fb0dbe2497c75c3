"""Plain, slow restatement of the Sabolorn decoder in float64 numpy, one function per mechanism.

Test infrastructure only.  Arrays are [tokens, features] of ONE sequence from its first token on, `cfg` is the
model's configuration (the dictionary of its config.json) and `sd` its tensors by name.  Nothing here is shared with the
product path: a sequence is always evaluated as a whole and from scratch, the recurrence token by token, keys and values are
made for every head, every token runs its experts one by one, and nothing is cached.

`rnd` (default: nothing) is applied where a 16-bit evaluation rounds - what enters a matrix product and what a projection
gives - so that tests can measure how much of a difference rounding alone explains.
"""
import numpy as np

from .golapel import exact, plain_frequencies, rms_norm, rotate, sigmoid, yarn_frequencies


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(np.sqrt(2.0 / np.pi) * (z + 0.044715 * z ** 3)))


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def layer_norm(x, w, eps):
    c = x - x.mean(-1, keepdims=True)
    return c / np.sqrt(np.mean(c * c, axis=-1, keepdims=True) + eps) * w


def short_convolution(u, w, bias=None):
    """u [T, C], w [C, taps]: every channel's weighted sum of its newest `taps` values, the last weight being the current one's."""
    taps = w.shape[1]
    before = np.concatenate([np.zeros((taps - 1, u.shape[1])), u])
    y = sum(before[j:j + len(u)] * w[:, j] for j in range(taps))
    return y if bias is None else y + bias


def softmax_attention(q, k, v, scale, penalty=None):
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E], causal; penalty(head, distances) is taken off the scores."""
    T, H = q.shape[:2]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // k.shape[1])
        for i in range(T):
            s = k[:i + 1, g] @ q[i, h] * scale
            if penalty is not None:
                s = s - penalty(h, i - np.arange(i + 1))
            p = np.exp(s - s.max())
            out[i, h] = p @ v[:i + 1, g] / p.sum()
    return out


def log_distance(r1, r2):
    return lambda h, back: r1[h] * np.log(1.0 + r2[h] * back)


# ------------------------------------------------------------------------------------------- mixers
def attention(sd, p, m, h, eps, kept, rnd=exact):
    """Queries, keys and values through short convolutions, positions as a logarithmic penalty of the distance."""
    H, G, D, E, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], h.shape[0]
    q, k, v = (rnd(short_convolution(rnd(h @ sd[p + n].T + sd[p + n + ".b"]), sd[p + n + ".conv"])) for n in "qkv")
    o = softmax_attention(q.reshape(T, H, D), k.reshape(T, G, D), v.reshape(T, G, E), m["scale"], log_distance(sd[p + "r1"], sd[p + "r2"]))
    return rnd(o.reshape(T, -1)) @ sd[p + "o"].T


def rotation_of(rot):
    s = rot.get("scaling")
    if s is None:
        return plain_frequencies(rot["base"], rot["dims"]), 1.0
    return yarn_frequencies(rot["base"], rot["dims"], s["factor"], s["original"], s["fast"], s["slow"])


def latent_attention(sd, p, m, h, eps, kept, rnd=exact):
    """Keys and values from a latent and one rotated key part; `kept` holds what the layers before have left, by layer."""
    H, D, P, E, R, T = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], h.shape[0]
    f, amplitude = rotation_of(m["rot"])
    turn = lambda x: rotate(x, f, amplitude, interleaved=True)
    c_q = rnd(rms_norm(rnd(h @ sd[p + "dq"].T), sd[p + "dq.norm"], eps))
    q = rnd(c_q @ sd[p + "uq"].T).reshape(T, H, D + P)
    q = np.concatenate([q[..., :D], rnd(turn(q[..., D:]))], -1)
    if m.get("kv_from") is None:
        c = rnd(h @ sd[p + "dkv"].T)
        kept[p] = rnd(rms_norm(c[:, :R], sd[p + "dkv.norm"], eps)), rnd(turn(c[:, R:]))
        source = p
    else:
        source = f"l{m['kv_from']}.mix."
    c, shared = kept[source]
    k = np.concatenate([rnd(c @ sd[p + "uk"].T).reshape(T, H, D), np.repeat(shared[:, None], H, 1)], -1)
    v = rnd(c @ sd[p + "uv"].T).reshape(T, H, E)
    o = softmax_attention(q, k, v, m["scale"]).reshape(T, -1) * sigmoid(rnd(h @ sd[p + "g"].T))
    return rnd(o) @ sd[p + "o"].T


def state_space(x, B, C, dt, A_log, D):
    """x [T, H, E], B and C [T, G, N], dt [T, H] (positive): S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x."""
    T, H, E = x.shape
    G, N = B.shape[1:]
    y, S = np.zeros((T, H, E)), np.zeros((H, N, E))
    for t in range(T):
        for h in range(H):
            g = h // (H // G)
            S[h] = np.exp(-np.exp(A_log[h]) * dt[t, h]) * S[h] + dt[t, h] * np.outer(B[t, g], x[t, h])
            y[t, h] = S[h].T @ C[t, g] + D[h] * x[t, h]
    return y


def gated_group_norm(y, z, w, groups, eps):
    """y silu(z), each of `groups` equal parts over its own root mean square, times w."""
    parts = (y * silu(z)).reshape(len(y), groups, -1)
    return (parts / np.sqrt(np.mean(parts ** 2, -1, keepdims=True) + eps)).reshape(y.shape) * w


def mamba2(sd, p, m, h, eps, kept, rnd=exact):
    H, E, N, G, T = m["heads"], m["vdim"], m["state"], m["groups"], h.shape[0]
    inner = H * E
    full = h @ sd[p + "in"].T
    z, u, dt = rnd(full[:, :inner]), rnd(full[:, inner:2 * inner + 2 * G * N]), full[:, 2 * inner + 2 * G * N:]
    u = rnd(silu(short_convolution(u, sd[p + "conv"], sd[p + "conv.b"])))
    x, B, C = u[:, :inner].reshape(T, H, E), u[:, inner:inner + G * N].reshape(T, G, N), u[:, inner + G * N:].reshape(T, G, N)
    y = state_space(x, B, C, softplus(dt + sd[p + "dt_bias"]), sd[p + "A_log"], sd[p + "D"]).reshape(T, inner)
    return rnd(gated_group_norm(y, z, sd[p + "norm"], m["norm_groups"], eps)) @ sd[p + "o"].T


MIXERS = {"attention": attention, "latent_attention": latent_attention, "mamba2": mamba2}


# ------------------------------------------------------------------------------------------- feed-forwards
def dense(sd, p, h, rnd=exact):
    return rnd(np.maximum(h @ sd[p + "up"].T, 0.0) ** 2) @ sd[p + "down"].T


def expert(sd, p, h, rnd=exact):
    return rnd(silu(h @ sd[p + "gate"].T) * (h @ sd[p + "up"].T)) @ sd[p + "down"].T


def route(z, correction, top, groups=1, keep=1):
    """Router logits z [experts] of one token -> (chosen experts, their weights).  Chosen are the best by sigmoid score and
    correction among the groups whose two best sum up highest; the weights are the scores alone, as shares of their sum."""
    s = sigmoid(z)
    c = s + correction
    size = len(z) // groups
    best_two = [np.sort(c[g * size:(g + 1) * size])[-2:].sum() for g in range(groups)]
    kept = np.argsort(-np.array(best_two), kind="stable")[:keep]
    open_ = np.isin(np.arange(len(z)) // size, kept)
    chosen = np.argsort(-np.where(open_, c, -np.inf), kind="stable")[:top]
    return chosen, s[chosen] / (s[chosen].sum() + 1e-20)


def experts(sd, p, f, h, rnd=exact):
    r = f["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    z = h @ sd[p + "router"].T
    y = np.zeros_like(h)
    for t in range(len(h)):
        for e, w in zip(*route(z[t], sd[p + "correction"], r["top"], g["count"], g["keep"])):
            y[t] += w * expert(sd, f"{p}e{e}.", h[t], rnd)
    return y


# ------------------------------------------------------------------------------------------- a layer's end
def token_input(sd, p, x, e, eps, rnd=exact):
    """x plus the normed projection of the token's own part of this layer, gated by x."""
    g = gelu_tanh(rnd(x) @ sd[p + "side.gate"].T) * e
    return x + rms_norm(rnd(g) @ sd[p + "side.proj"].T, sd[p + "side.norm"], eps)


def depth_average(history, w):
    return sum(a * x for a, x in zip(w, history))


def forward(sd, cfg, ids, collect=None, rnd=exact):
    """Logits [T, vocab] of one sequence.  `collect` (a list) receives the residual after every layer."""
    sd = {k: np.asarray(v, np.float64) for k, v in sd.items()}
    eps, ids = cfg["norm"]["eps"], np.asarray(ids)
    x = sd["embed"][ids] * cfg["embedding"]["scale"]
    n = cfg["token_side"]["dim"]
    history, kept = [x], {}
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = rnd(layer_norm(x, sd[p + "norm1"], eps))
        y = MIXERS[layer["type"]](sd, p + "mix.", layer["mixer"], h, eps, kept, rnd)
        f = layer.get("mlp")
        if f is not None:
            y = y + (dense(sd, p + "mlp.", h, rnd) if f["kind"] == "dense" else experts(sd, p + "mlp.", f, h, rnd))
        x = token_input(sd, p, x + y, sd["side.embed"][ids, i * n:(i + 1) * n], eps, rnd)
        history.append(x)
        x = depth_average(history, sd[p + "dwa"])
        if collect is not None:
            collect.append(x)
    logits = rnd(layer_norm(x, sd["final.norm"], eps)) @ sd["embed"].T
    cap = cfg.get("logit_softcap")
    return cap * np.tanh(logits / cap) if cap else logits
