"""Decoders whose results are averaged over the depths without a GPU: the oracle's mechanisms against independent forms, the
recorded graph against the oracle, what the compiler and the loader read, and the cache."""
import json

import numpy as np
import pytest
import torch

from oracle import sabolorn as S
from tests.depth_models import DEPTH, attention, config, dense, latent, mamba, moe, random_depth
from tests.hybrid_models import token_ids
from tests.test_hybrid_cpu import _HostInterpreter


# ------------------------------------------------------------------------------------------- oracle pins
def test_small_functions_against_torch():
    rng = np.random.default_rng(0)
    x, w = rng.standard_normal((5, 30)) * 4, rng.standard_normal(30)
    t, F = torch.from_numpy(x), torch.nn.functional
    assert np.allclose(S.silu(x), F.silu(t).numpy()) and np.allclose(S.softplus(9 * x), F.softplus(9 * t).numpy())
    assert np.allclose(S.gelu_tanh(x), F.gelu(t, approximate="tanh").numpy())
    assert np.allclose(S.layer_norm(x, w, 1e-3), F.layer_norm(t, (30,), torch.from_numpy(w), None, 1e-3).numpy())
    got = S.gated_group_norm(x, x[::-1], w, 3, 1e-3)
    want = np.concatenate([F.rms_norm((t * F.silu(t.flip(0)))[:, k:k + 10], (10,), None, 1e-3).numpy() for k in (0, 10, 20)], 1) * w
    assert np.allclose(got, want)


@pytest.mark.parametrize("taps", [1, 2, 5])
def test_short_convolution_against_torch(taps):
    rng = np.random.default_rng(1)
    u, w, b = rng.standard_normal((12, 7)), rng.standard_normal((7, taps)), rng.standard_normal(7)
    padded = torch.nn.functional.pad(torch.from_numpy(u.T), (taps - 1, 0))
    want = torch.nn.functional.conv1d(padded[None], torch.from_numpy(w)[:, None], torch.from_numpy(b), groups=7)[0].T.numpy()
    assert np.allclose(S.short_convolution(u, w, b), want) and np.allclose(S.short_convolution(u, w), want - b)
    assert np.allclose(S.short_convolution(u, w)[0], u[0] * w[:, -1])          # zeros before the start


def test_attention_against_a_masked_softmax():
    rng = np.random.default_rng(2)
    T, H, G, D, E = 15, 6, 2, 8, 5
    q, k, v = rng.standard_normal((T, H, D)), rng.standard_normal((T, G, D)), rng.standard_normal((T, G, E))
    r1, r2 = rng.uniform(0, 2, H), rng.uniform(0, 1, H)
    back = np.arange(T)[:, None] - np.arange(T)[None]
    mask = np.where(back >= 0, 0.0, -np.inf) - r1[:, None, None] * np.log1p(r2[:, None, None] * back.clip(0))
    tq, tk, tv = (torch.from_numpy(np.repeat(a, r, 1)).transpose(0, 1)[None] for a, r in ((q, 1), (k, 3), (v, 3)))
    want = torch.nn.functional.scaled_dot_product_attention(tq, tk, tv, attn_mask=torch.from_numpy(mask)[None], scale=0.37)
    assert np.allclose(S.softmax_attention(q, k, v, 0.37, S.log_distance(r1, r2)), want[0].transpose(0, 1).numpy())


def test_the_recurrence_is_a_weighted_sum_over_the_past():
    """y_t = sum_{s <= t} exp(-exp(A) sum of the steps after s) dt_s (c_t . b_s) x_s + D x_t"""
    rng = np.random.default_rng(3)
    T, H, G, N, E = 13, 4, 2, 6, 5
    x, b, c = rng.standard_normal((T, H, E)), rng.standard_normal((T, G, N)), rng.standard_normal((T, G, N))
    dt, A, D = rng.uniform(0.01, 1, (T, H)), rng.uniform(-2, 1, H), rng.standard_normal(H)
    got = S.state_space(x, b, c, dt, A, D)
    for h in range(H):
        run = np.cumsum(dt[:, h])
        w = np.exp(-np.exp(A[h]) * (run[:, None] - run[None])) * dt[None, :, h] * (c[:, h // 2] @ b[:, h // 2].T)
        assert np.allclose(got[:, h], np.tril(w) @ x[:, h] + D[h] * x[:, h])


def test_router():
    c = np.array([0.0, 0.0, 0.0, 0.0, -0.5, 0.0])
    z = np.array([2.0, -3.0, 1.0, 0.5, 3.0, -1.0])
    s = 1 / (1 + np.exp(-z))
    chosen, w = S.route(z, c, 2)
    assert list(chosen) == [0, 2] and np.allclose(w, s[[0, 2]] / s[[0, 2]].sum())          # the correction keeps 4 away
    assert list(S.route(z, 0 * c, 2)[0]) == [4, 0]
    # two groups of three: .88 + .73 against .95 + .62; an expert of the other group is not taken though it is better
    chosen, w = S.route(z, 0 * c, 3, 2, 1)
    assert list(chosen) == [0, 2, 1] and np.allclose(w.sum(), 1)
    # negative choice scores: experts of closed groups do not come in as zeros
    assert list(S.route(z, c - 9, 3, 2, 1)[0]) == [0, 2, 1]
    assert list(S.route(z, 0 * c, 2, 3, 2)[0]) == [4, 2]                                   # sums .93, 1.35, 1.22


def test_choices_in_the_tests_models_are_not_close(monkeypatch):
    gaps, plain = [], S.route

    def route(z, c, top, groups=1, keep=1):
        chosen, w = plain(z, c, top, groups, keep)
        s, size = S.sigmoid(z) + c, len(z) // groups
        two = np.array([np.sort(s[k * size:(k + 1) * size])[-2:].sum() for k in range(groups)])
        order = np.argsort(-two)
        if keep < groups:
            gaps.append(two[order[keep - 1]] - two[order[keep]])
        rest = [s[e] for e in range(len(z)) if e // size in order[:keep] and e not in chosen]
        gaps.extend([s[chosen].min() - max(rest)] if rest else [])
        return chosen, w
    monkeypatch.setattr(S, "route", route)
    for name, cfg in DEPTH.items():
        S.forward(random_depth(cfg, 5), cfg, token_ids(1, 40, cfg))
    assert min(gaps) > 0.03


# ------------------------------------------------------------------------------------------- recorded graph
def _recorded(cfg, sd, B, L, steps, precision="fp32"):
    from poptransformer_amd.models.sabolorn import SabolornDecModel
    from poptransformer_amd.utils import REGISTRY, register_global_args
    REGISTRY.reset()
    register_global_args({"batch_size": B, "precision": precision})
    m = SabolornDecModel(hf_config=cfg, state_dict=sd, pad_token_id=0, eos_token_id=1, max_length=L, max_loop=steps)
    m.build_graph()
    return m


@pytest.mark.parametrize("name", ["small", "odd", "alike"])
def test_the_recorded_graph_is_the_model(name):
    cfg = DEPTH[name]
    B, L, steps = 2, 40, 34
    sd = random_depth(cfg, 11)
    m = _recorded(cfg, sd, B, L, steps)
    it = _HostInterpreter(m.graph).it
    it.input_trace = {"aiOnnx.topk": []}
    ids = np.zeros((B, L), np.int32)
    ids[0, :7] = np.random.default_rng(0).integers(2, cfg["vocab"], 7)
    ids[1, :2] = [5, 9]
    it.run_graph(m.graph, {"input_ids": torch.from_numpy(ids)})
    logits = [x[0].reshape(B, -1) for x in it.input_trace["aiOnnx.topk"]]
    assert len(logits) == steps
    container = ids.copy()
    for t in range(steps):                                      # the loop: a stored prompt token wins
        for b in range(B):
            if container[b, t + 1] == 0:
                container[b, t + 1] = logits[t][b].argmax()
    assert name != "small" or len(set(container[0, 8:steps])) > 3                        # (generation does not stand still)
    for b in range(B):
        want = S.forward(sd, cfg, container[b, :steps])
        got = np.stack([x[b] for x in logits])
        assert np.abs(got - want).max() < 2e-4 * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("name", list(DEPTH))
def test_the_compiler_reads_the_model_off_the_graph(monkeypatch, name):
    """Specification and tensors that the compiler recovers from the recorded graph equal those of the configuration."""
    from poptransformer_amd.engine import compiler, depth, loader
    cfg = json.loads(json.dumps(DEPTH[name]))
    first = [lay for lay in cfg["layers"] if lay["type"] == "latent_attention"][-1]
    if first["mixer"].get("kv_from") is None:
        first["mixer"]["rot"]["base"] = 1234567.891             # not an fp32 number
    sd = random_depth(cfg, 2)
    facts = compiler.GraphFacts(_recorded(cfg, sd, 3, 50, 10, "bf16").graph)
    assert compiler._family(facts) == "sabolorn" and compiler._sampling_k(facts) == 1
    seen = {}
    monkeypatch.setattr(loader, "depth_weights", lambda tensors, spec: seen.update(tensors=tensors))
    monkeypatch.setattr(depth, "DepthDecoder", lambda spec, w: spec)
    got = compiler._build_depth(facts)
    want = loader.sabolorn_spec(cfg, 50, 3, pad_id=0, eos_id=1)
    assert got == want
    assert all(np.array_equal(seen["tensors"][k], v) for k, v in sd.items())


# ------------------------------------------------------------------------------------------- configuration, cache, angles
def test_configurations_that_do_not_exist_are_refused():
    from poptransformer_amd.engine import registry
    from poptransformer_amd.engine.loader import depth_layers
    for bad in (dict(mamba(), type="other"), mamba(mlp=dict(dense(), kind="other"))):
        with pytest.raises(NotImplementedError):
            depth_layers([bad])
    for bad in ([latent(of=0)], [mamba(), latent(of=0)], [latent(), latent(of=0), latent(of=1)], [latent(), latent(of=0, kv_rank=32)],
                [latent(), latent(of=0, base=61.0)], [latent(rot_dim=7)], [attention(heads=5)], [mamba(groups=3)], [mamba(norm_groups=7)],
                [mamba(mlp=moe(experts=8, top=5))], [mamba(mlp=moe(experts=9))]):
        with pytest.raises(ValueError):
            depth_layers(bad)
    assert registry.architecture({"architecture": "Sabolorn"})[1] == ("hybrid",)


def test_cache_state_and_growth(monkeypatch):
    from poptransformer_amd import hybrid_kernels as HK
    from poptransformer_amd.engine.loader import sabolorn_spec
    from poptransformer_amd.engine.sequences import SequenceStore
    monkeypatch.setattr(HK, "ssd_state", lambda slots, heads, dim, vdim, device: torch.zeros(slots, heads * dim * vdim))
    cfg = config([latent(), mamba(state=21, vdim=20, taps=3), attention(dim=10, vdim=13, taps=5), latent(of=0), mamba(taps=1)])
    store = SequenceStore(sabolorn_spec(cfg, 600, 1), torch.float32, 2, 600, 50, device="cpu")
    assert store.stores[0][0].shape == (2, 640, 64) and store.stores[3] == ()
    assert store.stores[1][0].shape == (2, 4 * 24 * 24) and store.recent[1].shape == (2, 3, 4 * 24 + 2 * 2 * 24)
    assert [t.shape for t in store.stores[2]] == [(2, 2, 1, 640, 16), (2, 2, 640, 16)] and store.recent[2].shape == (2, 5, 8 * 16 + 2 * 16)
    assert store.recent[0] is None and store.recent[4].shape[1] == 1
    store.recent[2][1], store.stores[1][0][1] = 3.0, 4.0
    for _ in range(3):
        store.open()                                            # the third does not fit: what is there moves along
    assert store.capacity == 4 and (store.recent[2][1] == 3).all() and (store.stores[1][0][1] == 0).all()       # (opened: from the start)
    assert store.nbytes == sum(t.numel() * 4 for s in store.stores for t in s) + sum(t.numel() * 4 for t in store.recent if t is not None)


def test_numbers_of_the_mixers_come_back():
    from poptransformer_amd.engine.hybrid import Experts, HeadMixer, LatentMixer, Rotation, StateSpaceMixer
    from poptransformer_amd.engine.loader import depth_layers
    layers = depth_layers([latent(mlp=moe(groups=(4, 2), experts=12)), latent(of=0, scaling=(3.0, 64, 4.0, 1.0)), mamba(), attention(heads=4, taps=3)])
    a, b, c, d = (lay.mixer for lay in layers)
    for m in (a, b):
        assert LatentMixer.of(m.numbers(), m.dim, m.rot_dim, m.vdim, m.q_rank, m.kv_rank, Rotation.of(m.rot.numbers())) == m
    assert StateSpaceMixer.of(c.numbers()) == c and HeadMixer.of(d.numbers(), d.dim, d.vdim, d.biases, None) == d
    e = layers[0].mlp
    assert Experts.of(e.numbers(), e.expert) == e and (e.groups, e.keep, e.share, e.corrected, e.score) == (4, 2, True, True, "sigmoid")


def test_rotated_pairs_and_angles_of_a_latent():
    from poptransformer_amd.engine.loader import depth_layers
    for layer in (latent(rot_dim=6, scaling=None), latent(rot_dim=40, base=1e4, scaling=(8.0, 100, 8.0, 0.5))):
        m = depth_layers([layer])[0].mixer
        f, amplitude = S.rotation_of(layer["mixer"]["rot"])
        x = np.random.default_rng(0).standard_normal((50, m.rot_dim))
        cs, n = m.angles(50), m.rot_dim // 2
        assert cs.shape == (50, (m.rot_dim + 31) // 32 * 16, 2) and (cs[:, n:] == [1.0, 0.0]).all()
        u, v = x[:, 0::2], x[:, 1::2]
        got = np.stack([u * cs[:, :n, 0] - v * cs[:, :n, 1], v * cs[:, :n, 0] + u * cs[:, :n, 1]], -1).reshape(50, -1)
        assert np.array_equal(m.pairs(), np.arange(m.rot_dim)) and np.allclose(got, S.rotate(x, f, amplitude, True), atol=1e-5)
