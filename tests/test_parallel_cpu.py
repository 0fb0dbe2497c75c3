"""Decoders with latent attention and parallel sublayers without a GPU: the oracle's mechanisms against independent forms,
the recorded graph against the oracle, what the compiler and the loader read."""
import json

import numpy as np
import pytest
import torch

from oracle import ruperax as R
from tests.parallel_models import PARALLEL, latent, parallel_config, random_parallel, small_parallel
from tests.test_hybrid_cpu import _HostInterpreter


# ------------------------------------------------------------------------------------------- oracle pins
def test_norms_against_torch():
    rng = np.random.default_rng(0)
    x, w = rng.standard_normal((5, 30)), rng.standard_normal(30)
    t = torch.from_numpy(x)
    assert np.allclose(R.rms_norm(x, w, 1e-3), torch.nn.functional.rms_norm(t, (30,), torch.from_numpy(w), 1e-3).numpy(), atol=1e-12)
    want = np.concatenate([torch.nn.functional.rms_norm(t[:, k:k + 10], (10,), None, 1e-3).numpy() for k in (0, 10, 20)], 1) * w
    assert np.allclose(R.group_rms_norm(x, w, 3, 1e-3), want, atol=1e-12)
    assert np.allclose(R.group_rms_norm(x, w, 1, 1e-3), R.rms_norm(x, w, 1e-3))
    assert np.allclose(R.silu(9 * x), torch.nn.functional.silu(9 * t).numpy())


def test_token_shift_reads_the_token_before():
    h = np.arange(12.0).reshape(4, 3)
    got = R.token_shift(h, np.array([0.0, 1.0, 0.25]))
    assert np.array_equal(got[:, 0], h[:, 0])                          # nothing of the token before
    assert np.array_equal(got[:, 1], [0, 1, 4, 7])                     # all of it, zeros before the first
    assert np.allclose(got[:, 2], [1.5, 4.25, 7.25, 10.25])


def test_rotation_is_a_complex_product_and_depends_on_distance():
    rng = np.random.default_rng(1)
    x = rng.standard_normal((9, 2, 11))
    got = R.rotate_half(x, 7.0, 8)
    z = (x[..., :4] + 1j * x[..., 4:8]) * np.exp(1j * np.arange(9)[:, None, None] * 7.0 ** (-np.arange(4) / 4))
    assert np.allclose(got, np.concatenate([z.real, z.imag, x[..., 8:]], -1))
    q, k = (np.repeat(rng.standard_normal((1, 8)), 9, 0) for _ in range(2))
    a, b = R.rotate_half(q, 7.0, 8), R.rotate_half(k, 7.0, 8)
    assert np.isclose(a[5] @ b[2], a[8] @ b[5]) and not np.isclose(a[5] @ b[2], a[8] @ b[2])


@pytest.mark.parametrize("window", [1, 5, None])
def test_attention_against_a_masked_softmax(window):
    rng = np.random.default_rng(2)
    T, H, D, E = 20, 3, 8, 5
    q, k, v = rng.standard_normal((T, H, D)), rng.standard_normal((T, H, D)), rng.standard_normal((T, H, E))
    dist = np.arange(T)[:, None] - np.arange(T)[None]
    mask = torch.from_numpy((dist >= 0) & (dist < (window or T)))
    tq, tk, tv = (torch.from_numpy(a).transpose(0, 1) for a in (q, k, v))
    want = torch.nn.functional.scaled_dot_product_attention(tq, tk, tv, mask, scale=0.7).transpose(0, 1).numpy()
    assert np.allclose(R.sliding_softmax_attention(q, k, v, 0.7, window), want, atol=1e-12)


def test_a_layer_that_reads_another_ones_cache():
    """Equal to a layer that makes the very same latents itself: with the other layer's input they are the same, with its own
    they are not."""
    cfg = parallel_config([latent(window=5), latent(window=5, of=0)])
    sd = random_parallel(cfg, 3)
    rng = np.random.default_rng(0)
    m, h0, h1 = cfg["layers"][1]["mixer"], rng.standard_normal((8, 84)), rng.standard_normal((8, 84))
    own = {**{k.replace("l1.", "l9."): v for k, v in sd.items() if k.startswith("l1.")}, "l9.mix.dkv": sd["l0.mix.dkv"],
           "l9.mix.dkv.norm": sd["l0.mix.dkv.norm"]}
    shared = R.latent_attention(sd, "l1.mix.", m, h1, R.latent_of(sd, "l0.mix.", m, h0, 1e-5), 1e-5)
    assert np.allclose(shared, R.latent_attention(own, "l9.mix.", m, h1, R.latent_of(own, "l9.mix.", m, h0, 1e-5), 1e-5))
    assert not np.allclose(shared, R.latent_attention(own, "l9.mix.", m, h1, R.latent_of(own, "l9.mix.", m, h1, 1e-5), 1e-5))


def test_the_products_can_be_taken_in_another_order():
    """q . (W_uk c) = (W_uk^T q) . c and sum p (W_uv c) = W_uv sum p c: what decoding relies on."""
    cfg = small_parallel()
    sd = random_parallel(cfg, 4)
    m, eps = cfg["layers"][0]["mixer"], 1e-5
    H, D, P, E = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    h = np.random.default_rng(1).standard_normal((20, 84))
    c, k_rot = R.latent_of(sd, "l0.mix.", m, h, eps)
    q = (R.rms_norm(h @ sd["l0.mix.dq"].T, sd["l0.mix.dq.norm"], eps) @ sd["l0.mix.uq"].T).reshape(20, H, D + P)
    q_rot = R.rotate_half(q[..., D:], m["rot"]["base"], P)
    uk, uv = sd["l0.mix.uk"].reshape(H, D, -1), sd["l0.mix.uv"].reshape(H, E, -1)
    absorbed = np.concatenate([np.einsum("thd,hdr->thr", q[..., :D], uk), q_rot], -1)
    keys = np.repeat(np.concatenate([c, k_rot], -1)[:, None], H, 1)
    o = np.einsum("thr,her->the", R.sliding_softmax_attention(absorbed, keys, np.repeat(c[:, None], H, 1), m["scale"], 12), uv)
    o = o * R.sigmoid(h @ sd["l0.mix.g"].T)[..., None]
    assert np.allclose(o.reshape(20, -1) @ sd["l0.mix.o"].T, R.latent_attention(sd, "l0.mix.", m, h, (c, k_rot), eps))


# ------------------------------------------------------------------------------------------- recorded graph
def _recorded(cfg, sd, B, L, steps, precision="fp32"):
    from poptransformer_amd.models.ruperax import RuperaxDecModel
    from poptransformer_amd.utils import REGISTRY, register_global_args
    REGISTRY.reset()
    register_global_args({"batch_size": B, "precision": precision})
    m = RuperaxDecModel(hf_config=cfg, state_dict=sd, pad_token_id=0, eos_token_id=1, max_length=L, max_loop=steps)
    m.build_graph()
    return m


@pytest.mark.parametrize("name", ["small", "odd", "alike"])
def test_the_recorded_graph_is_the_model(name):
    cfg = PARALLEL[name]
    B, L, steps = 2, 40, 34
    sd = random_parallel(cfg, 1)
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
    for b in range(B):
        want = R.forward(sd, cfg, container[b, :steps])
        got = np.stack([x[b] for x in logits])
        assert np.abs(got - want).max() < 2e-4 * max(1.0, np.abs(want).max())


def test_the_compiler_reads_the_model_off_the_graph(monkeypatch):
    """Specification and tensors that the compiler recovers from the recorded graph equal those of the configuration."""
    from poptransformer_amd.engine import compiler, loader, parallel
    cfg = small_parallel()
    cfg["layers"][0]["mixer"]["rot"]["base"] = cfg["layers"][1]["mixer"]["rot"]["base"] = 1234567.891       # not an fp32 number
    sd = random_parallel(cfg, 2)
    facts = compiler.GraphFacts(_recorded(cfg, sd, 3, 50, 10, "bf16").graph)
    assert compiler._family(facts) == "ruperax" and compiler._sampling_k(facts) == 1
    seen = {}
    monkeypatch.setattr(loader, "parallel_weights", lambda tensors, spec: seen.update(tensors=tensors))
    monkeypatch.setattr(parallel, "ParallelDecoder", lambda spec, w: spec)
    got = compiler._build_parallel(facts)
    want = loader.ruperax_spec(cfg, 50, 3, pad_id=0, eos_id=1)
    for f in ("eps", "embed_scale"):
        assert np.isclose(getattr(got, f), getattr(want, f), rtol=1e-6)
        setattr(got, f, getattr(want, f))
    for a, b in zip(got.layers, want.layers):
        assert np.isclose(a.mixer.scale, b.mixer.scale, rtol=1e-6)
        a.mixer.scale = b.mixer.scale
    assert got == want
    assert all(np.array_equal(seen["tensors"][k], v) for k, v in sd.items())


# ------------------------------------------------------------------------------------------- configuration, tensors, cache
def test_configurations_that_do_not_exist_are_refused():
    from poptransformer_amd.engine.loader import latent_layers
    for bad in ([dict(latent(), type="other")], [dict(latent(), mlp={"kind": "other", "ff": 8})]):
        with pytest.raises(NotImplementedError):
            latent_layers(bad)
    for bad in ([latent(of=0)], [latent(), latent(of=0), latent(of=1)], [latent(), latent(of=2), latent()], [latent(), latent(of=0, kv_rank=64)],
                [latent(), latent(of=0, rot_dim=4)], [latent(), latent(of=0, base=9.0)]):
        with pytest.raises(ValueError):
            latent_layers(bad)
    from poptransformer_amd.engine import registry
    assert registry.architecture({"architecture": "Ruperax"})[1] == ("hybrid",)
    cfg = small_parallel()
    with pytest.raises(ValueError):
        _recorded(cfg, random_parallel(cfg, 0), 1, cfg["max_positions"] + 1, 4)


def test_a_cache_holds_the_widest_window_over_it():
    from poptransformer_amd.engine.loader import ruperax_spec
    from poptransformer_amd.engine.sequences import SequenceStore
    cfg = parallel_config([latent(window=20), latent(window=100), latent(window=150, of=0), latent(window=10, of=1), latent(window=9),
                           latent(window=None, of=4)])
    store = SequenceStore(ruperax_spec(json.loads(json.dumps(cfg)), 600, 1), torch.float32, 2, 600, 50, device="cpu")
    assert [store.cache_window(i) for i in (0, 1, 4)] == [150, 100, None]
    for i, least in ((0, 199), (1, 149), (4, 600)):
        assert least <= store.stores[i][0].shape[1] < least + 64
    assert [len(s) for s in store.stores] == [1, 1, 0, 0, 1, 0]
    store.stores[0][0][1] = 3.0
    store.shifted[5][1] = 4.0
    for _ in range(3):
        store.open()                                            # the third does not fit: what is there moves along
    assert store.capacity == 4 and (store.stores[0][0][1] == 3).all() and (store.shifted[5][1] == 4).all()


def test_rotated_pairs_and_angles():
    from poptransformer_amd.engine.loader import latent_layers
    m = latent_layers([latent(rot_dim=6, base=10.0)])[0].mixer
    x = np.random.default_rng(0).standard_normal((30, 6))
    cs, want = m.angles(30), R.rotate_half(x, 10.0, 6)
    got = x[:, m.pairs()].reshape(30, 3, 2)
    c, s = cs[:, :3, 0], cs[:, :3, 1]
    got = np.stack([got[..., 0] * c - got[..., 1] * s, got[..., 1] * c + got[..., 0] * s], -1).reshape(30, 6)
    assert np.allclose(got, want[:, m.pairs()], atol=1e-6)
    assert (cs[:, 3:] == [1.0, 0.0]).all() and cs.shape == (30, 16, 2)
