"""Decoders with attention by heads and mixtures of experts without a GPU: the oracle's mechanisms against independent forms, the
recorded graph against the oracle, configuration reading, and the cache."""
import json

import numpy as np
import pytest
import torch

from oracle import golapel as G
from tests.head_models import HEADS, chunked, config, dense, differential, moe, random_heads, windowed
from tests.test_hybrid_cpu import _HostInterpreter


# ------------------------------------------------------------------------------------------- oracle pins
def test_masks_and_attention_against_a_masked_softmax():
    rng = np.random.default_rng(1)
    T, H, Gk, D, E = 20, 6, 2, 8, 5
    q, k, v = rng.standard_normal((T, H, D)), rng.standard_normal((T, Gk, D)), rng.standard_normal((T, Gk, E))
    near = G.window_mask(T, 5, 3)
    assert [list(np.flatnonzero(near[i])) for i in (0, 4, 9)] == [[0], [0, 1, 2, 3, 4], [0, 1, 2, 5, 6, 7, 8, 9]]
    part = G.chunk_mask(T, 6)
    assert [list(np.flatnonzero(part[i])) for i in (5, 6, 13)] == [[0, 1, 2, 3, 4, 5], [6], [12, 13]]
    assert np.array_equal(G.window_mask(T), G.chunk_mask(T)) and np.array_equal(G.window_mask(T), np.tril(np.ones((T, T), bool)))
    tq, tk, tv = (torch.from_numpy(np.repeat(a, r, 1)).transpose(0, 1)[None] for a, r in ((q, 1), (k, 3), (v, 3)))
    for mask in (near, part):
        want = torch.nn.functional.scaled_dot_product_attention(tq, tk, tv, attn_mask=torch.from_numpy(mask), scale=0.37)
        assert np.allclose(G.attend(q, k, v, 0.37, mask), want[0].transpose(0, 1).numpy(), atol=1e-12)
    # a sink is one more key of that score, without a value
    sink = rng.standard_normal(H)
    k1 = np.concatenate([k, np.zeros((1, Gk, D))])
    out = G.attend(q, k, v, 0.37, near, sink)
    s = np.where(near[None], np.einsum("ihd,jhd->hij", q, np.repeat(k, 3, 1)) * 0.37, -np.inf)
    p = torch.softmax(torch.from_numpy(np.concatenate([s, np.broadcast_to(sink[:, None, None], (H, T, 1))], 2)), -1).numpy()[..., :-1]
    assert k1.shape[0] == T + 1 and np.allclose(out, np.einsum("hij,jhe->ihe", p, np.repeat(v, 3, 1)), atol=1e-12)


def test_rotations():
    rng = np.random.default_rng(2)
    x = rng.standard_normal((40, 3, 10))
    f = G.plain_frequencies(7.0, 6)
    assert np.allclose(f, [1.0, 7.0 ** (-1 / 3), 7.0 ** (-2 / 3)])
    turns = np.exp(1j * np.arange(40)[:, None] * f)[:, None]
    halves, neighbours = G.rotate(x, f), G.rotate(x, f, 1.5, True)
    z = (x[..., :3] + 1j * x[..., 3:6]) * turns
    assert np.allclose(halves[..., :3], z.real) and np.allclose(halves[..., 3:6], z.imag) and np.array_equal(halves[..., 6:], x[..., 6:])
    z = (x[..., 0:6:2] + 1j * x[..., 1:6:2]) * turns * 1.5
    assert np.allclose(neighbours[..., 0:6:2], z.real) and np.allclose(neighbours[..., 1:6:2], z.imag)
    assert np.array_equal(neighbours[..., 6:], x[..., 6:])
    # stretched: fast features stay, slow ones are divided, and nothing lies outside the two
    f, amplitude = G.yarn_frequencies(10000.0, 64, 8.0, 512, 32.0, 1.0)
    plain = G.plain_frequencies(10000.0, 64)
    assert np.isclose(amplitude, 0.1 * np.log(8.0) + 1) and np.allclose(f[0], plain[0]) and np.allclose(f[-1], plain[-1] / 8)
    turns_within = 512 * plain / (2 * np.pi)
    assert np.allclose(f[turns_within > 40], plain[turns_within > 40]) and np.allclose(f[turns_within < 0.7], plain[turns_within < 0.7] / 8)
    assert (np.diff(plain / f) > -1e-12).all()


def test_router_and_experts():
    rng = np.random.default_rng(3)
    z = rng.standard_normal((30, 7))
    chosen, weight = G.route(z, 3, 1.7)
    p = torch.softmax(torch.from_numpy(z), -1)
    v, i = torch.topk(p, 3)
    assert np.array_equal(chosen, i.numpy()) and np.allclose(weight, 1.7 * v.numpy())
    assert (weight.sum(1) < 1.7).all()                          # what is not chosen keeps its share
    cfg = config([windowed(mlp=moe())])
    sd = random_heads(cfg, 1)
    h = rng.standard_normal((5, cfg["width"])) * 4
    f = cfg["layers"][0]["mlp"]
    y = G.experts(sd, "l0.mlp.", f, h)
    chosen, weight = G.route(h @ sd["l0.mlp.router"].T, 2, 1.7)
    t = torch.from_numpy(h).double()
    for r in range(5):
        want = torch.zeros(cfg["width"], dtype=torch.float64)
        for e, w in list(zip(chosen[r], weight[r])) + [(None, None)]:
            p, limit = (f"l0.mlp.e{e}.", 1.2) if e is not None else ("l0.mlp.shared.", 0.9)
            a, b, c = (torch.from_numpy(sd[p + n]).double() for n in ("gate", "up", "down"))
            g, u = (a @ t[r]).clamp(max=limit), (b @ t[r]).clamp(-limit, limit)
            if e is None:
                w = torch.sigmoid(torch.from_numpy(sd["l0.mlp.shared.sg"]).double() @ t[r])
            want += w * (c @ (g * torch.sigmoid(1.702 * g) * (u + 1)))
        assert np.allclose(y[r], want.numpy(), atol=1e-9)


def test_two_equal_maps_leave_a_fixed_direction():
    """With both maps alike the result is (1 - lambda) a, so its normed form is that of a up to the sign."""
    rng = np.random.default_rng(4)
    a = rng.standard_normal((3, 2, 6))
    got = G.differential_combine(a, a, 0.4, 0.25, 0.0)
    assert np.allclose(got, 0.75 * a / np.sqrt((a ** 2).mean(-1, keepdims=True)))
    assert np.allclose(G.differential_combine(a, a, 1.4, 0.25, 0.0), -got)
    sd = {n: np.array(v) for n, v in (("lq1", [1.0, 2.0]), ("lk1", [0.5, -0.25]), ("lq2", [1.0, 0.0]), ("lk2", [-1.0, 3.0]))}
    assert np.isclose(G.differential_lambda(sd, "", 0.3), 1.0 - np.exp(-1.0) + 0.3)


# ------------------------------------------------------------------------------------------- recorded graph
def _recorded(cfg, sd, B, L, steps, precision="fp32"):
    from poptransformer_amd.models.golapel import GolapelDecModel
    from poptransformer_amd.utils import REGISTRY, register_global_args
    REGISTRY.reset()
    register_global_args({"batch_size": B, "precision": precision})
    m = GolapelDecModel(hf_config=cfg, state_dict=sd, pad_token_id=0, eos_token_id=1, max_length=L, max_loop=steps)
    m.build_graph()
    return m


@pytest.mark.parametrize("name", ["small", "odd", "alike", "plain"])
def test_the_recorded_graph_is_the_model(name):
    cfg = HEADS[name]
    B, L, steps = 2, 40, 34
    sd = random_heads(cfg, 1)
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
    assert name not in ("small", "plain") or len(set(container[0, 8:steps])) > 3         # (generation does not stand still)
    for b in range(B):
        want = G.forward(sd, cfg, container[b, :steps])
        got = np.stack([x[b] for x in logits])
        assert np.abs(got - want).max() < 2e-4 * max(1.0, np.abs(want).max())


@pytest.mark.parametrize("name", list(HEADS))
def test_the_compiler_reads_the_model_off_the_graph(monkeypatch, name):
    """Specification and tensors that the compiler recovers from the recorded graph equal those of the configuration."""
    from poptransformer_amd.engine import compiler, loader, result_norm
    cfg = json.loads(json.dumps(HEADS[name]))
    cfg["layers"][1]["mixer"].setdefault("rot", {"base": 1.0, "dims": 2})["base"] = 1234567.891       # not an fp32 number
    sd = random_heads(cfg, 2)
    facts = compiler.GraphFacts(_recorded(cfg, sd, 3, 50, 10, "bf16").graph)
    assert compiler._family(facts) == "golapel" and compiler._sampling_k(facts) == 1
    seen = {}
    monkeypatch.setattr(loader, "result_norm_weights", lambda tensors, spec: seen.update(tensors=tensors))
    monkeypatch.setattr(result_norm, "ResultNormDecoder", lambda spec, w: spec)
    got = compiler._build_result_norm(facts)
    want = loader.golapel_spec(cfg, 50, 3, pad_id=0, eos_id=1)
    assert got == want
    assert all(np.array_equal(seen["tensors"][k], v) for k, v in sd.items())


# ------------------------------------------------------------------------------------------- configuration, cache, angles
def test_configurations_that_do_not_exist_are_refused():
    from poptransformer_amd.engine import registry
    from poptransformer_amd.engine.loader import head_layers
    for bad in (dict(windowed(), type="other"), windowed(mlp=dict(dense(), kind="other"))):
        with pytest.raises(NotImplementedError):
            head_layers([bad])
    unequal = windowed()
    unequal["mixer"]["vdim"] = 8
    for bad in (unequal, windowed(turned=18), windowed(turned=3), windowed(heads=5, kv_heads=2)):
        with pytest.raises(ValueError):
            head_layers([bad])
    assert registry.architecture({"architecture": "Golapel"})[1] == ("hybrid",)


def test_cache_rows_and_growth():
    from poptransformer_amd.engine.loader import golapel_spec
    from poptransformer_amd.engine.sequences import SequenceStore
    cfg = config([windowed(window=100, keep=5), differential(chunk=70, dim=10, vdim=12), chunked(chunk=None), windowed(window=4, keep=700)])
    store = SequenceStore(golapel_spec(cfg, 600, 1), torch.float32, 2, 600, 50, device="cpu")
    for i, least in enumerate((5 + 99 + 50, 69 + 50, 600, 701)):
        assert least <= store.stores[i][0].shape[-2] == store.stores[i][1].shape[-2] < least + 64
    assert store.stores[1][0].shape[:3] == (2, 2, 2) and store.stores[1][0].shape[-1] == 16
    store.stores[1][0][1] = 3.0
    for _ in range(3):
        store.open()                                            # the third does not fit: what is there moves along
    assert store.capacity == 4 and (store.stores[1][0][1] == 3).all()


@pytest.mark.parametrize("layer", [windowed(turned=6, base=10.0), windowed(turned=16, factor=None), chunked(turned=10),
                                   chunked(turned=24, base=300.0, scaling=(5.0, 200, 8.0, 0.5)), chunked(scaling=(2.0, 64, 3.0, 3.0))])
def test_rotated_pairs_and_angles(layer):
    from poptransformer_amd.engine.loader import head_layers
    m = head_layers([layer])[0].mixer
    r, s = layer["mixer"]["rot"], layer["mixer"]["rot"].get("scaling")
    if layer["type"] == "attention":
        f, amplitude = (G.linear_frequencies(r["base"], r["dims"], s["factor"]) if s else G.plain_frequencies(r["base"], r["dims"])), 1.0
    else:
        f, amplitude = G.yarn_frequencies(r["base"], r["dims"], **s)
    x = np.random.default_rng(0).standard_normal((50, m.dim))
    pairs, cs, n = m.rot.pairs(m.dim), m.rot.angles(50), r["dims"] // 2
    want = G.rotate(x, f, amplitude, m.rot.neighbours)[:, pairs]
    got = x[:, pairs]
    u, v, c, sn = got[:, 0:2 * n:2].copy(), got[:, 1:2 * n:2].copy(), cs[:, :n, 0], cs[:, :n, 1]
    got[:, 0:2 * n:2], got[:, 1:2 * n:2] = u * c - v * sn, v * c + u * sn
    assert np.allclose(got, want, atol=1e-5)
    assert cs.shape == (50, (r["dims"] + 7) // 8 * 4, 2) and (cs[:, n:] == [1.0, 0.0]).all()


def test_visible_positions():
    from poptransformer_amd.engine.loader import head_layers
    for layer, mask in ((windowed(window=5, keep=3), G.window_mask(30, 5, 3)), (windowed(window=None), G.window_mask(30)),
                        (chunked(chunk=7), G.chunk_mask(30, 7)), (differential(chunk=1), G.chunk_mask(30, 1))):
        table = head_layers([layer])[0].mixer.visible(30)
        for i in range(30):
            assert np.array_equal(table[i, :i + 1][::-1], mask[i, :i + 1]) and not table[i, i + 1:].any()
