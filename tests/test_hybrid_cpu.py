"""Hybrid decoders without a GPU: the oracle's mechanisms against independent forms, the recorded graph against the oracle,
configuration and checkpoint reading, and the library's exports."""
import ctypes
import json
import os
import re

import numpy as np
import pytest
import torch

from oracle import zekilix as Z
from tests.hybrid_models import attention, bf16, config, dense, mlstm, random_tensors, small_config

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ------------------------------------------------------------------------------------------- oracle pins
def test_norms_and_gates_against_torch():
    rng = np.random.default_rng(0)
    x, w = rng.standard_normal((5, 30)), rng.standard_normal(30)
    t = torch.from_numpy(x)
    want = torch.nn.functional.layer_norm(t, (30,), torch.from_numpy(w), None, 1e-3).numpy()
    assert np.allclose(Z.layer_norm(x, w, 1e-3), want, atol=1e-12)
    assert np.allclose(Z.rms_norm(x, 1e-3), torch.nn.functional.rms_norm(t, (30,), None, 1e-3).numpy(), atol=1e-12)
    assert np.allclose(Z.log_sigmoid(50 * x), torch.nn.functional.logsigmoid(50 * t).numpy(), atol=1e-12)
    assert np.allclose(Z.clamped_glu(np.array([9.0, -9.0]), np.array([9.0, -9.0]), 2.0),
                       [2 * Z.sigmoid(3.404) * 3, -9 * Z.sigmoid(-9 * 1.702) * -1])


@pytest.mark.parametrize("window", [1, 5, None])
def test_windowed_attention_against_a_masked_softmax(window):
    rng = np.random.default_rng(1)
    T, H, G, D = 20, 6, 2, 8
    q, k, v = rng.standard_normal((T, H, D)), rng.standard_normal((T, G, D)), rng.standard_normal((T, G, D))
    slopes = Z.head_slopes(H)
    assert np.allclose(slopes[[2, 5]], [2.0 ** -4, 2.0 ** -8])
    dist = np.arange(T)[:, None] - np.arange(T)[None]
    bias = np.where((dist >= 0) & (dist < (window or T)), -slopes[:, None, None] * dist, -np.inf)
    tq, tk, tv = (torch.from_numpy(np.repeat(a, r, 1)).transpose(0, 1) for a, r in ((q, 1), (k, H // G), (v, H // G)))
    want = torch.nn.functional.scaled_dot_product_attention(tq[None], tk[None], tv[None], attn_mask=torch.from_numpy(bias)[None], scale=0.37)
    assert np.allclose(Z.windowed_attention(q, k, v, 0.37, slopes, window), want[0].transpose(0, 1).numpy(), atol=1e-12)


def test_mlstm_against_its_unrolled_form():
    """o_t = sum_s w_ts (q_t . k_s) v_s / max(|sum_s w_ts q_t . k_s|, 1) with w_ts = exp(i_s + f_{s+1} + .. + f_t), up to the
    1e-6 of the denominator (scaled by the running maximum): the running maximum cancels."""
    rng = np.random.default_rng(2)
    T, H, D, E = 30, 2, 6, 5
    q, k, v = rng.standard_normal((T, H, D)), rng.standard_normal((T, H, D)), rng.standard_normal((T, H, E))
    i, f = rng.standard_normal((T, H)), Z.log_sigmoid(2 + rng.standard_normal((T, H)))
    got = Z.mlstm_recurrence(q, k, v, i, f)
    b = np.cumsum(f, 0)
    for t in range(T):
        for h in range(H):
            w = np.exp(i[:t + 1, h] + b[t, h] - b[:t + 1, h]) * (k[:t + 1, h] @ q[t, h])
            want = w @ v[:t + 1, h] / max(abs(w.sum()), 1.0)
            assert np.allclose(got[t, h], want, rtol=1e-4, atol=1e-5)


def test_connections_are_from_to():
    x = np.array([[[1.0]], [[10.0]]])
    mix = np.array([[0.0, 1.0], [0.0, 0.0]])                    # stream 0 goes to stream 1, stream 1 nowhere
    got = Z.connect(x, np.array([1.0, 2.0]), np.array([3.0, 5.0]), mix, 0.5, lambda u: u)
    assert np.allclose(got[:, 0, 0], [0.5 * 3 * 21, 1 + 0.5 * 5 * 21])


def test_a_layer_that_uses_another_ones_weights_equals_a_copy():
    shared = small_config()
    sd = random_tensors(shared, 3)
    copied = json.loads(json.dumps(shared))
    full = dict(sd)
    for i, lay in enumerate(copied["layers"]):
        j = lay.pop("weights_of", None)
        if j is not None:
            full.update({f"l{i}." + k[len(f"l{j}."):]: v for k, v in sd.items() if k.startswith(f"l{j}.")})
    ids = [3, 1, 4, 1, 5]
    assert np.array_equal(Z.forward(sd, shared, ids), Z.forward(full, copied, ids))


# ------------------------------------------------------------------------------------------- recorded graph
def _recorded(cfg, sd, B, L, steps, precision="fp32"):
    from poptransformer_amd.models.zekilix import ZekilixDecModel
    from poptransformer_amd.utils import REGISTRY, register_global_args
    REGISTRY.reset()
    register_global_args({"batch_size": B, "precision": precision})
    m = ZekilixDecModel(hf_config=cfg, state_dict=sd, pad_token_id=0, eos_token_id=1, max_length=L, max_loop=steps)
    m.build_graph()
    return m


class _HostInterpreter:
    """The op-by-op interpreter on the host, with the two native operators it meets here written out."""

    def __init__(self, graph):
        from poptransformer_amd.engine.interpreter import Interpreter
        it = self.it = Interpreter(graph, device="cpu")

        def cache(n, env, step, upd):
            axis, length = n.attrs["sequence_axis"], n.attrs["max_len"]
            old = it.state.get(n.outputs[0])
            if old is None or int(step) == 0:
                shape = list(upd.shape)
                shape[axis] = length
                old = torch.zeros(shape)
            it.state[n.outputs[0]] = torch.cat([upd, old.narrow(axis, 0, length - 1)], axis)
            return it.state[n.outputs[0]]
        it._custom_KVCache = cache
        it._custom_SoftmaxV3 = lambda n, env, x: torch.softmax(x, -1)


@pytest.mark.parametrize("make", [small_config, lambda: small_config(streams=None), lambda: small_config(streams=1, cap=None)])
def test_the_recorded_graph_is_the_model(make):
    cfg = make()
    B, L, steps = 2, 36, 30
    sd = random_tensors(cfg, 1)
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
        want = Z.forward(sd, cfg, container[b, :steps])
        got = np.stack([x[b] for x in logits])
        assert np.abs(got - want).max() < 2e-5 * max(1.0, np.abs(want).max()) * 10


def test_the_compiler_reads_the_model_off_the_graph(monkeypatch):
    """Specification and tensors that the compiler recovers from the recorded graph equal those of the configuration."""
    from poptransformer_amd.engine import compiler, hybrid, loader
    cfg = small_config()
    sd = random_tensors(cfg, 2)
    m = _recorded(cfg, sd, 3, 50, 10, "bf16")
    facts = compiler.GraphFacts(m.graph)
    assert compiler._family(facts) == "zekilix" and compiler._sampling_k(facts) == 1
    seen = {}
    monkeypatch.setattr(loader, "hybrid_weights", lambda tensors, spec: seen.update(tensors=tensors))
    monkeypatch.setattr(hybrid, "HybridDecoder", lambda spec, w: spec)
    got = compiler._build_hybrid(facts)
    want = loader.zekilix_spec(cfg, 50, 3, pad_id=0, eos_id=1)
    for f in ("eps", "residual_mult", "embed_scale", "logit_cap"):
        assert np.isclose(getattr(got, f), getattr(want, f), rtol=1e-6)
        setattr(got, f, getattr(want, f))
    for a, b in zip(got.layers, want.layers):
        for part in ("mixer", "mlp"):
            x, y = getattr(a, part), getattr(b, part)
            assert type(x) is type(y)
            if y is not None:
                assert all(np.isclose(v, vars(y)[k], rtol=1e-6) if isinstance(v, float) else v == vars(y)[k] for k, v in vars(x).items())
        assert a.source == b.source
    assert (got.width, got.vocab, got.streams, got.dtype, got.batch, got.max_len) == (want.width, want.vocab, want.streams, want.dtype, 3, 50)
    assert all(np.array_equal(seen["tensors"][k], v) for k, v in sd.items())


# ------------------------------------------------------------------------------------------- configuration, checkpoints
def test_configurations_that_do_not_exist_are_refused():
    from poptransformer_amd.engine.loader import hybrid_layers
    lay = attention()
    lay["mixer"]["vdim"] = 8
    with pytest.raises(ValueError):
        hybrid_layers([lay])
    with pytest.raises(NotImplementedError):
        hybrid_layers([dict(attention(), type="other")])
    with pytest.raises(NotImplementedError):
        hybrid_layers([attention(mlp=dict(dense(), kind="other"))])
    chain = hybrid_layers([mlstm(), mlstm(of=0), mlstm(of=1)])
    assert [c.source for c in chain] == [0, 0, 0]


def test_registry_and_bf16_checkpoints(tmp_path):
    from safetensors.torch import save_file
    from poptransformer_amd.engine import registry
    from poptransformer_amd.utils import checkpoint
    w = bf16(np.random.default_rng(0).standard_normal((4, 6)) * 1e-6)        # below what fp16 holds well
    save_file({"w": torch.from_numpy(w).to(torch.bfloat16)}, str(tmp_path / "model.safetensors"))
    got = checkpoint.load_state_dict(str(tmp_path), floats="fp32")["w"]
    assert got.dtype == np.float32 and np.array_equal(got, w)
    assert checkpoint.load_state_dict(str(tmp_path))["w"].dtype == np.float16
    assert registry.architecture({"architecture": "Zekilix"})[1] == ("hybrid",)
    assert registry.architecture({"architectures": ["LlamaForCausalLM"]})[0] == "LlamaForCausalLM"
    with pytest.raises(ValueError):
        registry.architecture({"architecture": "Nothing"})


def test_ring_lengths():
    from poptransformer_amd.engine.loader import zekilix_spec
    from poptransformer_amd.engine.sequences import SequenceStore
    spec = zekilix_spec(config([attention(window=100), attention(window=None)]), 1000, 1)
    store = SequenceStore(spec, torch.float32, 0, 1000, 50, device="cpu")
    for i, least in enumerate((149, 1000)):
        assert least <= store.ring_len(i) < least + 64


def test_every_declared_symbol_is_exported_and_bound():
    from poptransformer_amd import _hybrid_lib, build
    if not os.path.exists(_hybrid_lib.LIB_PATH):
        build.build(force=False, libraries=("hybrid",))
    text = open(os.path.join(ROOT, "include", "poptransformer_hybrid.h")).read()
    text = re.sub(r"/\*.*?\*/", "", text, flags=re.S)
    names = set(re.findall(r"\b(pta_[a-z0-9_]+)\s*\(", text))
    lib = ctypes.CDLL(_hybrid_lib.LIB_PATH)
    assert names == set(_hybrid_lib.SIGNATURES)
    assert all(hasattr(lib, n) for n in names)
    # argument validation happens on the host before any launch
    lib = _hybrid_lib.load()
    assert lib.pta_wide_linear(ctypes.byref(_hybrid_lib.WideLinearArgs()), None) == -1
    assert lib.pta_hybrid_last_error()
    assert lib.pta_mlstm_state_floats(2, 16, 40) == 2 * 2 * (16 * 32 + 20)
