"""Whole decoders with attention by heads and mixtures of experts against the plain evaluation of oracle/golapel.py."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import golapel as G
from tests.head_models import HEADS, chunked, config, dense, differential, moe, random_heads, windowed
from tests.hybrid_models import Reference, feed, greedy, token_ids

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]


def _decoder(cfg, sd, dtype, max_len=400, slots=2, batch=1, **kw):
    from poptransformer_amd.engine import loader, result_norm
    own = {k: kw.pop(k) for k in ("pass_rows", "direct_rows", "router_bytes", "router_rows", "head_rows") if k in kw}
    spec = loader.golapel_spec(cfg, max_len, batch, dtype=dtype, **kw)
    cls = type("Decoder", (result_norm.ResultNormDecoder,), own)
    return cls(spec, loader.result_norm_weights(sd, spec), slots=slots)


def _reference(sd, cfg, ids, dtype):
    return Reference(G.forward, sd, cfg, ids, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(HEADS))
def test_prompts_portions_and_decoding(name, dtype):
    cfg = HEADS[name]
    sd = random_heads(cfg, 5)
    T = 150
    ids = token_ids(1, T, cfg)
    want = _reference(sd, cfg, ids, dtype)
    dec = _decoder(cfg, sd, dtype)
    for cuts in ((T,), (2, 2, 3, 64, 65), (1, 70, 2, 63), (100,), (1,)):
        print(f"{name} {dtype} cuts {cuts}", flush=True)
        s = dec.open()                       # the slot of the sequence before
        want.check(feed(dec, s, ids, cuts))
        dec.close(s)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("router_bytes", [0, 1 << 20])
def test_layers_one_by_one(dtype, router_bytes):
    cfg = HEADS["small"]
    sd = random_heads(cfg, 4)
    ids = token_ids(3, 60, cfg)
    layers = []
    G.forward(sd, cfg, ids, layers)
    for cuts in ((60,), (10, 16, 16), (1,)):
        dec, got = _decoder(cfg, sd, dtype, router_bytes=router_bytes), [[] for _ in layers]
        dec.probe = lambda i, x: got[i].append(x.cpu().numpy())
        feed(dec, dec.open(), ids, cuts)
        for a, b in zip(got, layers):
            assert np.abs(np.concatenate(a) - b).max() < (2e-5 if dtype == "float32" else 4e-2) * np.abs(b).max()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_short_sequence_from_its_first_token(dtype):
    cfg = HEADS["small"]
    sd = random_heads(cfg, 6)
    dec = _decoder(cfg, sd, dtype)
    for n in (1, 2, 3, 4):
        ids = token_ids(n, n, cfg)
        for cuts in ((n,), (1,)):
            s = dec.open()
            _reference(sd, cfg, ids, dtype).check(feed(dec, s, ids, cuts))
            dec.close(s)


@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_batches_against_each_alone_and_slots_used_again(dtype):
    """Prompts of very different lengths in one batch, decoded together while the shorter ones end; then other sequences in the
    slots that were given back, and more sequences than there were slots."""
    cfg = HEADS["small"]
    sd = random_heads(cfg, 7)
    dec = _decoder(cfg, sd, dtype, slots=1)
    for round_, lens in enumerate(((1, 90, 33, 140), (130, 2, 64), (65, 17, 1, 3, 80, 129), [1 + k for k in range(20)])):
        seqs = [token_ids(10 * round_ + i, n + 12, cfg) for i, n in enumerate(lens)]
        want = [_reference(sd, cfg, q, dtype) for q in seqs]
        slots = [dec.open() for _ in seqs]
        got = dec.advance([(s, q[:n], list(range(n))) for s, q, n in zip(slots, seqs, lens)]).cpu().numpy()
        at = 0
        for n, w in zip(lens, want):
            w.check(got[at:at + n], slice(0, n))
            at += n
        live = list(range(len(seqs)))
        for t in range(12):
            got = dec.advance([(slots[i], [seqs[i][lens[i] + t]], [0]) for i in live]).cpu().numpy()
            for r, i in enumerate(live):
                want[i].check(got[r:r + 1], [lens[i] + t])
            if t % 3 == 2 and len(live) > 1:
                dec.close(slots[live.pop(0)])
        for i in live:
            dec.close(slots[i])
    assert dec.store.capacity >= 6


@pytest.mark.parametrize("dtype", DTYPES)
def test_mixed_batches_and_passes_smaller_than_a_prompt(dtype):
    """Sequences that decode beside sequences that bring portions, and prompts cut into passes by the row limit (the cut falls
    inside sequences, the rings wrap several times)."""
    cfg = HEADS["small"]
    sd = random_heads(cfg, 8)
    dec = _decoder(cfg, sd, dtype, slots=3, pass_rows=48, head_rows=4)
    seqs = [token_ids(30 + i, 170, cfg) for i in range(3)]
    want = [_reference(sd, cfg, q, dtype) for q in seqs]
    slots = [dec.open() for _ in seqs]
    at = [0, 0, 0]
    for counts in ((100, 1, 20), (1, 60, 2), (2, 1, 1), (1, 1, 1), (50, 50, 50), (3, 2, 90)):
        entries, rows = [], []
        for i, c in enumerate(counts):
            entries.append((slots[i], seqs[i][at[i]:at[i] + c], [c - 1, 0]))       # wanted places in any order
            rows += [(i, at[i] + c - 1), (i, at[i])]
            at[i] += c
        got = dec.advance(entries).cpu().numpy()
        for r, (i, p) in enumerate(rows):
            want[i].check(got[r:r + 1], [p])


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dtype):
    """Several windows, chunks and ring lengths of decoded tokens (the rings of a decoder whose passes are short wrap often)."""
    cfg = config([windowed(mlp=moe()), differential(chunk=130, mlp=dense()), chunked(chunk=70), windowed(window=90, keep=40)])
    sd = random_heads(cfg, 9)
    dec = _decoder(cfg, sd, dtype, max_len=700, pass_rows=16)
    ids = token_ids(2, 600, cfg)
    _reference(sd, cfg, ids, dtype).check(feed(dec, dec.open(), ids, (16,)))


SIGHT = [
    # (layer, token that differs, last position that sees it)
    (windowed(window=21, keep=0), 30, 50), (windowed(window=21, keep=4), 4, 24), (windowed(window=21, keep=4), 3, 89),
    (windowed(window=1, keep=0), 30, 30), (windowed(window=None), 30, 89), (windowed(window=64, keep=9), 20, 83),
    (chunked(chunk=32), 32, 63), (chunked(chunk=32), 63, 63), (chunked(chunk=31), 40, 61), (chunked(chunk=None), 3, 89),
    (differential(chunk=25), 30, 49), (differential(chunk=25), 49, 49), (differential(chunk=64), 10, 63), (differential(chunk=1), 10, 10),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layer,place,last", SIGHT)
def test_one_token_is_seen_by_those_that_see_it_only(layer, place, last, dtype):
    """Two sequences that differ in one token only, in a model of one layer: logits differ wherever the token is seen, and are
    equal bit for bit everywhere else."""
    cfg = config([layer])
    sd = random_heads(cfg, 10)
    a = token_ids(5, 90, cfg)
    b = list(a)
    b[place] = (b[place] + 1) % cfg["vocab"]
    for cuts in ((90,), (29, 3), (20, 11, 40)):
        dec = _decoder(cfg, sd, dtype)
        x, y = (feed(dec, dec.open(), q, cuts) for q in (a, b))
        differs = np.flatnonzero(np.abs(x - y).max(1) > 0)
        assert differs.min() == place
        # (in bf16 a difference may round away)
        assert np.array_equal(differs, np.arange(place, last + 1)) if dtype == "float32" else differs.max() <= last


def test_requests_that_do_not_fit_are_refused():
    cfg = HEADS["small"]
    dec = _decoder(cfg, random_heads(cfg, 1), "float32", max_len=20)
    s = dec.open()
    for bad in ([(s, [], [])], [(s, list(range(21)), [])], [(s, [cfg["vocab"]], [])], [(s, [1], [1])], [(s, [1], []), (s, [2], [])],
                [(1 - s, [1], [])]):
        with pytest.raises(ValueError):
            dec.advance(bad)
    dec.close(s)
    with pytest.raises(ValueError):
        dec.close(s)


# ------------------------------------------------------------------------------------------- generation
def _session(cfg, sd, precision, B, L, steps, allow_fused=True, **kw):
    from poptransformer_amd.models.golapel import GolapelDecModel
    from poptransformer_amd.utils import prepare_model_session
    extra = {k: kw.pop(k) for k in ("topk", "early_stop") if k in kw}
    model = dict(hf_config=cfg, state_dict=sd, pad_token_id=0, eos_token_id=1, max_length=L, max_loop=steps, **extra)
    return prepare_model_session({"global_args": {"batch_size": B, "precision": precision}, "model": model,
                                  "session": dict(kw, allow_fused=allow_fused)}, GolapelDecModel)


@pytest.mark.parametrize("precision,allow_fused", [("fp32", False), ("fp32", True), ("bf16", True)])
@pytest.mark.parametrize("name", ["small", "odd", "plain"])
def test_generation_through_the_session(name, precision, allow_fused):
    cfg = HEADS[name]
    sd = random_heads(cfg, 11)
    B, L, steps = 3, 48, 40
    rng = np.random.default_rng(4)
    ids = np.zeros((B, L), np.int32)
    for b, n in enumerate((9, 4, 20)):                       # unequal prompts
        ids[b, :n] = rng.integers(2, cfg["vocab"], n)
    session, model = _session(cfg, sd, precision, B, L, steps, allow_fused, **({"strict": True} if allow_fused else {}))
    assert session.executor_kind == ("fused:golapel" if allow_fused else "interpreter"), session.fallback_reason
    want, cols = greedy(G.forward, cfg, sd, ids, steps, 0, 1e-4 if precision == "fp32" else 0.05)
    for _ in range(2):                                       # the second run starts from a used cache
        session.run(model.build_input_dict(input_ids=[list(r[r != 0]) for r in ids]))
        got = session.anchor_arrays["Loop:0"]
        for b in range(B):
            assert np.array_equal(got[b, :cols[b]], want[b, :cols[b]]), f"row {b}"
    lens = (ids != 0).sum(1)
    assert (cols - lens).clip(0).sum() >= (30 if precision == "fp32" else 3)         # generated tokens were compared


def test_generation_ends_early_and_draws_from_the_top_k():
    cfg = HEADS["small"]
    sd = random_heads(cfg, 12)
    session, model = _session(cfg, sd, "fp32", 2, 40, 30, topk=4, strict=True)
    session.run(model.build_input_dict(input_ids=[[5, 6, 7], [8, 9, 10, 11]]))
    got = session.anchor_arrays["Loop:0"]
    assert session.executor_kind == "fused:golapel"
    for b in range(2):
        n = 4 + 20
        logits = G.forward(sd, cfg, got[b, :n])
        for t in range(4, n - 1):
            assert got[b, t + 1] in np.argsort(-logits[t])[:5]
    session, model = _session(cfg, sd, "fp32", 1, 40, 39, early_stop=True, strict=True)
    session.run(model.build_input_dict(input_ids=[[5, 1, 7]]))          # the end token is in the prompt
    assert int(np.asarray(session.anchor_arrays["Loop:1"]).reshape(-1)[0]) < 39


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,batch", [("small", 3), ("plain", 20), ("odd", 1)])
def test_prompt_passes_leave_what_the_loop_leaves(dtype, name, batch):
    cfg = HEADS[name]
    sd = random_heads(cfg, 13)
    L, n = 120, 90
    ids = np.zeros((batch, L), np.int32)
    ids[:, :n] = np.random.default_rng(0).integers(2, cfg["vocab"], (batch, n))
    want = [_reference(sd, cfg, ids[b, :n], dtype) for b in range(batch)]

    def check():
        for b in range(batch):
            want[b].check(dec.logits[b:b + 1], [n - 1])
    dec = _decoder(cfg, sd, dtype, max_len=L, batch=batch)
    dec.capture()
    for passes in (None, 7, 64):
        dec.reset(ids)
        done = dec.consume_prompt(n - 1, rows_per_pass=passes) if passes else 0
        dec.run_steps(n - done)                              # replays, the last one on the prompt's last token
        torch.cuda.synchronize()
        assert int(dec.step.item()) == n
        check()
    for _ in range(3):                                       # replays between eager work give what eager iterations give
        dec.reset(ids)
        dec.run_steps(n)
        torch.cuda.synchronize()
        check()


# ------------------------------------------------------------------------------------------- trace runner
@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_runner(tmp_path, dtype):
    from safetensors.torch import save_file
    cfg = HEADS["small"]
    sd = random_heads(cfg, 14)
    model, out = tmp_path / "model", tmp_path / "out"
    model.mkdir()
    out.mkdir()
    (model / "config.json").write_text(json.dumps(cfg))
    save_file({k: torch.from_numpy(v).to(torch.bfloat16) for k, v in sd.items()}, str(model / "model.safetensors"))
    a, b = token_ids(1, 40, cfg), token_ids(2, 7, cfg)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [29, 0]}, {"id": "b", "tokens": b[:5], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[5:6], "want": [0]}, {"id": "a", "tokens": a[30:31], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[31:32], "want": []}], "end": ["a"]},
             {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [6]}], "end": ["c"]}]
    run = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(model), "--dtype", dtype, "--out",
                          str(out), "--max-tokens", "64"], input="".join(json.dumps(s) + "\n" for s in steps), text=True,
                         capture_output=True, timeout=100)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [x for x in run.stdout.splitlines() if x.startswith("done ")] == ["done 0", "done 1", "done 2", "done 3"]
    wa, wb = _reference(sd, cfg, a, dtype), _reference(sd, cfg, b, dtype)
    want = {0: [(wa, 29), (wa, 0)], 1: [(wb, 5), (wa, 30)], 3: [(wb, 6)]}
    assert sorted(os.listdir(out)) == [f"{k}.f32" for k in want]
    for k, rows in want.items():
        got = np.fromfile(out / f"{k}.f32", "<f4").reshape(len(rows), -1)
        for r, (w, p) in enumerate(rows):
            w.check(got[r:r + 1], [p])
