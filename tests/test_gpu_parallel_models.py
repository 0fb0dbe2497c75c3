"""Whole decoders with latent attention and parallel sublayers against the plain evaluation of oracle/ruperax.py."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import ruperax as R
from tests.hybrid_models import Reference, feed, greedy, token_ids
from tests.parallel_models import PARALLEL, latent, parallel_config, random_parallel, small_parallel

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]


def _decoder(cfg, sd, dtype, max_len=400, slots=2, pass_rows=None, absorbed_rows=None, batch=1, branch_bytes=None, **kw):
    from poptransformer_amd.engine import loader, parallel
    spec = loader.ruperax_spec(cfg, max_len, batch, dtype=dtype, **kw)

    class Decoder(parallel.ParallelDecoder):
        pass
    if pass_rows:
        Decoder.pass_rows = pass_rows
    if absorbed_rows is not None:
        Decoder.absorbed_rows = absorbed_rows
    if branch_bytes is not None:
        Decoder.branch_bytes = branch_bytes
    return Decoder(spec, loader.parallel_weights(sd, spec), slots=slots)


def _reference(sd, cfg, ids, dtype):
    return Reference(R.forward, sd, cfg, ids, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(PARALLEL))
def test_prompts_portions_and_decoding(name, dtype):
    cfg = PARALLEL[name]
    sd = random_parallel(cfg, 5)
    T = 150
    ids = token_ids(1, T, cfg)
    want = _reference(sd, cfg, ids, dtype)
    dec = _decoder(cfg, sd, dtype)
    for cuts in ((T,), (2, 2, 3, 64, 65), (1, 70, 2, 63), (100,), (17, 16, 18), (1,)):
        print(f"{name} {dtype} cuts {cuts}", flush=True)
        s = dec.open()                       # the slot of the sequence before
        want.check(feed(dec, s, ids, cuts))
        dec.close(s)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_residual_after_every_layer(dtype):
    cfg = small_parallel()
    sd = random_parallel(cfg, 4)
    ids = token_ids(3, 60, cfg)
    layers, got = [], []
    R.forward(sd, cfg, ids, layers)
    dec = _decoder(cfg, sd, dtype)
    dec.probe = lambda i, x: got.append(x.cpu().numpy())
    dec.advance([(dec.open(), ids, [])])
    assert len(got) == len(layers)
    for a, b in zip(got, layers):
        assert np.abs(a - b).max() < (2e-5 if dtype == "float32" else 3e-2) * np.abs(b).max()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_short_sequence_from_its_first_token(dtype):
    cfg = small_parallel()
    sd = random_parallel(cfg, 6)
    dec = _decoder(cfg, sd, dtype, absorbed_rows=1)
    for n in (1, 2, 3):
        ids = token_ids(n, n, cfg)
        for cuts in ((n,), (1,)):
            s = dec.open()
            _reference(sd, cfg, ids, dtype).check(feed(dec, s, ids, cuts))
            dec.close(s)


@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_batches_against_each_alone_and_slots_used_again(dtype):
    """Prompts of very different lengths in one batch, decoded together while the shorter ones end; then other sequences in
    the slots that were given back, and more sequences than there were slots."""
    cfg = small_parallel()
    sd = random_parallel(cfg, 7)
    dec = _decoder(cfg, sd, dtype, slots=1)
    for round_, lens in enumerate(((1, 90, 33, 140), (130, 2, 64), (65, 17, 1, 3, 80, 129))):
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
@pytest.mark.parametrize("absorbed_rows", [0, 16])
def test_mixed_batches_and_passes_smaller_than_a_prompt(dtype, absorbed_rows):
    """Sequences that decode beside sequences that bring portions, and prompts cut into passes by the row limit (the cut falls
    inside sequences, the rings wrap several times)."""
    cfg = small_parallel()
    sd = random_parallel(cfg, 8)
    dec = _decoder(cfg, sd, dtype, slots=3, pass_rows=48, absorbed_rows=absorbed_rows)
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
    """Several windows and ring lengths of decoded tokens (the rings of a decoder whose passes are short wrap often)."""
    cfg = small_parallel()
    sd = random_parallel(cfg, 9)
    dec = _decoder(cfg, sd, dtype, max_len=700, pass_rows=16, branch_bytes=0)
    ids = token_ids(2, 500, cfg)
    _reference(sd, cfg, ids, dtype).check(feed(dec, dec.open(), ids, (16,)))


@pytest.mark.parametrize("dtype", DTYPES)
def test_one_token_is_seen_from_inside_the_window_only(dtype):
    """Two sequences that differ in one token only, in a model whose one layer gives that token's key a large score: logits
    differ as long as the token is in the window (or is the token before the last), and are equal bit for bit afterwards."""
    window = 21
    cfg = parallel_config([latent(window=window, scale=4.0, ff=None)])
    sd = random_parallel(cfg, 10)
    a = token_ids(5, 80, cfg)
    b = list(a)
    b[30] = (b[30] + 1) % cfg["vocab"]
    for cuts in ((80,), (29, 3), (20, 11, 40)):
        dec = _decoder(cfg, sd, dtype)
        x, y = (feed(dec, dec.open(), q, cuts) for q in (a, b))
        differs = np.flatnonzero(np.abs(x - y).max(1) > 0)
        assert differs.min() == 30
        # token 31's latent holds a share of token 30 (the shift), so the last place to see it is one further
        # (in bf16 a difference may round away)
        assert differs.max() == 31 + window - 1 if dtype == "float32" else 31 < differs.max() <= 31 + window - 1


def test_requests_that_do_not_fit_are_refused():
    cfg = small_parallel()
    cfg["max_positions"] = 24
    dec = _decoder(cfg, random_parallel(cfg, 1), "float32", max_len=100)
    s = dec.open()
    for bad in ([(s, [], [])], [(s, list(range(25)), [])], [(s, [cfg["vocab"]], [])], [(s, [1], [1])], [(s, [1], []), (s, [2], [])],
                [(1 - s, [1], [])]):
        with pytest.raises(ValueError):
            dec.advance(bad)
    with pytest.raises(ValueError):
        dec.capture()                            # a loop of 100 positions
    dec.advance([(s, list(range(24)), [23])])
    dec.close(s)
    with pytest.raises(ValueError):
        dec.close(s)


# ------------------------------------------------------------------------------------------- generation
def _session(cfg, sd, precision, B, L, steps, allow_fused=True, **kw):
    from poptransformer_amd.models.ruperax import RuperaxDecModel
    from poptransformer_amd.utils import prepare_model_session
    extra = {k: kw.pop(k) for k in ("topk", "early_stop") if k in kw}
    model = dict(hf_config=cfg, state_dict=sd, pad_token_id=0, eos_token_id=1, max_length=L, max_loop=steps, **extra)
    return prepare_model_session({"global_args": {"batch_size": B, "precision": precision}, "model": model,
                                  "session": dict(kw, allow_fused=allow_fused)}, RuperaxDecModel)


@pytest.mark.parametrize("precision,allow_fused", [("fp32", False), ("fp32", True), ("bf16", True)])
@pytest.mark.parametrize("name", ["small", "odd"])
def test_generation_through_the_session(name, precision, allow_fused):
    cfg = PARALLEL[name]
    sd = random_parallel(cfg, 11)
    B, L, steps = 3, 48, 40
    rng = np.random.default_rng(4)
    ids = np.zeros((B, L), np.int32)
    for b, n in enumerate((9, 4, 20)):                       # unequal prompts
        ids[b, :n] = rng.integers(2, cfg["vocab"], n)
    session, model = _session(cfg, sd, precision, B, L, steps, allow_fused, **({"strict": True} if allow_fused else {}))
    assert session.executor_kind == ("fused:ruperax" if allow_fused else "interpreter"), session.fallback_reason
    want, cols = greedy(R.forward, cfg, sd, ids, steps, 0, 1e-4 if precision == "fp32" else 0.05)
    for _ in range(2):                                       # the second run starts from a used cache
        session.run(model.build_input_dict(input_ids=[list(r[r != 0]) for r in ids]))
        got = session.anchor_arrays["Loop:0"]
        for b in range(B):
            assert np.array_equal(got[b, :cols[b]], want[b, :cols[b]]), f"row {b}"
    lens = (ids != 0).sum(1)
    assert (cols - lens).clip(0).sum() >= (30 if precision == "fp32" else 3)         # generated tokens were compared


def test_generation_ends_early_and_draws_from_the_top_k():
    cfg = small_parallel()
    sd = random_parallel(cfg, 12)
    session, model = _session(cfg, sd, "fp32", 2, 40, 30, topk=4, strict=True)
    session.run(model.build_input_dict(input_ids=[[5, 6, 7], [8, 9, 10, 11]]))
    got = session.anchor_arrays["Loop:0"]
    assert session.executor_kind == "fused:ruperax"
    for b in range(2):
        logits = R.forward(sd, cfg, got[b, :24])
        for t in range(4, 23):
            assert got[b, t + 1] in np.argsort(-logits[t])[:5]
    session, model = _session(cfg, sd, "fp32", 1, 40, 39, early_stop=True, strict=True)
    session.run(model.build_input_dict(input_ids=[[5, 1, 7]]))          # the end token is in the prompt
    assert int(np.asarray(session.anchor_arrays["Loop:1"]).reshape(-1)[0]) < 39


@pytest.mark.parametrize("dtype,branch_bytes", [("float32", 0), ("bfloat16", 0), ("bfloat16", 1 << 60)])
def test_prompt_passes_leave_what_the_loop_leaves(dtype, branch_bytes):
    """The loop with the feed-forwards on a stream of their own, and without."""
    cfg = small_parallel()
    sd = random_parallel(cfg, 13)
    B, L, n = 3, 120, 90
    ids = np.zeros((B, L), np.int32)
    ids[:, :n] = np.random.default_rng(0).integers(2, cfg["vocab"], (B, n))
    want = [_reference(sd, cfg, ids[b, :n], dtype) for b in range(B)]

    def check():
        for b in range(B):
            want[b].check(dec.logits[b:b + 1], [n - 1])
    dec = _decoder(cfg, sd, dtype, max_len=L, batch=B, branch_bytes=branch_bytes)
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
    cfg = small_parallel()
    sd = random_parallel(cfg, 14)
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
