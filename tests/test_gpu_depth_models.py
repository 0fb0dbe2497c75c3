"""Whole decoders whose results are averaged over the depths against the plain evaluation of oracle/sabolorn.py."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from oracle import sabolorn as S
from tests.depth_models import DEPTH, attention, config, dense, latent, mamba, moe, random_depth
from tests.hybrid_models import Reference, feed, greedy, token_ids

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DTYPES = ["float32", "bfloat16"]


def _decoder(cfg, sd, dtype, max_len=400, slots=2, batch=1, **kw):
    from poptransformer_amd.engine import depth, loader
    own = {k: kw.pop(k) for k in ("pass_rows", "direct_rows", "router_bytes", "router_rows", "head_rows", "absorbed_rows", "scanned_rows") if k in kw}
    spec = loader.sabolorn_spec(cfg, max_len, batch, dtype=dtype, **kw)
    cls = type("Decoder", (depth.DepthDecoder,), own)
    return cls(spec, loader.depth_weights(sd, spec), slots=slots)


def _reference(sd, cfg, ids, dtype):
    return Reference(S.forward, sd, cfg, ids, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(DEPTH))
def test_prompts_portions_and_decoding(name, dtype):
    cfg = DEPTH[name]
    sd = random_depth(cfg, 5)
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
@pytest.mark.parametrize("kw", [dict(router_bytes=0), dict(absorbed_rows=0, scanned_rows=1), dict(absorbed_rows=400, scanned_rows=400, direct_rows=0)])
def test_layers_one_by_one(dtype, kw):
    """The residual after every layer, with each way to the same numbers."""
    cfg = DEPTH["small"]
    sd = random_depth(cfg, 4)
    ids = token_ids(3, 60, cfg)
    layers = []
    S.forward(sd, cfg, ids, layers)
    for cuts in ((60,), (10, 16, 16), (1,)):
        dec, got = _decoder(cfg, sd, dtype, **kw), [[] for _ in layers]
        dec.probe = lambda i, x: got[i].append(x.cpu().numpy())
        feed(dec, dec.open(), ids, cuts)
        for a, b in zip(got, layers):
            assert np.abs(np.concatenate(a) - b).max() < (2e-5 if dtype == "float32" else 5e-2) * np.abs(b).max()


ALONE = {"latent": latent(), "latent, plain rotation": latent(scaling=None, mlp=dense()), "attention": attention(), "attention, one tap": attention(taps=1),
         "mamba": mamba(), "mamba, one group": mamba(groups=1, norm_groups=1, taps=2), "dense": mamba(mlp=dense()), "experts": mamba(mlp=moe()),
         "experts, no groups": mamba(mlp=moe(groups=None))}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ALONE))
def test_each_mechanism_alone(name, dtype):
    cfg = config([ALONE[name]])
    sd = random_depth(cfg, 3)
    ids = token_ids(4, 140, cfg)
    want, dec = _reference(sd, cfg, ids, dtype), _decoder(cfg, sd, dtype)
    for cuts in ((140,), (2, 3, 129), (1,)):
        s = dec.open()
        want.check(feed(dec, s, ids, cuts))
        dec.close(s)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_short_sequence_from_its_first_token(dtype):
    cfg = DEPTH["small"]
    sd = random_depth(cfg, 6)
    dec = _decoder(cfg, sd, dtype)
    for n in (1, 2, 3, 4, 5):
        ids = token_ids(n, n, cfg)
        for cuts in ((n,), (1,)):
            s = dec.open()
            _reference(sd, cfg, ids, dtype).check(feed(dec, s, ids, cuts))
            dec.close(s)


@pytest.mark.parametrize("dtype", DTYPES)
def test_unequal_batches_against_each_alone_and_slots_used_again(dtype):
    """Prompts of very different lengths in one batch, decoded together while the shorter ones end; then other sequences in the
    slots that were given back, and more sequences than there were slots."""
    cfg = DEPTH["small"]
    sd = random_depth(cfg, 7)
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
    inside sequences)."""
    cfg = DEPTH["small"]
    sd = random_depth(cfg, 8)
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
    cfg = config([mamba(mlp=moe()), latent(mlp=dense()), attention(mlp=dense()), latent(of=1)])
    sd = random_depth(cfg, 9)
    dec = _decoder(cfg, sd, dtype, max_len=700, pass_rows=16)
    ids = token_ids(2, 600, cfg)
    _reference(sd, cfg, ids, dtype).check(feed(dec, dec.open(), ids, (16,)))


@pytest.mark.parametrize("layer", [latent(), attention(taps=1), attention(taps=4), mamba(), mamba(taps=3, mlp=moe())])
def test_one_token_is_seen_by_those_after_it_only(layer):
    """Two sequences that differ in one token only, in a model of one layer: logits are equal bit for bit before it and differ from it on,
    whatever the cuts; a sequence that another one stands beside, or that had another one's slot, is the same bit for bit."""
    cfg = config([layer])
    sd = random_depth(cfg, 10)
    a, other = token_ids(5, 90, cfg), token_ids(6, 90, cfg)
    for place in (0, 33):
        b = list(a)
        b[place] = (b[place] + 1) % cfg["vocab"]
        for cuts in ((90,), (29, 3), (20, 11, 40)):
            dec = _decoder(cfg, sd, "float32")
            x, y = (feed(dec, dec.open(), q, cuts) for q in (a, b))
            assert np.array_equal(np.flatnonzero(np.abs(x - y).max(1) > 0), np.arange(place, 90))
    dec = _decoder(cfg, sd, "float32")
    s, t = dec.open(), dec.open()
    feed(dec, s, other, (50,))
    dec.close(s)
    s = dec.open()
    got = np.concatenate([dec.advance([(t, other[p:p + c], []), (s, a[p:p + c], list(range(c)))]).cpu().numpy() for p, c in ((0, 40), (40, 2), (42, 48))])
    dec = _decoder(cfg, sd, "float32")
    assert np.array_equal(got, feed(dec, dec.open(), a, (40, 2, 48)))


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_slot_that_is_used_again_remembers_nothing(dtype):
    """A sequence in a slot whose cache, state and convolution rows hold large numbers of an earlier one."""
    cfg = DEPTH["small"]
    sd = random_depth(cfg, 8)
    ids = token_ids(3, 40, cfg)
    want, dec = _reference(sd, cfg, ids, dtype), _decoder(cfg, sd, dtype, slots=1)
    for cuts in ((40,), (1,), (2, 7)):
        for t in [t for store in dec.store.stores for t in store] + [t for t in dec.store.recent if t is not None]:
            t.fill_(1e4)
        s = dec.open()
        want.check(feed(dec, s, ids, cuts))
        dec.close(s)


def test_requests_that_do_not_fit_are_refused():
    cfg = DEPTH["small"]
    dec = _decoder(cfg, random_depth(cfg, 1), "float32", max_len=20)
    s = dec.open()
    for bad in ([(s, [], [])], [(s, list(range(21)), [])], [(s, [cfg["vocab"]], [])], [(s, [1], [1])], [(s, [1], []), (s, [2], [])],
                [(1 - s, [1], [])]):
        with pytest.raises(ValueError):
            dec.advance(bad)


# ------------------------------------------------------------------------------------------- generation
def _session(cfg, sd, precision, B, L, steps, allow_fused=True, **kw):
    from poptransformer_amd.models.sabolorn import SabolornDecModel
    from poptransformer_amd.utils import prepare_model_session
    extra = {k: kw.pop(k) for k in ("topk", "early_stop") if k in kw}
    model = dict(hf_config=cfg, state_dict=sd, pad_token_id=0, eos_token_id=1, max_length=L, max_loop=steps, **extra)
    return prepare_model_session({"global_args": {"batch_size": B, "precision": precision}, "model": model,
                                  "session": dict(kw, allow_fused=allow_fused)}, SabolornDecModel)


@pytest.mark.parametrize("precision,allow_fused", [("fp32", False), ("fp32", True), ("bf16", True)])
@pytest.mark.parametrize("name", ["small", "odd"])
def test_generation_through_the_session(name, precision, allow_fused):
    cfg = DEPTH[name]
    sd = random_depth(cfg, 5)
    B, L, steps = 3, 48, 40
    rng = np.random.default_rng(4)
    ids = np.zeros((B, L), np.int32)
    for b, n in enumerate((9, 4, 20)):                       # unequal prompts
        ids[b, :n] = rng.integers(2, cfg["vocab"], n)
    session, model = _session(cfg, sd, precision, B, L, steps, allow_fused, **({"strict": True} if allow_fused else {}))
    assert session.executor_kind == ("fused:sabolorn" if allow_fused else "interpreter"), session.fallback_reason
    want, cols = greedy(S.forward, cfg, sd, ids, steps, 0, 1e-4 if precision == "fp32" else 0.05)
    for _ in range(2):                                       # the second run starts from a used cache
        session.run(model.build_input_dict(input_ids=[list(r[r != 0]) for r in ids]))
        got = session.anchor_arrays["Loop:0"]
        for b in range(B):
            assert np.array_equal(got[b, :cols[b]], want[b, :cols[b]]), f"row {b}"
    lens = (ids != 0).sum(1)
    assert (cols - lens).clip(0).sum() >= (30 if precision == "fp32" else 3)         # generated tokens were compared


def test_generation_ends_early_and_draws_from_the_top_k():
    cfg = DEPTH["small"]
    sd = random_depth(cfg, 12)
    session, model = _session(cfg, sd, "fp32", 2, 40, 30, topk=4, strict=True)
    session.run(model.build_input_dict(input_ids=[[5, 6, 7], [8, 9, 10, 11]]))
    got = session.anchor_arrays["Loop:0"]
    assert session.executor_kind == "fused:sabolorn"
    for b in range(2):
        n = 4 + 20
        logits = S.forward(sd, cfg, got[b, :n])
        for t in range(4, n - 1):
            assert got[b, t + 1] in np.argsort(-logits[t])[:5]
    session, model = _session(cfg, sd, "fp32", 1, 40, 39, early_stop=True, strict=True)
    session.run(model.build_input_dict(input_ids=[[5, 1, 7]]))          # the end token is in the prompt
    assert int(np.asarray(session.anchor_arrays["Loop:1"]).reshape(-1)[0]) < 39


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,batch", [("small", 3), ("alike", 20), ("odd", 1)])
def test_prompt_passes_leave_what_the_loop_leaves(dtype, name, batch):
    cfg = DEPTH[name]
    sd = random_depth(cfg, 9)
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
    cfg = DEPTH["small"]
    sd = random_depth(cfg, 10)
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
