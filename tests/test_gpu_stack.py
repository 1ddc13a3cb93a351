"""Layer-stack engine against the whole-sequence oracle (oracle/stack_oracle.py): prompts, decoding,
portions, batches, slots used again, generation, in fp32 (1e-5-level) and bf16.

The fp32 bar is TOL on every row: rms over the vocabulary of the difference to the fp64 oracle,
relative to the logits' rms.  A wrong key, position, pass or expert moves rows by 1e-2 and more."""
from __future__ import annotations

import json
import os
import subprocess
import sys

import numpy as np
import pytest

import stack_oracle as S
from conftest import ROOT
from stack_models import CONFIGS, LOOP_ALL, MIXED, PLAIN, engine, f64, random_weights, row_error, tokens, write_model

pytestmark = pytest.mark.gpu
TOL = 3e-5
_cache = {}


def model(name, seed=3):
    if (name, seed) not in _cache:
        cfg = CONFIGS[name]
        _cache[name, seed] = (cfg, random_weights(cfg, seed))
    return _cache[name, seed]


def reference(name, toks, seed=3):
    key = (name, seed, tuple(toks))
    if key not in _cache:
        cfg, w = model(name, seed)
        _cache[key] = S.forward(toks, f64(w), cfg)
    return _cache[key]


def close(got, ref, what=""):
    e = row_error(got, ref)
    assert np.isfinite(np.asarray(got)).all() and e.max() < TOL, f"{what}: row {int(e.argmax())} differs by {e.max():.2e}"


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_logits_and_layer_residuals(ti, name):
    cfg, w = model(name)
    t = tokens(cfg, 150, 5)
    lay = []
    ref = S.forward(t, f64(w), cfg, lay)
    e = engine(ti, cfg, w)
    got, gl = e.prefill(1, t, 0, range(len(t)), want_layers=True)
    e.close()
    assert gl.shape[0] == len(lay) == len(S.schedule(cfg))
    for i, (a, b) in enumerate(zip(gl, lay)):
        assert np.abs(a - b).max() < 2e-4 * np.abs(b).max(), f"run {i}"
    close(got, ref, name)


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("n", [1, 2, 15, 16, 17, 63, 64, 65, 128, 129])
def test_prompt_lengths(ti, name, n):
    cfg, w = model(name)
    t = tokens(cfg, n, 100 + n)
    e = engine(ti, cfg, w, max_seq=136)
    close(e.prefill(0, t, 0, range(n)), reference(name, t), f"{n} tokens")
    e.close()


@pytest.mark.parametrize("name", ["mixed", "loop_all"])
def test_token_by_token_equals_prompt(ti, name):
    cfg, w = model(name)
    t = tokens(cfg, 140, 7)
    e = engine(ti, cfg, w, max_seq=140)
    got = np.concatenate([e.step([t[i]], [i]) for i in range(len(t))])
    e.close()
    close(got, reference(name, t), "decoded")


@pytest.mark.parametrize("rows", [2, 3, 16, 17, 50, 64])
def test_prompt_portions(ti, rows):
    cfg, w = model("mixed")
    t = tokens(cfg, 150, 5)
    e = engine(ti, cfg, w)
    e.set_prefill(rows)
    got = e.prefill(2, t, 0, range(len(t)))
    # and the caller's own portions, the second starting inside a block
    cut = 3 * rows + 1 if 3 * rows + 1 < len(t) - 1 else rows
    a = e.prefill(0, t[:cut], 0, range(cut))
    b = e.prefill(0, t[cut:], cut, range(len(t) - cut))
    e.close()
    close(got, reference("mixed", t), f"chunks of {rows}")
    close(np.concatenate([a, b]), reference("mixed", t), f"cut at {cut}")


@pytest.mark.parametrize("name", ["mixed", "plain"])
def test_unequal_requests_in_one_batch(ti, name):
    cfg, w = model(name)
    lens, steps = [1, 70, 129, 16], 30
    seqs = [tokens(cfg, n + steps, 40 + n) for n in lens]
    refs = [reference(name, s) for s in seqs]
    e = engine(ti, cfg, w)
    for i, (s, n) in enumerate(zip(seqs, lens)):
        close(e.prefill(i, s[:n]), refs[i][n - 1 : n], f"request {i} prompt")
    for k in range(steps):
        live = 4 if k < 10 else 3 if k < 20 else 2          # later requests end earlier
        got = e.step([s[n + k] for s, n in zip(seqs, lens)][:live], [n + k for n in lens][:live])
        for i in range(live):
            close(got[i : i + 1], refs[i][lens[i] + k][None], f"request {i} step {k}")
    e.close()


@pytest.mark.parametrize("streams", [17, 33, 64, 70])
def test_many_streams(ti, streams):
    """More streams than one, two and four 16-row tiles hold, and past the skinny products."""
    cfg, w = model("loop_all")
    seqs = [tokens(cfg, 5 + (i % 7) + 4, 500 + i) for i in range(streams)]
    e = engine(ti, cfg, w, max_seq=64, max_batch=streams)
    for i, s in enumerate(seqs):
        e.prefill(i, s[:-4])
    for k in range(4):
        got = e.step([s[len(s) - 4 + k] for s in seqs], [len(s) - 4 + k for s in seqs])
        for i, s in enumerate(seqs):
            close(got[i : i + 1], reference("loop_all", s)[len(s) - 4 + k][None], f"stream {i}")
    e.close()


def test_steps_over_chosen_slots(ti):
    """Rows in any order of slots, some slots left out: their caches stay as they are."""
    cfg, w = model("mixed")
    lens = [20, 65, 7]
    seqs = [tokens(cfg, n + 8, 70 + n) for n in lens]
    refs = [reference("mixed", s) for s in seqs]
    e = engine(ti, cfg, w)
    for i, (s, n) in enumerate(zip(seqs, lens)):
        e.prefill(i + 1, s[:n])
    at = list(lens)
    for live in ([2, 0], [1], [0, 1, 2], [2, 1], [0]):
        got = e.step_slots([i + 1 for i in live], [seqs[i][at[i]] for i in live], [at[i] for i in live])
        for r, i in enumerate(live):
            close(got[r : r + 1], refs[i][at[i]][None], f"slot {i + 1} position {at[i]}")
            at[i] += 1
    e.close()


def test_slots_are_used_again(ti):
    cfg, w = model("mixed")
    e = engine(ti, cfg, w)
    long_, short = tokens(cfg, 200, 1), tokens(cfg, 21, 2)
    e.prefill(0, long_)
    e.prefill(1, long_[:90])
    for slot in (0, 1):
        close(e.prefill(slot, short[:9]), reference("mixed", short)[8:9], f"slot {slot}")
    for i in range(9, len(short)):
        got = e.step([short[i]] * 2, [i] * 2)
        close(got, np.repeat(reference("mixed", short)[i : i + 1], 2, 0), f"position {i}")
    e.close()


def test_long_decoding(ti):
    cfg, w = model("loop_all")
    t = tokens(cfg, 600, 9)
    e = engine(ti, cfg, w, max_seq=600, max_batch=2)
    ref = reference("loop_all", t)
    e.prefill(1, t[:5])
    got = []
    for i in range(5, len(t)):
        got.append(e.step([0, t[i]], [0, i])[1])
    e.close()
    close(np.array(got), ref[5:], "long decode")


def test_long_prompt_over_chunks(ti):
    cfg, w = model("plain")
    t = tokens(cfg, 2600, 4)      # more than one prefill chunk
    want = [0, 1, 63, 64, 2046, 2047, 2048, 2049, 2111, 2112, 2599]
    e = engine(ti, cfg, w, max_seq=2650, max_batch=1)
    got = e.prefill(0, t, 0, want)
    step = e.step([7], [2600])
    e.close()
    ref = reference("plain", t + [7])
    close(got, ref[want], "prompt")
    close(step, ref[2600:], "next token")


def test_long_prompt_of_many_heads(ti):
    """Enough row blocks for the 32-row attention tiles, value sizes of 4, 8 and 16 tiles (the last in
    16-row tiles), in one portion and in two that start inside a key block."""
    from stack_models import config, mixer
    cfg = config(60, 40, [(mixer(17, 20, 12, 20, 24, 28), None), (mixer(18, 36, 6, 68, 20, 40), None),
                          (mixer(17, 12, 8, 132, 16, 24), None)])
    w = random_weights(cfg, 11)
    t = tokens(cfg, 1030, 12)
    ref = S.forward(t, f64(w), cfg)
    e = engine(ti, cfg, w, max_seq=1030, max_batch=2)
    close(e.prefill(0, t, 0, range(len(t))), ref, "whole")
    e.prefill(1, t[:21])
    close(e.prefill(1, t[21:], 21, range(len(t) - 21)), ref[21:], "second portion")
    e.close()


def needle_model():
    """One layer, one head of width 8, whose attention weight is decided by the token's embedding: token
    1 is the query, token 2 the key it looks for (score far above the others), token 0 the rest."""
    from stack_models import config, mixer, moe, shapes
    cfg = config(16, 32, [(mixer(1, 8, 4, 8, 8, 8, scale=1.0), None)])
    w = {n: np.zeros(s, np.float32) for n, s in shapes(cfg).items()}
    rng = np.random.default_rng(0)
    w["embed"][:] = rng.normal(0, 0.05, w["embed"].shape)
    w["embed"][1, 0], w["embed"][2, 1], w["embed"][0, 2] = 3, 3, 3
    for n in w:
        if w[n].ndim == 1 and not n.endswith((".b", "sink")):
            w[n][:] = 1
    w["l0.mix.dq"][0, 0] = w["l0.mix.dkv"][0, 1] = w["l0.mix.dkv"][1, 2] = 1
    w["l0.mix.dkv"][8:] = rng.normal(0, 0.02, (4, 32))
    w["l0.mix.uq"][:] = rng.normal(0, 0.02, w["l0.mix.uq"].shape)
    w["l0.mix.uq"][0, 0] = 3.0
    w["l0.mix.uk"][0, 0] = 2.0
    w["l0.mix.uv"][:] = rng.normal(0, 1, w["l0.mix.uv"].shape)
    w["l0.mix.sink"][:] = 4.0
    w["l0.mix.o"][:] = rng.normal(0, 1, w["l0.mix.o"].shape)
    w["head"][:] = rng.normal(0, 1, w["head"].shape)
    return cfg, w


@pytest.mark.parametrize("n", [64, 65, 128, 129, 300])
def test_single_far_key(ti, n):
    """The one key a query looks for, at block borders, first and last, in prompts and decoding."""
    cfg, w = needle_model()
    wd = f64(w)
    e = engine(ti, cfg, w, max_seq=384, max_batch=2)
    base = S.forward([0] * n + [1], wd, cfg)[-1]
    for at in sorted({0, 1, 15, 16, 31, 32, 62, 63, n - 65, n - 64, n - 33, n - 17, n - 2, n - 1} & set(range(n))):
        t = [0] * n + [1]
        t[at] = 2
        ref = S.forward(t, wd, cfg)[-1:]
        assert row_error(base[None], ref)[0] > 1e-2, "the key must show"
        close(e.prefill(0, t), ref, f"prompt, key at {at} of {n}")
        e.prefill(1, t[:-1])
        close(e.step([0, 1], [0, n])[1:], ref, f"decoded, key at {at} of {n}")
    e.close()


def test_first_token_sees_itself_and_the_sink(ti):
    cfg, w = needle_model()
    e = engine(ti, cfg, w, max_seq=16)
    for sink in (-60.0, 0.0, 8.0, 80.0):
        w["l0.mix.sink"][:] = sink
        e.set_weight("l0.mix.sink", w["l0.mix.sink"])
        ref = S.forward([2, 1], f64(w), cfg)
        close(e.prefill(0, [2, 1], 0, [0, 1]), ref, f"sink {sink}")
        close(e.step([2], [0]), ref[:1], f"sink {sink}, decoded")
    e.close()


@pytest.mark.parametrize("name", ["all_experts", "mixed", "loop_all"])
def test_bf16_rows(ti, name):
    """bf16: every row where each token uses every expert; elsewhere a close call of a router may pick
    another one, so the bar is on most rows."""
    cfg, w = model(name)
    t = tokens(cfg, 180, 5)
    ref = reference(name, t)
    e = engine(ti, cfg, w, "bfloat16")
    runs = {"whole": e.prefill(0, t, 0, range(len(t)))}
    e.set_prefill(33)
    runs["portions"] = e.prefill(1, t, 0, range(len(t)))
    runs["decoded"] = np.concatenate([e.step([t[i]], [i]) for i in range(100)])
    e.close()
    for what, got in runs.items():
        q = np.quantile(row_error(got, ref[: len(got)]), [0.5, 0.75, 1.0])
        assert np.isfinite(got).all() and q[0] < 0.04 and q[1] < 0.1, (what, q)
        assert name != "all_experts" or q[2] < 0.08, (what, q)


def greedy_reference(name, prompt, n):
    cfg, w = model(name)
    out, lg = S.greedy(prompt, n, f64(w), cfg)
    # every step decided by more than the engine's error
    for l in lg:
        s = np.sort(l)
        decided = bool(s[-1] - s[-2] > 1e-3 * np.abs(l).max())
        assert decided, "pick another prompt seed"
    return out


def test_generation_entry_points(ti):
    """Greedy generate, batched generate, continuous batching through few slots, the device sampler with
    top_k = 1 and a beam of one all give the oracle's greedy continuation."""
    cfg, w = model("mixed")
    prompts, n = [tokens(cfg, k, s) for k, s in ((3, 62), (40, 62), (1, 61), (17, 60), (70, 60))], 12
    refs = [greedy_reference("mixed", p, n) for p in prompts]
    e = engine(ti, cfg, w, max_seq=128, max_batch=3)
    for p, r in zip(prompts, refs):
        assert e.generate([p], n)[0].tolist() == r
    for a in (0, 2):
        assert e.generate(prompts[a : a + 3], n).tolist() == refs[a : a + 3]
    assert e.serve(prompts, n, eos=-1, chunk=5) == refs
    assert e.serve(prompts, n, eos=refs[1][3], chunk=4)[1] == refs[1][: refs[1].index(refs[1][3]) + 1]
    toks, _ = e.generate_sampled([prompts[1]], n, 1.0, 1, 1.0, np.full((1, n), 0.5))
    assert toks[0].tolist() == refs[1]
    beams = e.beam_search(prompts[3], n, 1, eos=-1)
    assert beams[0][0] == refs[3]
    assert len(e.beam_search(prompts[3], 6, 3, eos=-1)) == 3
    e.close()


def test_beam_search_scores(ti):
    """Forked caches: every beam's log-probability is that of its tokens under the oracle."""
    cfg, w = model("plain")
    p = tokens(cfg, 20, 8)
    e = engine(ti, cfg, w, max_seq=64, max_batch=4)
    for toks, lp, _, _ in e.beam_search(p, 6, 4, eos=-1):
        lg = S.forward(p + toks, f64(w), cfg)[len(p) - 1 : -1]
        lse = np.log(np.sum(np.exp(lg - lg.max(-1, keepdims=True)), -1)) + lg.max(-1)
        want = float(np.sum(lg[np.arange(len(toks)), toks] - lse))
        assert abs(lp - want) < 1e-3
    e.close()


def test_model_folder_and_cpp_engine(ti, tmp_path):
    """Engine.load and the C++ InferenceEngine read the same folder and continue a prompt alike."""
    cfg, w = model("mixed")
    write_model(tmp_path / "m", cfg, w)
    p = tokens(cfg, 17, 72)
    ref = greedy_reference("mixed", p, 10)
    e = ti.Engine.load(str(tmp_path / "m"), "float32", max_seq=64, max_batch=2)
    assert e.generate([p], 10)[0].tolist() == ref
    with pytest.raises(ti.TiError, match="layer-stack"):
        e.set_tensor(ti.W_Q, 0, np.zeros((4, 4)))
    e.close()
    exe = os.path.join(ROOT, "tests", "cpp", "bin", "stack_check")
    if not os.path.exists(exe):
        subprocess.run(["make", "-s", "-C", ROOT, "test-bins"], check=True)
    r = subprocess.run([exe, str(tmp_path / "m"), "10"] + [str(t) for t in p], capture_output=True, text=True,
                       env=dict(os.environ, TI_FLOAT32="1"), timeout=100)
    assert r.returncode == 0, r.stdout + r.stderr
    got = [int(t) for t in r.stdout.split("tokens:")[1].split()]
    stop = ref.index(2) + 1 if 2 in ref else len(ref)
    assert got == p + ref[:stop]


def test_missing_weights_are_reported(ti, tmp_path):
    cfg, w = model("plain")
    e = ti.Engine.stack(cfg, "float32", max_seq=32)
    with pytest.raises(ti.TiError, match="embed has not been set"):
        e.step([1], [0])
    with pytest.raises(ti.TiError, match="no tensor"):
        e.set_weight("l0.mix.nothing", np.zeros((2, 2)))
    with pytest.raises(ti.TiError, match="expected"):
        e.set_weight("head", np.zeros((3, 48)))
    e.close()
    part = {k: v for k, v in w.items() if k != "l1.mix.sink"}
    write_model(tmp_path / "m", cfg, part)
    with pytest.raises(ti.TiError, match="lacks tensor l1.mix.sink"):
        ti.Engine.load(str(tmp_path / "m"), "float32", max_seq=32)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay(ti, tmp_path, dtype):
    """bin/trace_run: a batch of unequal prompts decoded together, then the slots used by a second batch."""
    cfg, w = model("loop_all")
    write_model(tmp_path / "m", cfg, w)
    os.makedirs(tmp_path / "out")
    seqs = {k: tokens(cfg, n, 900 + n) for k, n in (("a", 9), ("b", 75), ("c", 1), ("d", 30))}
    steps, at = [], {}

    def add(counts, end=()):
        ent = []
        for k, c in counts.items():
            lo = at.get(k, 0)
            ent.append(dict(id=k, tokens=seqs[k][lo : lo + c], want=list(range(c)) if lo == 0 or lo % 2 else []))
            at[k] = lo + c
        steps.append(dict(step=len(steps), entries=ent, end=list(end)))

    add(dict(a=5, b=67), ())
    for i in range(4):
        add(dict(a=1, b=1), ("a",) if i == 3 else ())
    for i in range(4):
        add(dict(b=1), ("b",) if i == 3 else ())
    add(dict(d=26, c=1), ("c",))
    for i in range(4):
        add(dict(d=1), ("d",) if i == 3 else ())
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", dtype,
                        "--out", str(tmp_path / "out"), "--max-tokens", "90", "--slots", "3"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=110)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(len(steps))]
    pos = {}
    for s in steps:
        ref = []
        for q in s["entries"]:
            lo = pos.get(q["id"], 0)
            ref += [reference("loop_all", seqs[q["id"]])[lo + k] for k in q["want"]]
            pos[q["id"]] = lo + len(q["tokens"])
        path = tmp_path / "out" / f"{s['step']}.f32"
        assert os.path.exists(path) == bool(ref)
        if ref:
            got = np.fromfile(path, "<f4").reshape(len(ref), cfg["vocab"])
            err = row_error(got, np.array(ref))
            assert (err.max() < TOL) if dtype == "float32" else (np.median(err) < 0.06), s["step"]
