"""Nogitar engine against the whole-sequence oracle (oracle/nogitar_oracle.py): every kind of layer alone and
together, prompts, decoding, portions, batches, slots used again, generation, in fp32 and bf16.

The fp32 bar is TOL on every row: rms over the vocabulary of the difference to the fp64 oracle, relative to
the logits' rms.  A wrong key, position, tap or state moves rows by 1e-2 and more."""
from __future__ import annotations

import json
import os
import subprocess
import sys

import numpy as np
import pytest

import nogitar_oracle as S
from conftest import ROOT
from nogitar_models import CONFIGS, attn, config, mamba2, random_weights, rglru, shapes
from stack_models import engine, f64, row_error, tokens, write_model

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


def close(got, ref, what="", tol=TOL):
    e = row_error(got, ref)
    assert np.isfinite(np.asarray(got)).all() and e.max() < tol, f"{what}: row {int(e.argmax())} differs by {e.max():.2e}"


def new_engine(ti, name, dtype="float32", **kw):
    cfg, w = model(name)
    return engine(ti, cfg, {n: a.reshape(-1, a.shape[-1]) if a.ndim == 3 else a for n, a in w.items()}, dtype, **kw)


def build(ti, cfg, w, dtype="float32", **kw):
    return engine(ti, cfg, {n: a.reshape(-1, a.shape[-1]) if a.ndim == 3 else a for n, a in w.items()}, dtype, **kw)


# ------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_prompt_logits_and_layer_residuals(ti, name):
    cfg, w = model(name)
    t = tokens(cfg, 150, 5)
    lay = []
    ref = S.forward(t, f64(w), cfg, lay)
    e = new_engine(ti, name)
    got, gl = e.prefill(1, t, 0, range(len(t)), want_layers=True)
    e.close()
    assert gl.shape[0] == len(lay) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(gl, lay)):
        assert np.abs(a - b).max() < 2e-4 * np.abs(b).max(), f"layer {i}"
    close(got, ref, name)


@pytest.mark.parametrize("width", [32, 50, 33])
def test_embedding_alone(ti, width):
    """A layer whose norm weight is zero adds nothing: the residual is the embedding.  Positions past the
    tables' 256, in a prompt, in portions (the previous token comes from an earlier call) and decoded."""
    cfg = config(60, width, [(rglru(8, 1, 2), None)], emb_scale=3.0, bigram=(41, 5, 11))
    w = random_weights(cfg, 2)
    w["l0.norm1"][:] = 0
    t = tokens(cfg, 700, 3)
    ref = S.embed(t, f64(w), cfg)
    e = build(ti, cfg, w, max_seq=704, max_batch=2)
    lay = e.prefill(1, t, 0, [], want_layers=True)[1][0]
    assert np.abs(lay - ref).max() < 2e-6 * np.abs(ref).max()
    at = 0
    for n in (1, 2, 300, 1, 396):
        lay = e.prefill(0, t[at : at + n], at, [], want_layers=True)[1][0]
        assert np.abs(lay - ref[at : at + n]).max() < 2e-6 * np.abs(ref).max(), at
        at += n
    full = S.forward(t + [7, 9], f64(w), cfg)
    close(e.step([7, 7], [700, 700]), np.repeat(full[700:701], 2, 0), "decoded")
    close(e.step([9, 9], [701, 701]), np.repeat(full[701:702], 2, 0), "decoded")
    e.close()


@pytest.mark.parametrize("every,coef", [(1, 3.0), (5, 2.0), (64, 8.0), (2.5, 1.0)])
def test_query_temperature_edges(ti, every, coef):
    """Positions just before and at every step of the query scale, prompts and decoding."""
    cfg = config(60, 32, [(attn(4, 2, 16, 24, coef, every), None)])
    w = random_weights(cfg, 4, peak=1.0)
    t = tokens(cfg, 200, 6)
    ref = S.forward(t, f64(w), cfg)
    flat = json.loads(json.dumps(cfg))
    flat["layers"][0]["mixer"]["q_temp"]["coef"] = 0.0
    assert row_error(S.forward(t, f64(w), flat)[150:], ref[150:]).max() > 1e-2, "the scale must show"
    e = build(ti, cfg, w)
    close(e.prefill(0, t, 0, range(200)), ref, "prompt")
    e.prefill(1, t[:3])
    for i in range(3, 135):
        close(e.step_slots([1], [t[i]], [i]), ref[i : i + 1], f"position {i}")
    e.close()


def slow_decay_model(kind):
    """One layer whose state keeps everything (decays close to one): the first tokens still show at the end."""
    cfg = config(40, 32, [(mamba2(4, 16, 24, 2, 1, 4) if kind == "ssd" else rglru(48, 3, 4), None)])
    w = random_weights(cfg, 8)
    if kind == "ssd":
        w["l0.mix.A_log"][:] = -9.0
    else:
        w["l0.mix.lam"][:] = -11.0
    w["embed"][3] *= 40.0
    return cfg, w


@pytest.mark.parametrize("kind", ["ssd", "lru"])
def test_first_token_shows_at_the_end(ti, kind):
    cfg, w = slow_decay_model(kind)
    n = 1200
    t = [3] + tokens(cfg, n, 2)
    t = [t[0]] + [v if v != 3 else 4 for v in t[1:]]
    ref = S.forward(t, f64(w), cfg)
    other = S.forward([5] + t[1:], f64(w), cfg)
    assert row_error(other[-1:], ref[-1:])[0] > 3e-3, "the first token must show"
    e = build(ti, cfg, w, max_seq=1210, max_batch=2)
    close(e.prefill(0, t, 0, range(len(t))), ref, "prompt")
    for cut in (1, 2, 63, 64, 65, 700):
        e.prefill(1, t[:cut])
        close(e.prefill(1, t[cut:], cut), ref[-1:], f"cut at {cut}")
    e.prefill(1, t[: n - 90])
    got = np.concatenate([e.step_slots([1], [t[i]], [i]) for i in range(n - 90, n + 1)])
    close(got, ref[n - 90 :], "decoded")
    e.close()


@pytest.mark.parametrize("kind", ["ssd", "lru"])
def test_fast_and_mixed_decays(ti, kind):
    """Decays from one token to thousands in one layer, step sizes from tiny to large within a block."""
    cfg = config(60, 32, [(mamba2(8, 8, 16, 2, 2, 2) if kind == "ssd" else rglru(64, 2, 3), None)])
    w = random_weights(cfg, 9)
    if kind == "ssd":
        w["l0.mix.A_log"][:] = np.linspace(-8, 4, 8)
        w["l0.mix.in"][-8:] *= 6.0
    else:
        w["l0.mix.lam"][:] = np.linspace(-12, 6, 64)
        w["l0.mix.ra"] *= 3.0
    t = tokens(cfg, 330, 5)
    ref = S.forward(t, f64(w), cfg)
    e = build(ti, cfg, w, max_seq=330)
    close(e.prefill(0, t, 0, range(330)), ref, "prompt")
    e.prefill(1, t[:7])
    close(np.concatenate([e.step_slots([1], [t[i]], [i]) for i in range(7, 140)]), ref[7:140], "decoded")
    e.close()


@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7])
@pytest.mark.parametrize("kind", ["ssd", "lru"])
def test_convolution_taps(ti, taps, kind):
    """Each tap alone carries the layer; portions shorter than the taps, down to one token."""
    cfg = config(40, 32, [(mamba2(2, 16, 12, 1, 1, taps) if kind == "ssd" else rglru(24, 2, taps), None)])
    t = tokens(cfg, 40, taps)
    for tap in range(taps):
        w = random_weights(cfg, 10 + tap)
        w["l0.mix.conv"][:, [j for j in range(taps) if j != tap]] *= 0.0
        w["l0.mix.conv"][:, tap] *= taps ** 0.5
        ref = S.forward(t, f64(w), cfg)
        e = build(ti, cfg, w, max_seq=48, max_batch=2)
        close(e.prefill(0, t, 0, range(40)), ref, f"tap {tap}")
        at, got = 0, []
        for n in (1, 1, 2, 3, 1, 5, 2, 25):
            got.append(e.prefill(1, t[at : at + n], at, range(n)))
            at += n
        close(np.concatenate(got), ref, f"tap {tap} in portions")
        got = np.concatenate([e.step([t[i], t[i]], [i, i]) for i in range(12)])
        close(got[::2], ref[:12], f"tap {tap} decoded")
        close(got[1::2], ref[:12], f"tap {tap} decoded")
        e.close()


# ------------------------------------------------------------------ whole models
@pytest.mark.parametrize("name", ["mixed", "odd", "wide"])
@pytest.mark.parametrize("n", [1, 2, 3, 15, 16, 17, 63, 64, 65, 128, 129])
def test_prompt_lengths(ti, name, n):
    cfg, _ = model(name)
    t = tokens(cfg, n, 100 + n)
    e = new_engine(ti, name, max_seq=136)
    close(e.prefill(0, t, 0, range(n)), reference(name, t), f"{n} tokens")
    e.close()


@pytest.mark.parametrize("name", ["mixed", "odd", "wide"])
def test_token_by_token_equals_prompt(ti, name):
    cfg, _ = model(name)
    t = tokens(cfg, 140, 7)
    e = new_engine(ti, name, max_seq=140)
    got = np.concatenate([e.step([t[i]], [i]) for i in range(len(t))])
    e.close()
    close(got, reference(name, t), "decoded")


@pytest.mark.parametrize("name", ["mixed", "odd"])
@pytest.mark.parametrize("rows", [2, 3, 16, 17, 50, 64, 65])
def test_prompt_portions(ti, name, rows):
    cfg, _ = model(name)
    t = tokens(cfg, 150, 5)
    e = new_engine(ti, name)
    e.set_prefill(rows)
    got = e.prefill(2, t, 0, range(len(t)))
    cut = 3 * rows + 1 if 3 * rows + 1 < len(t) - 1 else rows
    a = e.prefill(0, t[:cut], 0, range(cut))
    b = e.prefill(0, t[cut:], cut, range(len(t) - cut))
    e.close()
    close(got, reference(name, t), f"chunks of {rows}")
    close(np.concatenate([a, b]), reference(name, t), f"cut at {cut}")


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_unequal_requests_in_one_batch(ti, name):
    cfg, _ = model(name)
    lens, steps = [1, 70, 129, 16], 30
    seqs = [tokens(cfg, n + steps, 40 + n) for n in lens]
    refs = [reference(name, s) for s in seqs]
    e = new_engine(ti, name)
    for i, (s, n) in enumerate(zip(seqs, lens)):
        close(e.prefill(i, s[:n]), refs[i][n - 1 : n], f"request {i} prompt")
    for k in range(steps):
        live = [0, 1, 2, 3] if k < 10 else [3, 0, 2] if k < 20 else [2, 0]   # some end earlier; rows in any order
        got = e.step_slots(live, [seqs[i][lens[i] + k] for i in live], [lens[i] + k for i in live])
        for r, i in enumerate(live):
            close(got[r : r + 1], refs[i][lens[i] + k][None], f"request {i} step {k}")
    e.close()


def test_idle_slots_keep_their_state(ti):
    """Slots that sit out some steps go on exactly where they stood."""
    cfg, _ = model("mixed")
    seqs = [tokens(cfg, 60, 300 + i) for i in range(3)]
    refs = [reference("mixed", s) for s in seqs]
    e = new_engine(ti, "mixed", max_seq=64, max_batch=3)
    at = [5, 20, 1]
    for i, s in enumerate(seqs):
        e.prefill(i, s[: at[i]])
    rng = np.random.default_rng(0)
    for k in range(40):
        live = [i for i in rng.permutation(3) if rng.random() < 0.6 and at[i] < 60]
        if not live:
            continue
        got = e.step_slots(live, [seqs[i][at[i]] for i in live], [at[i] for i in live])
        for r, i in enumerate(live):
            close(got[r : r + 1], refs[i][at[i]][None], f"step {k} slot {i}")
            at[i] += 1
    e.close()


@pytest.mark.parametrize("streams", [17, 33, 64, 70])
def test_many_streams(ti, streams):
    cfg, _ = model("mixed")
    seqs = [tokens(cfg, 5 + (i % 7) + 4, 500 + i) for i in range(streams)]
    e = new_engine(ti, "mixed", max_seq=64, max_batch=streams)
    for i, s in enumerate(seqs):
        e.prefill(i, s[:-4])
    for k in range(4):
        got = e.step([s[len(s) - 4 + k] for s in seqs], [len(s) - 4 + k for s in seqs])
        for i, s in enumerate(seqs):
            close(got[i : i + 1], reference("mixed", s)[len(s) - 4 + k][None], f"stream {i}")
    e.close()


def test_slots_are_used_again(ti):
    """A slot's next request starts from nothing, also when its first token is a decode step."""
    cfg, _ = model("mixed")
    e = new_engine(ti, "mixed")
    long_, short = tokens(cfg, 200, 1), tokens(cfg, 21, 2)
    e.prefill(0, long_)
    e.prefill(1, long_[:90])
    e.prefill(2, long_[:33])
    for slot in (0, 1):
        close(e.prefill(slot, short[:9]), reference("mixed", short)[8:9], f"slot {slot}")
    for i in range(9):
        close(e.step_slots([2], [short[i]], [i]), reference("mixed", short)[i : i + 1], f"decoded position {i}")
    for i in range(9, len(short)):
        got = e.step([short[i]] * 3, [i] * 3)
        close(got, np.repeat(reference("mixed", short)[i : i + 1], 3, 0), f"position {i}")
    e.close()


def test_a_state_does_not_go_back(ti):
    cfg, _ = model("mixed")
    t = tokens(cfg, 20, 1)
    e = new_engine(ti, "mixed", max_seq=64, max_batch=2)
    e.prefill(0, t[:10])
    for call in (lambda: e.prefill(0, t[5:8], 5), lambda: e.step([t[9], 0], [9, 0]), lambda: e.step_slots([0], [1], [11]),
                 lambda: e.generate([t[:3]], 2, [4])):
        with pytest.raises(ti.TiError, match="cannot go back"):
            call()
    with pytest.raises(ti.TiError, match="slot"):
        e.step_slots([1, 1], [0, 0], [0, 0])
    close(e.prefill(0, t[10:], 10), reference("mixed", t)[-1:])
    e.close()


def test_long_decoding(ti):
    cfg, _ = model("mixed")
    t = tokens(cfg, 600, 9)
    e = new_engine(ti, "mixed", max_seq=600, max_batch=2)
    ref = reference("mixed", t)
    e.prefill(1, t[:5])
    got = np.concatenate([e.step_slots([1], [t[i]], [i]) for i in range(5, len(t))])
    e.close()
    close(got, ref[5:], "long decode")


def test_long_prompt_over_chunks(ti):
    cfg, _ = model("odd")
    t = tokens(cfg, 2300, 4)      # more than one prefill chunk
    want = [0, 1, 63, 64, 2046, 2047, 2048, 2049, 2111, 2112, 2299]
    e = new_engine(ti, "odd", max_seq=2350, max_batch=1)
    got = e.prefill(0, t, 0, want)
    step = e.step([7], [2300])
    e.close()
    ref = reference("odd", t + [7])
    close(got, ref[want], "prompt")
    close(step, ref[2300:], "next token")


def test_prompt_attention_of_many_heads(ti):
    """Enough row tiles for the two-tile workgroups: heads per key/value head 1, 3 and 17, values of 2, 5 and 13
    tiles, in one portion and in two that start inside a block."""
    cfg = config(60, 40, [(attn(16, 16, 20, 20), None), (attn(24, 8, 36, 68), None), (attn(17, 1, 12, 200), None),
                          (attn(34, 2, 40, 33), None)])
    w = random_weights(cfg, 11)
    t = tokens(cfg, 1030, 12)
    ref = S.forward(t, f64(w), cfg)
    e = build(ti, cfg, w, max_seq=1030, max_batch=2)
    close(e.prefill(0, t, 0, range(len(t))), ref, "whole")
    e.prefill(1, t[:21])
    close(e.prefill(1, t[21:], 21, range(len(t) - 21)), ref[21:], "second portion")
    e.close()


def needle_model():
    """One attention layer of two heads on one key/value head: the query of token 1 meets the key of token 2
    with a score far above the others; tokens 0 are the rest."""
    cfg = config(16, 32, [(attn(2, 1, 8, 8, 0.1, 50, 1.0), None)], bigram=(3, 1, 1))
    w = {n: np.zeros(s, np.float32) for n, s in shapes(cfg).items()}
    rng = np.random.default_rng(0)
    w["embed"][:] = rng.normal(0, 0.05, w["embed"].shape)
    w["embed"][1, 4], w["embed"][2, 5], w["embed"][0, 6] = 40, 40, 40
    for n in w:
        if w[n].ndim == 1:
            w[n][:] = 1
    w["l0.mix.q"][:] = rng.normal(0, 0.02, w["l0.mix.q"].shape)
    w["l0.mix.k"][:] = rng.normal(0, 0.02, w["l0.mix.k"].shape)
    w["l0.mix.q"][[0, 8], 4] = 3.0
    w["l0.mix.k"][0, 5] = 3.0
    w["l0.mix.k"][1, 6] = 3.0
    w["l0.mix.v"][:] = rng.normal(0, 1, w["l0.mix.v"].shape)
    w["l0.mix.g"][:] = rng.normal(0, 0.05, w["l0.mix.g"].shape)
    w["l0.mix.o"][:] = rng.normal(0, 1, w["l0.mix.o"].shape)
    w["head"][:] = rng.normal(0, 1, w["head"].shape)
    return cfg, w


@pytest.mark.parametrize("n", [64, 65, 128, 129, 300])
def test_single_far_key(ti, n):
    """The one key a query looks for, at block borders, first and last, in prompts and decoding."""
    cfg, w = needle_model()
    wd = f64(w)
    e = build(ti, cfg, w, max_seq=384, max_batch=2)
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


def test_first_tokens_share_with_the_sink(ti):
    """With one or two keys of small scores the denominator's one carries much of the weight."""
    cfg, w = needle_model()
    w["l0.mix.q.norm"][:] = 0.2
    e = build(ti, cfg, w, max_seq=16)
    for t in ([2], [2, 1], [0, 1], [2, 0, 1]):
        ref = S.forward(t, f64(w), cfg)
        close(e.prefill(0, t, 0, range(len(t))), ref, str(t))
        got = np.concatenate([e.step_slots([1], [v], [i]) for i, v in enumerate(t)])
        close(got, ref, f"{t} decoded")
    e.close()


# ------------------------------------------------------------------ bf16
@pytest.mark.parametrize("name", ["mixed", "odd", "wide"])
def test_bf16_rows(ti, name):
    cfg, _ = model(name)
    t = tokens(cfg, 180, 5)
    ref = reference(name, t)
    e = new_engine(ti, name, "bfloat16")
    runs = {"whole": e.prefill(0, t, 0, range(len(t)))}
    e.set_prefill(33)
    runs["portions"] = e.prefill(1, t, 0, range(len(t)))
    runs["decoded"] = np.concatenate([e.step_slots([2], [t[i]], [i]) for i in range(100)])
    e.close()
    for what, got in runs.items():
        q = np.quantile(row_error(got, ref[: len(got)]), [0.5, 1.0])
        assert np.isfinite(got).all() and q[0] < 0.03 and q[1] < 0.12, (what, q)
    for what in ("portions", "decoded"):
        n = len(runs[what])
        assert np.median(row_error(runs[what], runs["whole"][:n])) < 0.02, what


# ------------------------------------------------------------------ entry points
def greedy_reference(name, prompt, n):
    cfg, w = model(name)
    out, lg = S.greedy(prompt, n, f64(w), cfg)
    for l in lg:   # every step decided by more than the engine's error
        s = np.sort(l)
        decided = bool(s[-1] - s[-2] > 1e-3 * np.abs(l).max())
        assert decided, "pick another prompt seed"
    return out


PROMPTS = ((3, 62), (40, 62), (1, 61), (17, 60), (70, 60))


def test_generation_entry_points(ti):
    """Greedy generate, batched generate, continuous batching through few slots, the device sampler with
    top_k = 1 and a beam of one all give the oracle's greedy continuation."""
    cfg, _ = model("mixed")
    prompts, n = [tokens(cfg, k, s) for k, s in PROMPTS], 12
    refs = [greedy_reference("mixed", p, n) for p in prompts]
    e = new_engine(ti, "mixed", max_seq=128, max_batch=3)
    for p, r in zip(prompts, refs):
        assert e.generate([p], n)[0].tolist() == r
    for a in (0, 2):
        assert e.generate(prompts[a : a + 3], n).tolist() == refs[a : a + 3]
    e.set_prefill(0)                                     # prompts through decode steps
    assert e.generate(prompts[:3], n).tolist() == refs[:3]
    e.set_prefill(16)
    assert e.serve(prompts, n, eos=-1, chunk=5) == refs
    stop = refs[1][3]
    assert e.serve(prompts, n, eos=stop, chunk=4)[1] == refs[1][: refs[1].index(stop) + 1]
    toks, _ = e.generate_sampled([prompts[1]], n, 1.0, 1, 1.0, np.full((1, n), 0.5))
    assert toks[0].tolist() == refs[1]
    beams = e.beam_search(prompts[3], n, 1, eos=-1)
    assert beams[0][0] == refs[3]
    e.close()


def test_generation_goes_on_where_it_stood(ti):
    """A second call that starts at the position the first one reached continues the same sequence."""
    cfg, _ = model("mixed")
    p = tokens(cfg, *PROMPTS[1])
    ref = greedy_reference("mixed", p, 12)
    e = new_engine(ti, "mixed", max_seq=128, max_batch=1)
    assert e.generate([p], 5)[0].tolist() == ref[:5]
    assert e.generate([[ref[4]]], 7, [len(p) + 4])[0].tolist() == ref[5:12]
    e.close()


def test_beam_search_scores(ti):
    """Forked caches and states: every beam's log-probability is that of its tokens under the oracle."""
    cfg, w = model("mixed")
    p = tokens(cfg, 20, 8)
    e = new_engine(ti, "mixed", max_seq=64, max_batch=4)
    for toks, lp, _, _ in e.beam_search(p, 6, 4, eos=-1):
        lg = S.forward(p + toks, f64(w), cfg)[len(p) - 1 : -1]
        lse = np.log(np.sum(np.exp(lg - lg.max(-1, keepdims=True)), -1)) + lg.max(-1)
        want = float(np.sum(lg[np.arange(len(toks)), toks] - lse))
        assert abs(lp - want) < 1e-3
    e.close()


def test_step_graph_replays_equal_fresh_steps(ti):
    """The same captured step replayed with other work between gives the eager prompt's rows every time."""
    cfg, _ = model("mixed")
    t = tokens(cfg, 40, 3)
    ref = reference("mixed", t)
    e = new_engine(ti, "mixed", max_seq=64, max_batch=2)
    for _ in range(3):
        e.prefill(0, t[:30])
        e.prefill(1, t[:17])
        for i in range(6):
            got = e.step([t[30 + i], t[17 + i]], [30 + i, 17 + i])
            close(got, np.stack([ref[30 + i], ref[17 + i]]), f"step {i}")
            e.sync()
    e.close()


def test_model_folder_and_cpp_engine(ti, tmp_path):
    cfg, w = model("mixed")
    write_model(tmp_path / "m", cfg, w)
    p = tokens(cfg, *PROMPTS[3])
    ref = greedy_reference("mixed", p, 10)
    e = ti.Engine.load(str(tmp_path / "m"), "float32", max_seq=64, max_batch=2)
    assert e.generate([p], 10)[0].tolist() == ref
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
    part = {k: v for k, v in w.items() if k != "l0.mix.ri.b"}
    write_model(tmp_path / "m", cfg, part)
    with pytest.raises(ti.TiError, match="lacks tensor l0.mix.ri.b"):
        ti.Engine.load(str(tmp_path / "m"), "float32", max_seq=32)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay(ti, tmp_path, dtype):
    """bin/trace_run: a batch of unequal prompts decoded together, one ending earlier, then its slots used by a
    second batch that starts with single tokens."""
    cfg, w = model("mixed")
    write_model(tmp_path / "m", cfg, w)
    os.makedirs(tmp_path / "out")
    seqs = {k: tokens(cfg, n, 900 + n) for k, n in (("a", 9), ("b", 75), ("c", 2), ("d", 30), ("e", 6))}
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
    add(dict(d=26, c=1, e=1), ())
    add(dict(c=1, d=1, e=1), ("c",))
    for i in range(3):
        add(dict(e=1, d=1), ("d",) if i == 2 else ())
    add(dict(e=1), ("e",))
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
            ref += [reference("mixed", seqs[q["id"]])[lo + k] for k in q["want"]]
            pos[q["id"]] = lo + len(q["tokens"])
        path = tmp_path / "out" / f"{s['step']}.f32"
        assert os.path.exists(path) == bool(ref)
        if ref:
            got = np.fromfile(path, "<f4").reshape(len(ref), cfg["vocab"])
            err = row_error(got, np.array(ref))
            assert (err.max() < TOL) if dtype == "float32" else (np.median(err) < 0.06), s["step"]
