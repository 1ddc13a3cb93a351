"""Nogitar models without a GPU: the oracle's own identities, configuration errors, argument checks."""
from __future__ import annotations

import ctypes as C
import json
import os

import numpy as np
import pytest

import nogitar_oracle as S
from nogitar_models import CONFIGS, MIXED, random_weights, shapes
from stack_models import f64, tokens, write_model


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_oracle_is_causal_and_finite(name):
    cfg = CONFIGS[name]
    w, t = f64(random_weights(cfg, 1)), tokens(cfg, 40, 2)
    full = S.forward(t, w, cfg)
    assert np.isfinite(full).all()
    np.testing.assert_allclose(S.forward(t[:17], w, cfg), full[:17], rtol=0, atol=1e-9)
    other = t[:20] + [(t[20] + 1) % cfg["vocab"]] + t[21:]
    assert np.abs(S.forward(other, w, cfg)[21:] - full[21:]).max(-1).min() > 1e-3   # every later row sees the change


def test_oracle_bigram_rows():
    assert S.bigram_rows([5, 7, 0], 10, 3, 2) == [10, (15 + 14) % 10, 21 % 10]


def test_oracle_sinusoid():
    p = S.sinusoid(4, 5)
    np.testing.assert_allclose(p[3], [np.sin(3), np.cos(3), np.sin(3 * 10000 ** -0.4), np.cos(3 * 10000 ** -0.4), np.sin(3 * 10000 ** -0.8)])


def test_oracle_temperature_steps():
    t = S.query_temperature(9, 0.5, 4)
    np.testing.assert_allclose(t[:3], 1.0)
    np.testing.assert_allclose(t[3:7], 1 + 0.5 * np.log(2))
    np.testing.assert_allclose(t[7:], 1 + 0.5 * np.log(3))


def test_oracle_softmax_plus_one():
    s = np.array([[0.3, -1.0, 2.0, -np.inf]])
    e = np.exp(s)
    np.testing.assert_allclose(S.softmax_plus_one(s), e / (1 + e.sum()))


def test_oracle_convolution_is_a_plain_one():
    rng = np.random.default_rng(0)
    x, w, b = rng.normal(size=(9, 2)), rng.normal(size=(2, 3)), rng.normal(size=2)
    got = S.causal_conv(x, w, b)
    for c in range(2):
        np.testing.assert_allclose(got[:, c], np.convolve(x[:, c], w[c][::-1])[:9] + b[c])


def test_oracle_recurrences_in_closed_form():
    """A state that never decays adds up; SSD with constant inputs is a geometric sum."""
    T = 6
    x, dt, one = np.ones((T, 1, 1)), np.full((T, 1), 0.5), np.ones((T, 1, 1))
    y = S.ssd_recurrence(x, dt, np.array([np.log(2.0)]), one, one, np.array([3.0]))[:, 0, 0]
    np.testing.assert_allclose(y, [3 + 0.5 * sum(np.exp(-1.0) ** k for k in range(t + 1)) for t in range(T)])
    u = np.ones((T, 1))
    s = S.lru_recurrence(u, 0 * u, u, np.array([0.0]))       # r = 0: a = 1, nothing enters
    np.testing.assert_allclose(s, 0.0, atol=1e-12)
    s = S.lru_recurrence(u, u, u, np.array([0.0]))[:, 0]
    a = np.exp(-8 * np.log(2.0))
    np.testing.assert_allclose(s, [np.sqrt(1 - a * a) * sum(a ** k for k in range(t + 1)) for t in range(T)])


def load_error(ti, folder):
    h = C.c_void_p()
    assert ti.lib().ti_engine_load(os.fsencode(str(folder)), ti.DT_F32, 16, 1, 0, C.byref(h)) != 0
    return ti.lib().ti_last_error().decode()


def test_load_reports_what_is_wrong(ti_host, tmp_path):
    w = random_weights(MIXED, 0)

    def broken(change):
        c = json.loads(json.dumps(MIXED))
        change(c)
        write_model(tmp_path / "m", c, w)
        return load_error(ti_host, tmp_path / "m")

    L = lambda i, **kw: (lambda c: c["layers"][i]["mixer"].update(**kw))
    assert "missing key \"bigram\"" in broken(lambda c: c["embedding"].pop("bigram"))
    assert "layer type \"latent_attention\"" in broken(lambda c: c["layers"][1].update(type="latent_attention"))
    assert "kind \"moe\"" in broken(lambda c: c["layers"][0]["mlp"].update(kind="moe"))
    assert "buckets" in broken(lambda c: c["embedding"]["bigram"].update(buckets=0))
    assert "every" in broken(lambda c: c["layers"][1]["mixer"]["q_temp"].update(every=0))
    assert "layer 1: attention sizes" in broken(L(1, kv_heads=4))
    assert "layer 3: cannot share" in broken(L(3, kv_from=3))
    assert "layer 3: cannot share" in broken(L(3, kv_from=0))
    assert "layer 6: cannot share" in broken(L(6, kv_from=3))
    assert "layer 6: cannot share" in broken(L(6, kv_from=5))
    assert "layer 2: SSD" in broken(L(2, groups=4))
    assert "layer 2: SSD" in broken(L(2, norm_groups=5))
    assert "state 300" in broken(L(2, state=300))
    assert "layer 0: RG-LRU" in broken(L(0, blocks=7))
    assert "missing key \"conv\"" in broken(lambda c: c["layers"][0]["mixer"].pop("conv"))


def test_argument_errors(ti_host):
    T, L = ti_host, ti_host.lib()
    d = T.DenseArgs(w=16, a=16, out=16, lda=64, ldo=64, M=1, N=16, K=64, batch=1, epi=T.DE_ACT, dtype=T.DT_BF16, t_cols=16)

    def err(**kw):
        b = type(d).from_buffer_copy(d)
        for k, v in kw.items():
            setattr(b, k, v)
        assert L.ti_dense(C.byref(b), None) in (1, 3)
        return L.ti_last_error().decode()

    assert "ACT" in err(t_cols=17)
    assert "ACT" in err(t_cols=8)               # fp32 columns without a place
    assert "ACT" in err(act=9)
    assert "LRU" in err(epi=T.DE_LRU)
    n = T.RownormArgs(x=16, M=1, H=8, w=16, kind=T.NORM_RMS, dtype=T.DT_F32)
    assert L.ti_rownorm(C.byref(n), None) == 1
    assert L.ti_gqa_block_elems(T.DT_BF16, 20, 28) == 64 * (32 + 32)
    assert L.ti_gqa_block_elems(T.DT_F32, 20, 28) == 64 * (32 + 32) and L.ti_gqa_block_elems(T.DT_F32, 16, 9) == 64 * 32
    for f in ("ti_gqa_prep", "ti_gqa_decode", "ti_gqa_prefill", "ti_conv", "ti_ssd_step", "ti_ssd_scan", "ti_ssd_norm", "ti_lru_scan", "ti_lru_step"):
        assert getattr(L, f)(None, None) == 1 and f in L.ti_last_error().decode()
    assert 1 <= L.ti_gqa_splits(1, 32, 4, 4096) <= 64 and L.ti_gqa_splits(512, 32, 4, 4096) == 1
    assert "l3.mix.k" not in shapes(MIXED) and "l1.mix.k" in shapes(MIXED)
