"""Layer-stack models without a GPU: the oracle's own identities, configuration and checkpoint errors,
host-side argument checks."""
from __future__ import annotations

import ctypes as C
import json
import os

import numpy as np
import pytest

import stack_oracle as S
from stack_models import CONFIGS, MIXED, ONCE, f64, random_weights, shapes, tokens, write_model


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_oracle_is_causal_and_finite(name):
    cfg = CONFIGS[name]
    w, t = f64(random_weights(cfg, 1)), tokens(cfg, 40, 2)
    full = S.forward(t, w, cfg)
    assert np.isfinite(full).all()
    np.testing.assert_allclose(S.forward(t[:17], w, cfg), full[:17], rtol=0, atol=1e-9)


def test_oracle_sink_is_one_more_key_without_a_value():
    s = np.array([[0.3, -1.0, 2.0]])
    p = S.softmax_with_sink(s, np.array([[0.7]]))
    e = np.exp(np.array([0.3, -1.0, 2.0, 0.7]))
    np.testing.assert_allclose(p[0], (e / e.sum())[:3])


def test_oracle_rotation_depends_on_the_distance_only():
    rng = np.random.default_rng(0)
    q, k = rng.normal(size=(1, 1, 12)), rng.normal(size=(1, 1, 12))
    dots = [float(S.rotate_half(q, [p + 5], 12, 100.0)[0, 0] @ S.rotate_half(k, [p], 12, 100.0)[0, 0]) for p in (0, 3, 900)]
    np.testing.assert_allclose(dots, dots[0])


def test_oracle_schedule():
    assert S.schedule(MIXED) == [(0, None), (1, 0), (2, None), (1, 1), (2, None)]
    assert S.schedule(ONCE) == [(0, None), (1, 0)]


def load_error(ti, folder):
    h = C.c_void_p()
    assert ti.lib().ti_engine_load(os.fsencode(str(folder)), ti.DT_F32, 16, 1, 0, C.byref(h)) != 0
    return ti.lib().ti_last_error().decode()


def test_load_reports_what_is_wrong(ti_host, tmp_path):
    assert "cannot open" in load_error(ti_host, tmp_path / "none")
    cfg = json.loads(json.dumps(CONFIGS["plain"]))
    w = random_weights(cfg, 0)

    def broken(change):
        c = json.loads(json.dumps(cfg))
        change(c)
        write_model(tmp_path / "m", c, w)
        return load_error(ti_host, tmp_path / "m")

    assert "architecture \"Other\"" in broken(lambda c: c.update(architecture="Other"))
    assert "missing key \"vocab\"" in broken(lambda c: c.pop("vocab"))
    assert "layer type \"other\"" in broken(lambda c: c["layers"][1].update(type="other"))
    assert "kind \"dense\"" in broken(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    assert "expected an integer" in broken(lambda c: c.update(width=47.5))
    write_model(tmp_path / "m", cfg, w)
    with open(tmp_path / "m" / "model.safetensors", "r+b") as f:
        f.truncate(os.path.getsize(f.name) - 100)
    assert "extent" in load_error(ti_host, tmp_path / "m")
    with open(tmp_path / "m" / "model.safetensors", "r+b") as f:
        f.truncate(50)
    assert "not a safetensors file" in load_error(ti_host, tmp_path / "m")
    with open(tmp_path / "m" / "config.json", "w") as f:
        f.write('{"architecture": "Gegepel", ')
    assert "JSON" in load_error(ti_host, tmp_path / "m")


def test_stack_argument_errors(ti_host):
    T, L = ti_host, ti_host.lib()
    assert L.ti_dense_args_bytes() == C.sizeof(T.DenseArgs)
    d = T.DenseArgs(w=16, a=16, out=16, lda=64, ldo=64, M=1, N=16, K=64, batch=1, epi=T.DE_F32, dtype=T.DT_BF16)

    def err(fn, a, **kw):
        b = type(a).from_buffer_copy(a)
        for k, v in kw.items():
            setattr(b, k, v)
        assert fn(C.byref(b), None) in (1, 3)
        return L.ti_last_error().decode()

    assert "not padded" in err(L.ti_dense, d, K=48)
    assert "lda" in err(L.ti_dense, d, lda=32)
    assert "dtype" in err(L.ti_dense, d, dtype=7)
    assert "epilogue" in err(L.ti_dense, d, epi=40)
    assert "ROPE" in err(L.ti_dense, d, epi=T.DE_ROPE)
    assert "grouped" in err(L.ti_dense, d, tile_rows=16)
    assert "fragments" in err(L.ti_dense, d, epi=T.DE_KFRAG, head_w=16, key_blocks=8)
    r = T.RouteArgs(logits=16, ld=8, M=1, E=8, top=2, idx=16, wgt=16)
    assert "ti_route" in err(L.ti_route, r, top=9)
    assert "ti_route" in err(L.ti_route, r, tile_rows=16)
    assert L.ti_route_max_tiles(64, 8, 2, 16) == 16 and L.ti_route_max_tiles(1, 64, 4, 16) == 4
    n = T.RownormArgs(x=16, M=1, H=8, w=16, xn=16, ldn=8, kind=T.NORM_LAYER, dtype=T.DT_F32)
    assert "inconsistent" in err(L.ti_rownorm, n)
    c = T.StackConfig(10, 8, 1, 0, 0, 0, 1e-5, 1.0, T.DT_F32, 8, 1, 0)
    ok = T.StackLayer(0, 1, 8, 8, 8, 8, 8, 8, 1e4, 1.0, T.MLP_MOE, 4, 2, 8)
    h = C.c_void_p()
    for field, v in (("rot_dim", 7), ("top", 5), ("mixer", 3), ("vdim", 300), ("rot_dims", 10)):
        l = T.StackLayer.from_buffer_copy(ok)
        setattr(l, field, v)
        assert L.ti_engine_create_stack(C.byref(c), C.byref(l), C.byref(h)) in (1, 3), field
    assert set(n for n in shapes(MIXED) if n.startswith("l1.")) and "l1.norm2" not in shapes(MIXED)
