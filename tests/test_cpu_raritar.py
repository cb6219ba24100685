"""Raritar without a GPU: config reading, tensor names and state sizes of the C ABI, refusals, and the plain oracle checked
against itself (a sequence in one run or continued; planted mistakes move its logits)."""
import copy
import ctypes

import numpy as np
import pytest

import raritar_cases as C
from oracle import raritar_np as R
from test_cpu_decoder import engine_ctx

ALL = {**C.MECHANISMS, **{"mixed_" + k: v for k, v in C.MIXED.items()}}


def test_reader_takes_every_size_and_constant_from_the_file():
    from pgmi import registry
    d = registry.decoder_config(C.MIXED["a"])
    assert (d.vocab, d.width, d.streams, d.norm_groups, d.norm_eps, d.embed_scale) == (211, 84, 1, 1, 2e-5, 1.0)
    assert (d.plain_residual, d.norm_scalar, d.untied_head, d.residual_mult, d.canon_taps) == (True, True, True, 0.6, 4)
    assert (d.bigram_buckets, d.bigram_mul_prev, d.bigram_mul_cur) == (67, 5, 3)
    a, b, c, e = d.layers
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.keep_first, a.softcap, a.kv_from) == (6, 3, 24, 36, 40, 5, 30.0, -1)
    assert (a.rot_dims, a.rot_base, a.rot_original, a.qk_norm, a.v_norm, a.proj_bias, a.distance_bias) == (12, 1e4, 0, 0, 1, 0, 0)
    assert (a.experts, a.identity, a.top, a.groups, a.groups_keep, a.expert_ff, a.shared_ff, a.ff) == (7, 1, 3, 4, 2, 44, 52, 0)
    assert (b.kv_from, b.softcap, b.experts, b.window) == (0, 12.0, 0, 23)
    assert (c.rot_dims, c.rot_base, c.rot_factor, c.rot_low, c.rot_high, c.rot_original) == (48, 3000.0, 4.0, 1.0, 4.0, 120.0)
    assert (e.kv_from, e.keep_first, e.identity, e.top) == (0, 0, 3, 4)
    big = registry.decoder_config(C.MECHANISMS["pairs"])
    assert (big.bigram_mul_prev, big.bigram_mul_cur) == ((2 ** 31 - 1) % 1009, 999983 % 1009)


@pytest.mark.parametrize("edit", [
    lambda c: c.pop("residual_mult"), lambda c: c["canon"].pop("taps"), lambda c: c["layers"][0].update(type="mamba1"),
    lambda c: c["layers"][0]["mlp"].update(kind="dense"), lambda c: c["layers"][0]["mixer"].pop("rot"),
    lambda c: c["layers"][0]["mixer"].pop("scale"), lambda c: c["layers"][2]["mixer"]["rot"]["scaling"].pop("low"),
    lambda c: c["layers"][0]["mlp"]["router"].pop("top"), lambda c: c["layers"][0]["mlp"]["router"]["groups"].pop("keep"),
    lambda c: c["embedding"].pop("bigram"), lambda c: c["embedding"]["bigram"].update(buckets=0)])
def test_reader_refuses_what_it_does_not_know(edit):
    from pgmi import registry
    cfg = copy.deepcopy(C.MIXED["a"])
    edit(cfg)
    with pytest.raises(ValueError):
        registry.decoder_config(cfg)


@pytest.mark.parametrize("name", list(ALL))
def test_weight_names_and_shapes(name):
    from pgmi import _native as N
    ctx = engine_ctx(ALL[name])
    lib = N.lib()
    got, end = {}, 0
    for i in range(lib.pgmi_weight_count(ctx)):
        nm, off, shape, nd = ctypes.c_char_p(), ctypes.c_int64(), (ctypes.c_int64 * 4)(), ctypes.c_int()
        N.check(lib.pgmi_weight_info(ctx, i, ctypes.byref(nm), ctypes.byref(off), ctypes.byref(shape), ctypes.byref(nd)))
        got[nm.value.decode()] = tuple(shape[j] for j in range(nd.value))
        assert off.value >= end  # no overlap
        end = off.value + 2 * int(np.prod(got[nm.value.decode()]))
    assert got == R.tensor_shapes(ALL[name])
    assert end <= lib.pgmi_weights_bytes(ctx)
    lib.pgmi_destroy(ctx)


def test_state_bytes():
    """Keys and values once per layer that has its own, the convolution's ring in every layer, the tokens once."""
    from pgmi import _native as N
    r8, up = (lambda n: (n + 7) // 8 * 8), (lambda n: (n + 255) // 256 * 256)
    for name, dtype in (("a", 0), ("a", 2), ("b", 0)):
        cfg = C.MIXED[name]
        ctx = engine_ctx(cfg, dtype)
        want = up(5 * 300 * 4)
        for entry in cfg["layers"]:
            m = entry["mixer"]
            if "kv_from" not in m:
                want += sum(up(5 * m["kv_heads"] * 300 * r8(m[k]) * (4 if dtype == 2 else 2)) for k in ("dim", "vdim"))
            want += up(5 * cfg["canon"]["taps"] * cfg["width"] * 4)
        assert N.lib().pgmi_kv_bytes(ctx, 5, 300) == want
        N.lib().pgmi_destroy(ctx)


@pytest.mark.parametrize("edit", [
    lambda c: c["layers"][1]["mixer"].update(kv_from=1), lambda c: c["layers"][3]["mixer"].update(kv_from=1),
    lambda c: c["layers"][3]["mixer"].update(kv_from=2), lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26),
    lambda c: c["layers"][0]["mixer"]["rot"].update(dims=11), lambda c: c["layers"][0]["mixer"]["mask"].update(size=0),
    lambda c: c["layers"][0]["mixer"].update(softcap=-1.0), lambda c: c["layers"][0]["mixer"].update(kv_heads=4),
    lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=3),
    lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(keep=5),
    lambda c: c["layers"][0]["mlp"]["router"].update(top=5), lambda c: c["layers"][0]["mlp"]["router"].update(top=0),
    lambda c: c["layers"][0]["mlp"]["router"].update(experts=2000), lambda c: c["layers"][0]["mlp"]["expert"].update(ff=0)])
def test_create_refuses_sizes_it_cannot_run(edit):
    cfg = copy.deepcopy(C.MIXED["a"])
    edit(cfg)
    with pytest.raises(ValueError):
        engine_ctx(cfg)


# ---------------------------------------------------------------- the oracle
def test_oracle_continues_a_sequence():
    cfg = C.MIXED["a"]
    W = R.Weights(R.random_weights(cfg, 5))
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], 60)
    whole = R.run(cfg, W, toks)
    st = R.new_state(cfg)
    cut = np.concatenate([R.run(cfg, W, toks[:23], st), R.run(cfg, W, toks[23:], st)])
    assert np.abs(whole - cut).max() < 1e-9


def test_oracle_mechanisms_by_hand():
    assert R.bigram_row(None, 9, {"buckets": 7, "mul_prev": 3, "mul_cur": 2}) == 7
    assert R.bigram_row(5, 9, {"buckets": 7, "mul_prev": 3, "mul_cur": 2}) == 33 % 7
    assert list(R.visible(6, {"size": 2, "keep_first": 3})) == [0, 1, 2, 5, 6]
    assert list(R.visible(1, {"size": 1, "keep_first": 0})) == [1]
    f = R.rotary_frequencies({"base": 16.0, "dims": 4, "scaling": {"factor": 2.0, "low": 1.0, "high": 4.0, "original": 1000.0}})
    assert np.allclose(f, [1.0, 0.25])  # turns of 6.3 and 25 tokens, below 1000 / 4
    f = R.rotary_frequencies({"base": 16.0, "dims": 4, "scaling": {"factor": 2.0, "low": 1.0, "high": 4.0, "original": 2.0}})
    assert np.allclose(f, [0.5, 0.125])  # both longer than 2 / 1
    f = R.rotary_frequencies({"base": 16.0, "dims": 2, "scaling": {"factor": 2.0, "low": 1.0, "high": 3.0, "original": 4 * np.pi}})
    assert np.allclose(f, [0.75])  # original / turn = 2, half way
    x = R.rotate(np.array([[1.0, 0.0, 5.0]]), 3, {"base": 10.0, "dims": 2})
    assert np.allclose(x, [[np.cos(3), np.sin(3), 5.0]])
    z = np.log(np.array([0.4, 0.3, 0.2, 0.1]))
    r = {"top": 2, "groups": {"count": 2, "keep": 1}}
    assert [e for e, _ in R.route(z, np.zeros(4), r)] == [0, 1]
    picks = R.route(z, np.array([-1.0, -1.0, -0.5, -0.5]), r)  # every choice score negative
    assert [e for e, _ in picks] == [2, 3] and np.allclose([w for _, w in picks], [0.2, 0.1])
    y = np.zeros((2, 1))
    assert R.canon(y, np.array([3.0]), np.array([[7.0, 5.0, 2.0]]))[0] == 9.0
    assert R.canon(y, np.array([1.0]), np.array([[7.0, 5.0, 2.0]]))[0] == 1 + 2 + 15
    assert R.canon(y, np.array([0.0]), np.array([[7.0, 5.0, 2.0]]))[0] == 5 + 21


@pytest.mark.parametrize("mistake", ["window", "kept", "cap", "rotation", "scaling", "value_norm", "taps", "pairs", "first_pair",
                                     "correction", "weights", "groups", "identity", "shared", "mult", "kv_from"])
def test_planted_mistakes_show(mistake, monkeypatch):
    """The random weights of the tests let every mechanism move the logits well past the tests' tolerances."""
    cfg = copy.deepcopy(C.MIXED["a"])
    W = R.Weights(R.random_weights(cfg, 5))
    toks = np.random.default_rng(2).integers(0, cfg["vocab"], 150)
    good = R.run(cfg, W, toks)
    visible, route = R.visible, R.route
    if mistake == "window":
        monkeypatch.setattr(R, "visible", lambda i, m: visible(i, {**m, "size": m["size"] + 1}))
    elif mistake == "kept":
        monkeypatch.setattr(R, "visible", lambda i, m: visible(i, {**m, "keep_first": 0}))
    elif mistake == "cap":
        monkeypatch.setattr(R, "capped", lambda s, c: s)
        for layer in cfg["layers"]:
            layer["mixer"]["scale"] *= 4
        good = None
    elif mistake == "rotation":
        monkeypatch.setattr(R, "rotate", lambda x, pos, rot: x)
    elif mistake == "scaling":
        cfg["layers"][2]["mixer"]["rot"].pop("scaling")
    elif mistake == "value_norm":
        unit = R.unit_rms
        monkeypatch.setattr(R, "unit_rms", lambda x, eps: x if x.ndim == 2 else unit(x, eps))
    elif mistake == "taps":
        canon = R.canon
        monkeypatch.setattr(R, "canon", lambda e, h, w: canon(np.zeros_like(e), h, w))
    elif mistake == "pairs":
        monkeypatch.setattr(R, "bigram_row", lambda p, c, m: m["buckets"] if p is None else (c * m["mul_prev"] + p * m["mul_cur"])
                            % m["buckets"])
    elif mistake == "first_pair":
        row = R.bigram_row
        monkeypatch.setattr(R, "bigram_row", lambda p, c, m: row(0 if p is None else p, c, m))
    elif mistake == "correction":
        monkeypatch.setattr(R, "route", lambda z, c, r: route(z, c * 0, r))
    elif mistake == "weights":
        monkeypatch.setattr(R, "route", lambda z, c, r: [(e, w / sum(v for _, v in route(z, c, r))) for e, w in route(z, c, r)])
    elif mistake == "groups":
        monkeypatch.setattr(R, "route", lambda z, c, r: route(z, c, {**r, "groups": {"count": 1, "keep": 1}}))
    elif mistake == "identity":
        monkeypatch.setattr(R, "route", lambda z, c, r: [(e, w if e < r["experts"] else 0.0) for e, w in route(z, c, r)])
    elif mistake == "shared":
        monkeypatch.setattr(R, "sigmoid", lambda x: np.ones_like(x))
    elif mistake == "mult":
        cfg["residual_mult"] = 1.0
    else:
        cfg["layers"][3]["mixer"]["kv_from"] = 0
        cfg["layers"][3]["mixer"]["mask"] = dict(cfg["layers"][1]["mixer"]["mask"])
    bad = R.run(cfg, W, toks)
    if good is None:
        monkeypatch.undo()
        good = R.run(cfg, W, toks)
    rel = np.sqrt(((good - bad) ** 2).mean(1)) / np.sqrt((good ** 2).mean(1))
    assert rel.max() > 0.02, rel.max()
