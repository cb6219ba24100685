"""Layered decoders without a GPU: config reading, the registry, state sizes and refusals of the C ABI, and the
plain oracle checked against itself (a sequence in one run or continued; planted mistakes move its logits)."""
import copy
import ctypes
import json

import numpy as np
import pytest

import decoder_cases as C
from oracle import decoder_np as O


def engine_ctx(cfg, dtype=0, max_batch=4):
    """A bare context (no device memory is touched until weights are bound)."""
    from pgmi import _native as N
    from pgmi import registry
    c, layers = registry.decoder_config(cfg).native(max_batch, dtype)
    h = ctypes.c_void_p()
    N.check(N.lib().pgmi_decoder_create(0, ctypes.byref(c), layers, ctypes.byref(h)))
    return h


def test_reader_takes_every_size_from_the_file():
    from pgmi import registry
    d = registry.decoder_config(C.MIXED["a"])
    assert (d.vocab, d.width, d.streams, d.norm_groups, d.norm_eps, d.embed_scale) == (211, 84, 2, 3, 3e-5, 2.5)
    kinds = [layer.mixer for layer in d.layers]
    assert kinds == [0, 2, 1, 0, 2, 1]
    a = d.layers[2]
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.window, a.ff) == (6, 3, 24, 36, 40, 100)
    m = d.layers[3]
    assert (m.inner, m.state, m.dt_rank, m.conv, m.ff) == (40, 9, 3, 5, 28)
    assert d.layers[4].width == 68 and d.layers[4].ff == 0


@pytest.mark.parametrize("edit", [
    lambda c: c.pop("streams"), lambda c: c["norm"].pop("groups"), lambda c: c["layers"][0].update(type="other"),
    lambda c: c["layers"][2]["mlp"].update(kind="routed"), lambda c: c["layers"][2]["mixer"].pop("scale"),
    lambda c: c["layers"][2]["mixer"].pop("mask"), lambda c: c["layers"][0]["mixer"].pop("conv"),
    lambda c: c.update(architecture="Nothing")])
def test_reader_refuses_what_it_does_not_know(edit):
    from pgmi import registry
    cfg = copy.deepcopy(C.MIXED["a"])
    edit(cfg)
    with pytest.raises(ValueError):
        registry.decoder_config(cfg)


def test_registry_families(tmp_path):
    from pgmi import registry
    assert registry.family(C.MIXED["b"]) == "decoder"
    assert registry.family({"vision_config": {}, "text_config": {}}) == "paligemma"
    with pytest.raises(ValueError):
        registry.family({"model_type": "something"})
    (tmp_path / "config.json").write_text(json.dumps(C.MIXED["b"]))
    assert registry.read_config(str(tmp_path)) == C.MIXED["b"]


@pytest.mark.parametrize("name", list(C.MECHANISMS) + list(C.MIXED))
def test_weight_names_and_shapes(name):
    from pgmi import _native as N
    cfg = {**C.MECHANISMS, **C.MIXED}[name]
    ctx = engine_ctx(cfg)
    lib = N.lib()
    got, end = {}, 0
    for i in range(lib.pgmi_weight_count(ctx)):
        nm, off, shape, nd = ctypes.c_char_p(), ctypes.c_int64(), (ctypes.c_int64 * 4)(), ctypes.c_int()
        N.check(lib.pgmi_weight_info(ctx, i, ctypes.byref(nm), ctypes.byref(off), ctypes.byref(shape), ctypes.byref(nd)))
        got[nm.value.decode()] = tuple(shape[j] for j in range(nd.value))
        assert off.value >= end  # no overlap
        end = off.value + 2 * int(np.prod(got[nm.value.decode()]))
    assert got == O.tensor_shapes(cfg)
    assert end <= lib.pgmi_weights_bytes(ctx)
    lib.pgmi_destroy(ctx)


def test_state_bytes_scale_with_slots_and_tokens():
    from pgmi import _native as N
    lib = N.lib()
    for name, dtype in (("a", 0), ("a", 2), ("b", 0)):
        ctx = engine_ctx(C.MIXED[name], dtype)
        es = 4 if dtype == 2 else 2
        want = 0
        for layer in C.MIXED[name]["layers"]:
            m = layer["mixer"]
            r8 = lambda n: (n + 7) // 8 * 8
            if layer["type"] == "mamba1":
                parts = [5 * (m["conv"] - 1) * m["inner"] * 4, 5 * m["inner"] * m["state"] * 4]
            elif layer["type"] == "mingru":
                parts = [5 * m["width"] * 4]
            else:
                parts = [5 * m["kv_heads"] * 300 * r8(m[k]) * es for k in ("dim", "vdim")]
            want += sum((p + 255) // 256 * 256 for p in parts)
        assert lib.pgmi_kv_bytes(ctx, 5, 300) == want
        lib.pgmi_destroy(ctx)


@pytest.mark.parametrize("edit", [
    lambda c: c.update(streams=9), lambda c: c["norm"].update(groups=5), lambda c: c["layers"][2]["mixer"].update(kv_heads=4),
    lambda c: c["layers"][0]["mixer"].update(state=300), lambda c: c["layers"][1]["mixer"].update(width=0)])
def test_create_refuses_sizes_it_cannot_run(edit):
    cfg = copy.deepcopy(C.MIXED["a"])
    edit(cfg)
    with pytest.raises(ValueError):
        engine_ctx(cfg)


def test_calls_of_another_family_are_refused():
    from pgmi import _native as N
    ctx = engine_ctx(C.MIXED["a"])
    with pytest.raises(AssertionError):
        N.check(N.lib().pgmi_vision(ctx, None, 0, 1, None, None))
    N.lib().pgmi_destroy(ctx)


def test_oracle_continues_a_sequence():
    cfg = C.MIXED["a"]
    W = O.Weights(O.random_weights(cfg, 5))
    toks = np.random.default_rng(1).integers(0, cfg["vocab"], 60)
    whole = O.run(cfg, W, toks)
    st = O.new_state(cfg)
    cut = np.concatenate([O.run(cfg, W, toks[:23], st), O.run(cfg, W, toks[23:], st)])
    assert np.abs(whole - cut).max() < 1e-9


@pytest.mark.parametrize("mistake", ["window", "bias", "taps", "state", "streams", "groups", "unit_norm"])
def test_planted_mistakes_show(mistake, monkeypatch):
    """The random weights of the tests let every mechanism move the logits well past the tests' tolerances."""
    cfg = C.MIXED["a"]
    W = O.Weights(O.random_weights(cfg, 5))
    toks = np.random.default_rng(2).integers(0, cfg["vocab"], 90)
    good = O.run(cfg, W, toks)
    if mistake == "window":
        keys = O.window_keys
        monkeypatch.setattr(O, "window_keys", lambda i, n: keys(i, n + 1))
    elif mistake == "bias":
        monkeypatch.setattr(O, "distance_bias", lambda r1, r2, d: np.zeros((len(r1), len(d))))
    elif mistake == "taps":
        step = O.causal_conv_step
        monkeypatch.setattr(O, "causal_conv_step", lambda t, *a: step(np.zeros_like(t), *a))
    elif mistake == "state":
        monkeypatch.setattr(O, "selective_scan_step", lambda S, x, dt, A, B, Cc, D: ((dt * x)[:, None] * B) @ Cc + D * x)
    elif mistake == "streams":
        write = O.streams_write
        monkeypatch.setattr(O, "streams_write", lambda X, y, mix, out: write(X, y, np.asarray(mix).T, out))
    elif mistake == "groups":
        norm = O.group_rms_norm
        monkeypatch.setattr(O, "group_rms_norm", lambda x, w, g, eps: norm(x, w, 1, eps))
    else:
        monkeypatch.setattr(O, "unit_rms", lambda x, eps: x)
    bad = O.run(cfg, W, toks)
    rel = np.sqrt(((good - bad) ** 2).mean(1)) / np.sqrt((good ** 2).mean(1))
    assert rel.max() > 0.02, rel.max()
