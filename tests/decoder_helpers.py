"""What the layered decoders' GPU tests share: an engine with given weights, portions, and the comparison with the oracle."""
import json
import os

import numpy as np
import torch

from oracle import decoder_np, raritar_np

REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
# rms of a position's logit error over the rms of its logits
TOL = {"float32": 2e-4, "bfloat16": 6e-2}
DTYPES = ["float32", "bfloat16"]


def oracle(cfg):
    return {"Tuvodra": decoder_np, "Raritar": raritar_np}[cfg["architecture"]]


def build(cfg, dtype, seed=3, weights=None, **kw):
    from pgmi import DecoderEngine, registry
    W = oracle(cfg).random_weights(cfg, seed) if weights is None else weights
    eng = DecoderEngine(registry.decoder_config(cfg), dtype=dtype, **kw)
    eng.load_state_dict({k: torch.from_numpy(np.array(v)) for k, v in W.items()})
    eng.prepare()
    return eng, decoder_np.Weights(W)


def tokens(cfg, n, seed=0):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def rel(got, want):
    got = got.double().cpu().numpy() if torch.is_tensor(got) else got
    assert np.isfinite(got).all()
    return np.sqrt(((got - want) ** 2).mean(-1)) / np.sqrt((want ** 2).mean(-1))


def close(got, want, dtype, factor=1.0):
    e = rel(got, want)
    worst, mean, place, tol = float(e.max()), float(e.mean()), int(e.argmax()), factor * TOL[dtype]
    if dtype == "float32":
        assert worst <= tol, (worst, place, mean)
    else:  # single positions of a random model can magnify bf16 rounding: one in fifty (or one) past the tolerance
        over = int((e > tol).sum())
        assert worst <= 2 * tol and mean <= tol / 2 and over <= max(1, e.size // 50), (worst, place, mean, over)


def feed(eng, cache, slot, toks, sizes, graph=False):
    """All logits of toks brought in portions of the given sizes (the last size repeats)."""
    out, at, k = [], 0, 0
    while at < len(toks):
        n = min(sizes[min(k, len(sizes) - 1)], len(toks) - at)
        out.append(eng.step(cache, [slot], [toks[at:at + n]], want=list(range(n)), graph=graph).clone())
        at += n
        k += 1
    return torch.cat(out)


def save(cfg, W, path):
    from safetensors.torch import save_file
    save_file({k: torch.from_numpy(np.array(v)).bfloat16() for k, v in W.items()}, os.path.join(path, "model.safetensors"))
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
