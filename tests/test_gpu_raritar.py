"""Raritar on the MI355X against the plain float64 oracle (oracle/raritar_np.py): each mechanism alone, whole prompts,
portions, single tokens, batches of unequal sequences, reused slots, window and kept-token edges, far keys, expert choice,
long decoding, replayed steps, greedy generation through the engine's own entry point, the trace runner, the command line."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import raritar_cases as C
from decoder_helpers import DTYPES, REPO, TOL, build, close, feed, rel, save, tokens
from oracle import raritar_np as R

pytestmark = pytest.mark.gpu
ALL = {**C.MECHANISMS, **{"mixed_" + k: v for k, v in C.MIXED.items()}}


# ---------------------------------------------------------------- mechanisms and whole models
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ALL))
def test_layers_and_logits_of_a_prompt(name, dtype):
    cfg = ALL[name]
    eng, W = build(cfg, dtype)
    toks = tokens(cfg, 150)
    taps = []
    want = R.run(cfg, W, toks, taps=taps)
    cache = eng.new_cache(2, 200)
    got = torch.zeros((len(cfg["layers"]), len(toks), cfg["width"]), device="cuda")
    lg = eng.forward(cache, [cache.alloc()], toks, [len(toks)], want=range(len(toks)), taps=got)
    for i, t in enumerate(np.stack(taps, 1)):
        close(got[i], t, dtype)
    close(lg, want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ALL))
def test_token_by_token(name, dtype):
    cfg = ALL[name]
    eng, W = build(cfg, dtype)
    toks = tokens(cfg, 100, 1)
    cache = eng.new_cache(2, 128)
    cache.slab.fill_(0x7F)
    got = feed(eng, cache, cache.alloc(), toks, [1], graph=True)
    close(got, R.run(cfg, W, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [[2], [3], [1, 2, 5, 4], [17, 1, 40], [63, 2], [64], [65, 64], [130, 3]])
@pytest.mark.parametrize("name", ["mixed_a", "mixed_b", "taps_7", "shared_kv"])
def test_portions(name, sizes, dtype):
    cfg = ALL[name]
    eng, W = build(cfg, dtype)
    toks = tokens(cfg, 200, 2)
    cache = eng.new_cache(3, 256)
    cache.alloc()
    got = feed(eng, cache, cache.alloc(), toks, sizes)
    close(got, R.run(cfg, W, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("lens", [[1, 70], [5, 1, 130], [64, 65, 63, 2, 129], [2 + r for r in range(19)]])
def test_unequal_batch_then_decoding(lens, dtype):
    """Prompts of unequal lengths in one step, then single tokens together; sequences leave one by one: batches of one row,
    of up to 16 (fused expert products), and of more."""
    cfg = C.MIXED["a"]
    eng, W = build(cfg, dtype)
    extra = 12
    seqs = [tokens(cfg, n + extra, 10 + n) for n in lens]
    want = [R.run(cfg, W, s) for s in seqs]
    cache = eng.new_cache(19, 160)
    slots = [cache.alloc() for _ in lens]
    lg = eng.step(cache, slots, [s[:n] for s, n in zip(seqs, lens)], want=list(range(sum(lens))))
    close(lg, np.concatenate([w[:n] for w, n in zip(want, lens)]), dtype)
    live = list(range(len(lens)))
    for t in range(extra):
        if t and t % 2 == 0 and len(live) > 1:
            cache.free(slots[live.pop(0)])
        lg = eng.step(cache, [slots[r] for r in live], [[seqs[r][lens[r] + t]] for r in live])
        close(lg, np.stack([want[r][lens[r] + t] for r in live]), dtype)


def test_mixed_portions_and_single_tokens_in_one_step():
    cfg = C.MIXED["b"]
    eng, W = build(cfg, "float32")
    seqs = [tokens(cfg, 90, 20), tokens(cfg, 90, 21), tokens(cfg, 90, 22)]
    want = [R.run(cfg, W, s) for s in seqs]
    cache = eng.new_cache(3, 100)
    slots = [cache.alloc() for _ in seqs]
    at = [0, 0, 0]
    for ns in ([40, 2, 7], [1, 30, 2], [2, 1, 66], [47, 57, 15]):
        lg = eng.step(cache, slots, [s[a:a + n] for s, a, n in zip(seqs, at, ns)], want=list(range(sum(ns))))
        close(lg, np.concatenate([w[a:a + n] for w, a, n in zip(want, at, ns)]), "float32")
        at = [a + n for a, n in zip(at, ns)]


@pytest.mark.parametrize("dtype", DTYPES)
def test_batch_equals_alone(dtype):
    cfg = C.MIXED["b"]
    eng, _ = build(cfg, dtype)
    seqs = [tokens(cfg, n, 30 + n) for n in (3, 64, 90, 17)]
    cache = eng.new_cache(6, 128)
    slots = [cache.alloc() for _ in seqs]
    together = eng.step(cache, slots, seqs).clone()
    for s in slots:
        cache.free(s)
    for r, s in enumerate(seqs):
        slot = cache.alloc()
        alone = eng.step(cache, [slot], [s])
        close(together[r:r + 1], alone.double().cpu().numpy(), dtype, 0.5)
        cache.free(slot)


def test_freed_slots_start_clean():
    cfg = C.MIXED["a"]
    eng, W = build(cfg, "float32")
    cache = eng.new_cache(2, 120)
    cache.slab.fill_(0x7F)  # NaN-like patterns everywhere: nothing of an old state may be read
    for k in range(4):
        toks = tokens(cfg, 30 + 20 * k, 40 + k)
        slot = cache.alloc()
        sizes = [[len(toks)], [1], [2], [25, 1]][k]
        close(feed(eng, cache, slot, toks, sizes), R.run(cfg, W, toks), "float32")
        cache.free(slot)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n", [1, 2, 3, 4, 5])
def test_first_tokens(n, dtype):
    """Prompts shorter than the convolution, in one step and token by token, in slots that held other sequences."""
    cfg = C.MIXED["a"]
    eng, W = build(cfg, dtype)
    cache = eng.new_cache(2, 64)
    slot = cache.alloc()
    eng.step(cache, [slot], [tokens(cfg, 20, 50)])
    cache.free(slot)
    toks = tokens(cfg, n + 4, 51)
    want = R.run(cfg, W, toks)
    for first in (n, 1):
        slot = cache.alloc()
        close(feed(eng, cache, slot, toks, [first, 1]), want, dtype)
        cache.free(slot)


# ---------------------------------------------------------------- window and kept-token edges, far keys
def standout(cfg, n_pairs, seed=6):
    """A single attention layer over three-part embeddings: the first part is a token's query code, the second its key
    code, the third feeds the values.  Tokens come in pairs (key vocab - 2k - 2, query vocab - 2k - 1) whose codes
    agree, so that one score stands out among all keys; the codes are projected to the dims that are not rotated."""
    W = R.random_weights(cfg, seed)
    rng = np.random.default_rng(seed)
    P = cfg["width"] // 3
    code = rng.standard_normal((2, cfg["vocab"], P))
    code *= np.sqrt(P) / np.sqrt((code ** 2).sum(-1, keepdims=True))
    for k in range(n_pairs):
        code[0, cfg["vocab"] - 2 * k - 1] = code[1, cfg["vocab"] - 2 * k - 2]
    W["embed"][:, :P], W["embed"][:, P:2 * P] = R.bf16(code[0]), R.bf16(code[1])
    W["embed"][:, 2 * P:] = R.bf16(rng.standard_normal((cfg["vocab"], P)))
    W["bigram"] = W["bigram"] * 0
    W["l0.canon1"] = W["l0.canon1"] * 0
    W["l0.norm1"] = W["l0.norm1"] * 0 + 1
    m = cfg["layers"][0]["mixer"]
    G, d, rot = m["kv_heads"], m["dim"], m["rot"]["dims"]
    proj = R.bf16(rng.standard_normal((G, d, P)) / np.sqrt(P))
    proj[:, :rot] = 0
    q, k = np.zeros_like(W["l0.mix.q"]), np.zeros_like(W["l0.mix.k"])
    q[:, :P] = np.repeat(proj, m["heads"] // G, 0).reshape(-1, P)
    k[:, P:2 * P] = proj.reshape(-1, P)
    W["l0.mix.q"], W["l0.mix.k"] = q, k
    W["l0.mix.v"][:, :2 * P] = 0
    W["l0.mix.o"] = R.bf16(rng.standard_normal(W["l0.mix.o"].shape) * (2.5 / np.sqrt(W["l0.mix.o"].shape[1])))
    return W


def plain_tokens(cfg, n, n_pairs, seed):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"] - 2 * n_pairs, n)]


def everywhere(eng, toks, want, dtype, cut):
    """The logits of a prompt in one step; of its last tokens decoded one by one; and of three of it decoded together."""
    n = len(toks)
    cache = eng.new_cache(4, n)
    slot = cache.alloc()
    close(eng.step(cache, [slot], [toks], want=list(range(n))), want, dtype)
    cache.free(slot)
    close(feed(eng, cache, cache.alloc(), toks, [cut, 1], graph=True), want, dtype)
    slots = [cache.alloc() for _ in range(3)]
    eng.step(cache, slots, [toks[:cut]] * 3)
    for t in range(cut, n):
        close(eng.step(cache, slots, [[toks[t]]] * 3), np.stack([want[t]] * 3), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size,keep,heads,kv,dim,vdim,cap", [
    (2, 1, 4, 2, 32, 24, 40.0), (63, 4, 3, 1, 64, 64, 40.0), (64, 64, 4, 4, 40, 72, 90.0), (65, 66, 8, 2, 96, 96, 40.0),
    (130, 20, 6, 3, 48, 128, 25.0), (64, 1, 2, 1, 264, 40, 40.0)])
def test_window_and_kept_edges(size, keep, heads, kv, dim, vdim, cap, dtype, monkeypatch):
    """A matching key at the window's last place, one place outside, and near them; and at the last kept token, the one
    after it, and the first: in a prompt and decoded.  The oracle with a window one wider or narrower, or one kept token
    more or fewer, must be far away at those positions."""
    rot = 8
    cfg = C.model([C.layer(heads, kv, dim, vdim, size, keep=keep, rot=rot, cap=cap, scale=16.0 / (dim - rot))], width=96,
                  vocab=400, mult=1.0)
    eng, W = build(cfg, dtype, weights=standout(cfg, 9))
    n = keep + 3 * size + 90
    toks = plain_tokens(cfg, n, 9, 7)
    at = []
    for k, dist in enumerate((size - 1, size, size - 1, size, max(1, size - 2), size + 1)):
        i = n - 1 - 6 * k
        toks[i - dist], toks[i] = cfg["vocab"] - 2 * k - 2, cfg["vocab"] - 2 * k - 1
        at.append(i)
    for k, j in ((6, keep - 1), (7, keep), (8, 0 if keep > 1 else keep + 1)):
        i = n - 3 - 6 * (k - 6)
        toks[j], toks[i] = cfg["vocab"] - 2 * k - 2, cfg["vocab"] - 2 * k - 1
        at.append(i)
    want = R.run(cfg, W, toks)
    visible = R.visible
    for wrong in ({"size": 1}, {"size": -1}, {"keep_first": 1}, {"keep_first": -1}):
        monkeypatch.setattr(R, "visible", lambda i, m, w=wrong: visible(i, {k: max(k == "size", m[k] + w.get(k, 0)) for k in m}))
        off = rel(R.run(cfg, W, toks), want)[at].max()
        monkeypatch.setattr(R, "visible", visible)
        assert off > 3 * TOL[dtype], (wrong, off)
    everywhere(eng, toks, want, dtype, n - 40)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("keep", [3, 200])
def test_far_key_among_hundreds(keep, dtype):
    """One matching key hundreds of tokens back, at a tile border or not, inside the window or kept."""
    cfg = C.model([C.layer(4, 2, 64, 64, 500, keep=keep, rot=16, cap=40.0, scale=17.0 / 48)], width=96, vocab=900, mult=1.0)
    eng, W = build(cfg, dtype, weights=standout(cfg, 5))
    toks = plain_tokens(cfg, 760, 5, 9)
    places = ((759, 261), (750, 2), (741, 320), (735, 256), (729, 0)) if keep == 3 else \
        ((759, 64), (750, 63), (741, 128), (735, 199), (729, 300))
    for k, (i, j) in enumerate(places):
        toks[j], toks[i] = cfg["vocab"] - 2 * k - 2, cfg["vocab"] - 2 * k - 1
    want = R.run(cfg, W, toks)
    lost = list(toks)
    for _, j in places:
        lost[j] = 5
    off = rel(R.run(cfg, W, lost), want)[[i for i, _ in places]].min()
    assert off > 3 * TOL[dtype], off
    everywhere(eng, toks, want, dtype, 725)


@pytest.mark.parametrize("dtype", DTYPES)
def test_rotation_far_from_the_start(dtype):
    """Angles of many turns: positions in the thousands, the fastest pairs one radian per token."""
    cfg = C.model([C.layer(2, 1, 16, 24, 40, keep=4, rot=16, base=30.0, scale=1.0)], width=48, vocab=60)
    eng, W = build(cfg, dtype)
    toks = tokens(cfg, 3000, 60)
    want = R.run(cfg, W, toks)
    cache = eng.new_cache(1, 3000)
    got = feed(eng, cache, cache.alloc(), toks, [2900, 60, 1], graph=True)
    close(got, want, dtype)


# ---------------------------------------------------------------- mixture of experts
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,mlp", [
    (104, C.moe(4, 24, 2, 40)), (104, C.moe(12, 72, 3, 16, identity=4, groups=(4, 2))), (104, C.moe(3, 136, 3, 8)),
    (104, C.moe(70, 16, 4, 8, identity=5, groups=(3, 2))), (576, C.moe(3, 512, 2, 24)), (512, C.moe(4, 520, 2, 16, identity=1))])
def test_long_expert_lists(width, mlp, dtype):
    """Hundreds of rows per expert and few: every row tile, in one step and in portions."""
    cfg = C.model([C.layer(2, 1, 16, 24, 30, keep=1, mlp=mlp)], width=width)
    eng, W = build(cfg, dtype)
    toks = tokens(cfg, 700, 61)
    want = R.run(cfg, W, toks)
    cache = eng.new_cache(2, 700)
    close(eng.step(cache, [cache.alloc()], [toks], want=range(700)), want, dtype)
    close(feed(eng, cache, cache.alloc(), toks, [333, 40, 100]), want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_choice_scores_below_zero_and_unused_experts(dtype):
    """Corrections far below zero: the other groups' experts must not win with a zero; experts nobody chooses."""
    cfg = C.model([C.layer(2, 1, 16, 24, 30, mlp=C.moe(11, 24, 3, 40, identity=1, groups=(3, 1)))])
    Wr = R.random_weights(cfg, 12)
    Wr["l0.mlp.correction"] = R.bf16(Wr["l0.mlp.correction"] - 5.0)
    Wr["l0.mlp.correction"][[1, 6, 9]] -= 40.0
    eng, W = build(cfg, dtype, weights=Wr)
    toks = tokens(cfg, 120, 62)
    want = R.run(cfg, W, toks)
    cache = eng.new_cache(2, 120)
    close(eng.step(cache, [cache.alloc()], [toks], want=range(120)), want, dtype)
    close(feed(eng, cache, cache.alloc(), toks, [60, 1], graph=True), want, dtype)


def test_router_without_numbers_stays_in_bounds():
    """Router scores that are not numbers give logits that are not numbers, and nothing worse."""
    cfg = C.model([C.layer(2, 1, 16, 24, 30, mlp=C.moe(6, 24, 3, 40, identity=1))])
    Wr = R.random_weights(cfg, 13)
    Wr["l0.mlp.router"][2] = np.nan
    for dtype in DTYPES:
        eng, _ = build(cfg, dtype, weights=Wr)
        cache = eng.new_cache(1, 90)
        slot = cache.alloc()
        assert torch.isnan(eng.step(cache, [slot], [tokens(cfg, 80, 63)])).all()
        assert torch.isnan(eng.step(cache, [slot], [[3]])).all()


# ---------------------------------------------------------------- long decoding, graphs, generation
@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dtype):
    cfg = C.MIXED["a"]
    eng, W = build(cfg, dtype)
    toks = tokens(cfg, 420, 50)
    cache = eng.new_cache(2, 420)
    got = feed(eng, cache, cache.alloc(), toks, [5, 1], graph=True)
    close(got, R.run(cfg, W, toks), dtype)


@pytest.mark.parametrize("dtype,B", [("bfloat16", 1), ("bfloat16", 2), ("bfloat16", 6), ("bfloat16", 20), ("float32", 1),
                                     ("float32", 3)])
def test_replayed_steps_equal_eager_steps(dtype, B):
    """Every replay against the eager step: same kernels, same bits; slots change between replays."""
    cfg = C.MIXED["b"]
    eng, _ = build(cfg, dtype)
    prompts = [tokens(cfg, 5 + 4 * r, 60 + r) for r in range(B)]
    ca, cb = eng.new_cache(B + 2, 128), eng.new_cache(B + 2, 128)
    sa, sb = [ca.alloc() for _ in range(B)], [cb.alloc() for _ in range(B)][::-1]
    eng.step(ca, sa, prompts)
    eng.step(cb, sb, prompts)
    ia = torch.arange(B, device="cuda") * 3 + 1
    ib = ia.clone()
    la = torch.empty((B, cfg["vocab"]), device="cuda")
    lb = torch.empty((B, cfg["vocab"]), device="cuda")
    for t in range(9):
        eng.decode(ca, sa, ia, logits=la, next_ids=ia, graph=True)
        x = (la * 2).sum()  # the program's own work between replays
        eng.decode(cb, sb, ib, logits=lb, next_ids=ib, graph=False)
        assert torch.equal(la, lb) and torch.equal(ia, ib), t
        assert torch.isfinite(x)
    rec = torch.empty((4, B), dtype=torch.int64, device="cuda")  # several steps per launch
    for t in range(3):
        eng.decode(ca, sa, ia, n_steps=4, logits=la, next_ids=ia, tokens=rec, graph=True)
        for k in range(4):
            eng.decode(cb, sb, ib, logits=lb, next_ids=ib, graph=False)
            assert torch.equal(rec[k], ib), (t, k)
        assert torch.equal(la, lb)


@pytest.mark.parametrize("B", [1, 2, 4])
def test_greedy_generation(B):
    """generate() through the registry's engine: the oracle's own greedy tokens (fp32; a token may differ only where
    the oracle's two best logits are within the tolerance)."""
    cfg = C.MIXED["a"]
    eng, W = build(cfg, "float32")
    prompts = [tokens(cfg, n, 70 + n) for n in (4, 37, 12, 81)[:B]]
    n = 21
    out = eng.generate(prompts, n, prefill_tokens=50).cpu().numpy()
    for r in range(B):
        toks, lg = R.greedy(cfg, W, prompts[r], n)
        for t in range(n):
            if out[r, t] != toks[t]:
                top = np.sort(lg[t])
                assert top[-1] - top[-2] < 1e-3 * np.abs(lg[t]).max(), (r, t)
                break


# ---------------------------------------------------------------- loading, the runner, the command line
def test_load_model_and_trace_runner(tmp_path):
    import utils
    cfg = C.MIXED["b"]
    Wr = R.random_weights(cfg, 8)
    save(cfg, Wr, tmp_path)
    W = R.Weights(Wr)
    eng = utils.load_model(str(tmp_path), device="cuda:0")
    toks = {"x": tokens(cfg, 40, 90), "y": tokens(cfg, 25, 91), "z": tokens(cfg, 1, 92)}
    want = {k: R.run(cfg, W, v) for k, v in toks.items()}
    cache = eng.new_cache(1, 64)
    close(eng.step(cache, [cache.alloc()], [toks["x"]], want=range(40)), want["x"], "bfloat16")
    del eng
    steps = [({"x": 30, "y": 20, "z": 1}, ["z"])] + [({"x": 1, "y": 1}, [])] * 4 + [({"x": 1, "y": 1}, ["y"])] + \
            [({"x": 1}, [])] * 4 + [({"x": 1}, ["x"])]
    for dtype in DTYPES:
        out = tmp_path / dtype
        out.mkdir()
        at, lines, rows = {}, [], []
        for n, (bring, end) in enumerate(steps):
            entries, w = [], []
            for k, c in bring.items():
                lo = at.get(k, 0)
                places = [] if n == 2 else sorted({0, c - 1})
                entries.append({"id": k, "tokens": toks[k][lo:lo + c], "want": places})
                w += [want[k][lo + p] for p in places]
                at[k] = lo + c
            lines.append(json.dumps({"step": n, "entries": entries, "end": end}))
            rows.append(w)
        p = subprocess.run([sys.executable, os.path.join(REPO, "bin", "trace_run"), "--model", str(tmp_path), "--dtype", dtype,
                            "--out", str(out), "--max-tokens", "64"], input="\n".join(lines) + "\n", capture_output=True,
                           text=True, timeout=100)
        assert p.returncode == 0, p.stderr[-2000:]
        assert [x for x in p.stdout.splitlines() if x.startswith("done")] == [f"done {n}" for n in range(len(steps))]
        for n, w in enumerate(rows):
            f = out / f"{n}.f32"
            assert f.exists() == bool(w)
            if w:
                close(np.fromfile(f, "<f4").reshape(len(w), -1).astype(np.float64), np.stack(w), dtype)


def test_command_line(tmp_path):
    from pgmi import registry
    cfg = C.MIXED["a"]
    save(cfg, R.random_weights(cfg, 11), tmp_path)
    prompts = [tokens(cfg, 6, 95), tokens(cfg, 14, 96)]
    want = registry.load_decoder(str(tmp_path)).generate(prompts, 7).cpu().tolist()
    cmd = [sys.executable, "-m", "pgmi", "--model", str(tmp_path), "--max-new-tokens", "7"]
    for p in prompts:
        cmd += ["--prompt", ",".join(map(str, p))]
    out = subprocess.run(cmd, capture_output=True, text=True, timeout=100,
                         cwd=os.path.join(REPO, "multimodal-financial-analysis-tool-using-paligemma_amd"))
    assert out.returncode == 0, out.stderr[-2000:]
    assert [[int(t) for t in x.split(",")] for x in out.stdout.split()] == want
