"""Layered decoders on the MI355X against the plain float64 oracle (oracle/decoder_np.py): each mechanism alone, whole
prompts, portions, single tokens, batches of unequal sequences, reused slots, window edges, long decoding, greedy
generation through the engine's own entry point, and the trace runner."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import decoder_cases as C
from decoder_helpers import DTYPES, REPO, TOL, build, close, feed, rel, save, tokens
from oracle import decoder_np as O

pytestmark = pytest.mark.gpu
ALL = {**C.MECHANISMS, **{"mixed_" + k: v for k, v in C.MIXED.items()}}


# ---------------------------------------------------------------- products
@pytest.mark.parametrize("M,N,K", [(1, 80, 16), (5, 33, 8), (70, 203, 104), (300, 515, 264), (130, 4096, 1024),
                                   (1100, 2304, 1088), (2048, 6144, 2048), (64, 160, 4096)])
@pytest.mark.parametrize("act", [0, 2])
def test_matmul_any_shape(M, N, K, act):
    import ctypes

    from pgmi import _native as N_
    if act == 2:  # the fp32 form has one tile shape: smaller sizes say as much
        M, N = min(M, 200), min(N, 600)
    eng, _ = build(C.MECHANISMS["gru"], "float32")
    g = torch.Generator(device="cuda").manual_seed(M + N + K)
    A = torch.randn((M, K + 8), generator=g, device="cuda")
    A = A.bfloat16() if act == 0 else A
    W = torch.randn((2 * N, K), generator=g, device="cuda").bfloat16()
    bias = torch.randn(N, generator=g, device="cuda").bfloat16()
    ref = A[:, :K].float() @ W.float().t()
    tol = 2e-5 * K ** 0.5
    ldo = (N + 7) // 8 * 8
    dt = torch.bfloat16 if act == 0 else torch.float32
    scratch = torch.empty((M, 2 * N), device="cuda")
    s = N_.stream_handle(eng.device)

    def call(mode, out, ld, b=None):
        sp = ctypes.c_int()
        N_.check(eng.lib.pgmi_op_matmul(eng.ctx, A.data_ptr(), K + 8, W.data_ptr(), K, M, N, K, act, mode, N_.ptr(b),
                                        out.data_ptr(), ld, out.numel() * out.element_size(), scratch.data_ptr(),
                                        ctypes.byref(sp), s))
        return sp.value

    out = torch.full((M, ldo), float("nan"), dtype=dt, device="cuda")
    call(0, out, ldo, bias)
    want = ref[:, :N] + bias.float()
    assert ((out[:, :N].float() - want).abs() <= (8e-3 * want.abs() + 1e-2 if act == 0 else tol)).all()
    assert (out[:, N:] == 0).all()
    out = torch.full((M, N), float("nan"), device="cuda")
    call(1, out, N)
    assert (out - ref[:, :N]).abs().max() <= tol
    slabs = torch.full((8, M, N), float("nan"), device="cuda")
    sp = call(2, slabs, N)
    assert 1 <= sp <= 8 and (slabs[:sp].sum(0) - ref[:, :N]).abs().max() <= tol
    out = torch.full((M, ldo), float("nan"), dtype=dt, device="cuda")
    call(3, out, ldo)
    want = torch.nn.functional.silu(ref[:, :N]) * ref[:, N:]
    assert ((out[:, :N].float() - want).abs() <= (8e-3 * want.abs() + 1e-2 if act == 0 else 4 * tol * (1 + want.abs()))).all()
    assert (out[:, N:] == 0).all()


# ---------------------------------------------------------------- mechanisms and whole models
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(ALL))
def test_layers_and_logits_of_a_prompt(name, dtype):
    cfg = ALL[name]
    eng, W = build(cfg, dtype)
    toks = tokens(cfg, 150)
    taps = []
    want = O.run(cfg, W, toks, taps=taps)
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
    got = feed(eng, cache, cache.alloc(), toks, [1], graph=True)
    close(got, O.run(cfg, W, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [[2], [3], [1, 2, 5, 4], [17, 1, 40], [63, 2], [64], [65, 64], [130, 3]])
@pytest.mark.parametrize("name", ["mixed_a", "mixed_b"])
def test_portions(name, sizes, dtype):
    cfg = ALL[name]
    eng, W = build(cfg, dtype)
    toks = tokens(cfg, 200, 2)
    cache = eng.new_cache(3, 256)
    cache.alloc()
    got = feed(eng, cache, cache.alloc(), toks, sizes)
    close(got, O.run(cfg, W, toks), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("lens", [[1, 70], [5, 1, 130], [64, 65, 63, 2, 129], [2 + r for r in range(17)]])
def test_unequal_batch_then_decoding(lens, dtype):
    """Prompts of unequal lengths in one step, then single tokens together; sequences leave one by one, so every
    batch size down to one is decoded (every form of the decode projections: one row, up to 16, more)."""
    cfg = C.MIXED["a"]
    eng, W = build(cfg, dtype)
    extra = 12
    seqs = [tokens(cfg, n + extra, 10 + n) for n in lens]
    want = [O.run(cfg, W, s) for s in seqs]
    cache = eng.new_cache(17, 160)
    slots = [cache.alloc() for _ in lens]
    lg = eng.step(cache, slots, [s[:n] for s, n in zip(seqs, lens)], want=list(range(sum(lens))))
    close(lg, np.concatenate([w[:n] for w, n in zip(want, lens)]), dtype)
    live = list(range(len(lens)))
    for t in range(extra):
        if t and t % 3 == 0 and len(live) > 1:
            cache.free(slots[live.pop(0)])
        lg = eng.step(cache, [slots[r] for r in live], [[seqs[r][lens[r] + t]] for r in live])
        close(lg, np.stack([want[r][lens[r] + t] for r in live]), dtype)


def test_mixed_portions_and_single_tokens_in_one_step():
    cfg = C.MIXED["b"]
    eng, W = build(cfg, "float32")
    seqs = [tokens(cfg, 90, 20), tokens(cfg, 90, 21), tokens(cfg, 90, 22)]
    want = [O.run(cfg, W, s) for s in seqs]
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
        close(feed(eng, cache, slot, toks, sizes), O.run(cfg, W, toks), "float32")
        cache.free(slot)
    with pytest.raises(ValueError):
        cache.free(slot)
    with pytest.raises(ValueError):
        eng.step(cache, [slot], [[1]])


# ---------------------------------------------------------------- window edges, far keys
def standout(cfg, n_pairs, seed=6):
    """A single attention layer over three-part embeddings: the first part is a token's query code, the second its key
    code, the third feeds the values.  Tokens come in pairs (key vocab - 2k - 2, query vocab - 2k - 1) whose codes
    agree, so that one score stands out among all keys of the window."""
    W = O.random_weights(cfg, seed)
    P = cfg["width"] // 3
    for k in range(n_pairs):
        W["embed"][cfg["vocab"] - 2 * k - 1][:P] = W["embed"][cfg["vocab"] - 2 * k - 2][P:2 * P]
    m = cfg["layers"][0]["mixer"]
    code = O.random_weights({**cfg, "vocab": 4}, seed + 1)["l0.mix.k"][:, :P].reshape(m["kv_heads"], m["dim"], P)
    q, k = np.zeros_like(W["l0.mix.q"]), np.zeros_like(W["l0.mix.k"])
    q[:, :P] = np.repeat(code, m["heads"] // m["kv_heads"], 0).reshape(-1, P)
    k[:, P:2 * P] = code.reshape(-1, P)
    W["l0.mix.q"], W["l0.mix.k"] = q, k
    W["l0.mix.v"][:, :2 * P] = 0
    for n in ("l0.mix.q.b", "l0.mix.k.b"):
        W[n] = W[n] * 0
    W["l0.mix.r1"] = W["l0.mix.r1"] * 0 + 0.25
    W["l0.mix.v"], W["l0.mix.o"] = W["l0.mix.v"] * 2, W["l0.mix.o"] * 2
    return W


def plain_tokens(cfg, n, n_pairs, seed):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"] - 2 * n_pairs, n)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("size,heads,kv,dim,vdim", [(2, 4, 2, 32, 24), (63, 3, 1, 64, 64), (64, 4, 4, 40, 72),
                                                    (65, 8, 2, 96, 96), (200, 6, 3, 48, 128)])
def test_window_edges(size, heads, kv, dim, vdim, dtype, monkeypatch):
    """A matching key exactly at the window's last place, one place outside, and near them: in a prompt and decoded.
    The oracle with its window one wider or narrower must be far away at those positions."""
    cfg = C.model([C.attn(heads, kv, dim, vdim, size, scale=13.0 / dim)], width=96, streams=2, groups=3, vocab=400,
                  escale=1.5)
    Wr = standout(cfg, 6)
    eng, W = build(cfg, dtype, weights=Wr)
    n = 3 * size + 80
    toks = plain_tokens(cfg, n, 6, 7)
    pairs = []
    for k, dist in enumerate((size - 1, size, size - 1, size, max(1, size - 2), size + 1)):
        i = n - 1 - 6 * k
        toks[i - dist], toks[i] = cfg["vocab"] - 2 * k - 2, cfg["vocab"] - 2 * k - 1
        pairs.append(i)
    want = O.run(cfg, W, toks)
    keys = O.window_keys
    for wrong in (-1, 1):
        monkeypatch.setattr(O, "window_keys", lambda i, s, w=wrong: keys(i, max(1, s + w)))
        off = rel(O.run(cfg, W, toks), want)[pairs].max()
        monkeypatch.setattr(O, "window_keys", keys)
        assert off > 3 * TOL[dtype], off
    cache = eng.new_cache(4, n)
    slot = cache.alloc()
    close(eng.step(cache, [slot], [toks], want=list(range(n))), want, dtype)
    cache.free(slot)
    slot, cut = cache.alloc(), n - 40
    got = feed(eng, cache, slot, toks, [cut, 1], graph=True)
    close(got, want, dtype)
    cache.free(slot)
    slots = [cache.alloc() for _ in range(3)]  # the batched decode form
    eng.step(cache, slots, [toks[:cut]] * 3)
    for t in range(cut, n):
        lg = eng.step(cache, slots, [[toks[t]]] * 3)
        close(lg, np.stack([want[t]] * 3), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_far_key_among_hundreds(dtype):
    """One matching key hundreds of tokens back, at a tile border or not, inside a window of many tiles."""
    cfg = C.model([C.attn(4, 2, 64, 64, 700, scale=14.0 / 64)], width=96, streams=2, groups=3, vocab=900, escale=1.5)
    Wr = standout(cfg, 5)
    eng, W = build(cfg, dtype, weights=Wr)
    toks = plain_tokens(cfg, 760, 5, 9)
    places = ((759, 64), (750, 63), (741, 128), (701, 2), (699, 0))
    for k, (i, j) in enumerate(places):
        toks[j], toks[i] = cfg["vocab"] - 2 * k - 2, cfg["vocab"] - 2 * k - 1
    want = O.run(cfg, W, toks)
    lost = list(toks)
    for _, j in places:
        lost[j] = 5
    off = rel(O.run(cfg, W, lost), want)[[i for i, _ in places]].min()
    assert off > 3 * TOL[dtype], off
    cache = eng.new_cache(2, 800)
    close(eng.step(cache, [cache.alloc()], [toks], want=list(range(760))), want, dtype)
    got = feed(eng, cache, cache.alloc(), toks, [690, 1], graph=True)
    close(got[690:], want[690:], dtype)


# ---------------------------------------------------------------- long decoding, graphs, generation
@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dtype):
    cfg = C.MIXED["a"]
    eng, W = build(cfg, dtype)
    toks = tokens(cfg, 420, 50)
    cache = eng.new_cache(2, 420)
    got = feed(eng, cache, cache.alloc(), toks, [5, 1], graph=True)
    close(got, O.run(cfg, W, toks), dtype)


@pytest.mark.parametrize("B", [1, 2, 3, 6])
def test_replayed_steps_equal_eager_steps(B):
    """Every replay against the eager step: same kernels, same bits; slots change between replays."""
    cfg = C.MIXED["b"]
    eng, _ = build(cfg, "bfloat16")
    prompts = [tokens(cfg, 5 + 9 * r, 60 + r) for r in range(B)]
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
    # several steps per launch
    rec = torch.empty((4, B), dtype=torch.int64, device="cuda")
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
        toks, lg = O.greedy(cfg, W, prompts[r], n)
        for t in range(n):
            if out[r, t] != toks[t]:
                top = np.sort(lg[t])
                assert top[-1] - top[-2] < 1e-3 * np.abs(lg[t]).max(), (r, t)
                break


def test_generation_stop_tokens_and_sampling():
    cfg = C.MIXED["a"]
    eng, _ = build(cfg, "bfloat16")
    prompts = [tokens(cfg, 9, 80), tokens(cfg, 30, 81), tokens(cfg, 3, 82)]
    free = eng.generate(prompts, 16).cpu()
    eos = int(free[1, 5])
    out, lens = eng.generate(prompts, 16, eos_token_id=eos, pad_token_id=0, sync_every=4, return_lengths=True)
    for r in range(3):
        hit = (free[r] == eos).nonzero()
        n = int(hit[0]) + 1 if len(hit) else 16
        assert int(lens[r]) == n and torch.equal(out[r, :n].cpu(), free[r, :n])
        assert (out[r, n:] == 0).all()
    g = torch.Generator(device="cuda").manual_seed(5)
    a = eng.generate(prompts, 8, do_sample=True, temperature=0.9, top_p=0.8, generator=g).cpu()
    b = eng.generate(prompts, 8, do_sample=True, temperature=0.9, top_p=0.8,
                     generator=torch.Generator(device="cuda").manual_seed(5)).cpu()
    assert torch.equal(a, b) and int(a.min()) >= 0 and int(a.max()) < cfg["vocab"]
    tiny = eng.generate(prompts, 8, do_sample=True, temperature=0.9, top_p=1e-9).cpu()
    assert torch.equal(tiny, free[:, :8])  # a nucleus of one token is the argmax


# ---------------------------------------------------------------- loading, refusals, the runner
def test_load_model_and_trace_runner(tmp_path):
    import utils
    cfg = C.MIXED["b"]
    Wr = O.random_weights(cfg, 8)
    save(cfg, Wr, tmp_path)
    W = O.Weights(Wr)
    eng = utils.load_model(str(tmp_path), device="cuda:0")
    toks = {"x": tokens(cfg, 40, 90), "y": tokens(cfg, 25, 91), "z": tokens(cfg, 1, 92)}
    want = {k: O.run(cfg, W, v) for k, v in toks.items()}
    cache = eng.new_cache(1, 64)
    close(eng.step(cache, [cache.alloc()], [toks["x"]], want=range(40)), want["x"], "bfloat16")
    del eng
    steps = [({"x": 30, "y": 20, "z": 1}, ["z"])] + [({"x": 1, "y": 1}, [])] * 4 + [({"x": 1, "y": 1}, ["y"])] + \
            [({"x": 1}, [])] * 4 + [({"x": 1}, ["x"])]
    steps.append(({"z": 1}, ["z"]))
    for dtype in DTYPES:
        out = tmp_path / dtype
        out.mkdir()
        at, lines, rows = {}, [], []
        for n, (bring, end) in enumerate(steps):
            if n == len(steps) - 1:
                at["z"] = 0
            entries, w = [], []
            for k, c in bring.items():
                lo = at.get(k, 0)
                places = [] if n == 2 else sorted({0, c - 1})
                entries.append({"id": k + ("2" if n == len(steps) - 1 else ""), "tokens": toks[k][lo:lo + c], "want": places})
                w += [want[k][lo + p] for p in places]
                at[k] = lo + c
            ends = [e + "2" for e in end] if n == len(steps) - 1 else end
            lines.append(json.dumps({"step": n, "entries": entries, "end": ends}))
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
    save(cfg, O.random_weights(cfg, 11), tmp_path)
    prompts = [tokens(cfg, 6, 95), tokens(cfg, 14, 96)]
    want = registry.load_decoder(str(tmp_path)).generate(prompts, 7).cpu().tolist()
    cmd = [sys.executable, "-m", "pgmi", "--model", str(tmp_path), "--max-new-tokens", "7"]
    for p in prompts:
        cmd += ["--prompt", ",".join(map(str, p))]
    out = subprocess.run(cmd, capture_output=True, text=True, timeout=100,
                         cwd=os.path.join(REPO, "multimodal-financial-analysis-tool-using-paligemma_amd"))
    assert out.returncode == 0, out.stderr[-2000:]
    assert [[int(t) for t in x.split(",")] for x in out.stdout.split()] == want


def test_refusals():
    cfg = C.MECHANISMS["gru"]
    eng, _ = build(cfg, "bfloat16", max_batch=2)
    cache = eng.new_cache(3, 16)
    a, b, c = (cache.alloc() for _ in range(3))
    with pytest.raises(MemoryError):
        cache.alloc()
    with pytest.raises(ValueError):
        eng.step(cache, [a], [[cfg["vocab"]]])
    with pytest.raises(ValueError):
        eng.step(cache, [a], [[1] * 17])
    with pytest.raises(ValueError):
        eng.step(cache, [a, a], [[1], [2, 3]])
    with pytest.raises(ValueError):
        eng.step(cache, [a, b, c], [[1], [2], [3, 4]])
    with pytest.raises(ValueError):
        eng.step(cache, [a], [[]])
    eng.step(cache, [a], [[1] * 16])
    with pytest.raises(ValueError):
        eng.step(cache, [a], [[1]])
    assert cache.length[a] == 16
