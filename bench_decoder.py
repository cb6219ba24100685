"""The layered-decoder legs of bench.py (`python bench.py --decoder 1b,2b,7b,raritar-2b`): prefill and decode throughput of
Tuvodra and Raritar at the layer sizes of real models (random weights), one JSON line per size, and for Tuvodra "2b"
PaliGemma's text decoder at the same width, feed-forward and vocabulary beside it.  One GPU."""
from __future__ import annotations

import gc
import json
import time

import torch

HBM_PEAK_GBS = 8000.0
PREFILLS = ((1, 512), (1, 2048), (8, 512))  # (sequences, tokens each)
BATCHES = (1, 2, 4, 8)
CONTEXT = 1024


def timed(fn, steps, warmup):
    """Milliseconds per call over exactly `steps` calls after `warmup` untimed ones."""
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(steps):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / steps * 1e3


def decode_entry(ms, B, weight_bytes):
    return {"ms_per_step": round(ms, 4), "tok_s": round(B / ms * 1e3, 1),
            "weights_GBs": round(weight_bytes / ms / 1e6, 1), "frac_hbm": round(weight_bytes / ms / 1e6 / HBM_PEAK_GBS, 4)}


def step_bytes(eng, cfg, B):
    """Weight bytes a decode step of B sequences reads: every weight once (a table's rows not counted, the embedding where
    it is the output matrix), of a mixture the experts that B rows choose on average."""
    total = 0.0
    for name, v in eng.views.items():
        n = v.numel() * 2
        if name == "bigram" or (name == "embed" and cfg.untied_head):
            n = 0
        elif ".mlp.e" in name:
            layer = cfg.layers[int(name[1:name.index(".")])]
            n *= 1.0 - (1.0 - layer.top / (layer.experts + layer.identity)) ** B
        total += n
    return total


def decoder_leg(size, steps, warmup, seed, dev):
    from pgmi import DecoderEngine, registry
    from pgmi.synthetic import decoder_bench_config, decoder_policy
    raw = decoder_bench_config(size)
    cfg = registry.decoder_config(raw)
    eng = DecoderEngine(cfg, device=dev)
    eng.fill_synthetic(seed, decoder_policy)
    eng.prepare()
    V = cfg.vocab
    weight_bytes = sum(v.numel() * 2 for v in eng.views.values())
    out = {"params_bytes": weight_bytes, "prefill": {}, "decode": {}}
    for B, T in PREFILLS:
        cache = eng.new_cache(B, T)
        slots = [cache.alloc() for _ in range(B)]
        toks = torch.randint(0, V, (B * T,), device=dev)

        def prefill():
            for s in slots:
                cache.length[s] = 0
            eng.forward(cache, slots, toks, [T] * B)

        ms = timed(prefill, max(3, steps // 20), 3)
        out["prefill"][f"{B}x{T}"] = {"ms": round(ms, 3), "tok_s": round(B * T / ms * 1e3, 1)}
        del cache
    for B in BATCHES:
        cache = eng.new_cache(B, CONTEXT + steps + warmup + 8)
        slots = [cache.alloc() for _ in range(B)]
        eng.forward(cache, slots, torch.randint(0, V, (B * CONTEXT,), device=dev), [CONTEXT] * B)
        ids = torch.randint(0, V, (B,), device=dev)
        lg = torch.empty((B, V), device=dev)
        ms = timed(lambda: eng.decode(cache, slots, ids, logits=lg, next_ids=ids, graph=True), steps, max(3, warmup))
        out["decode"][f"{B}x{CONTEXT}"] = decode_entry(ms, B, step_bytes(eng, cfg, B))
        del cache
    return raw, out


def gemma_leg(steps, warmup, seed, dev):
    """PaliGemma-3B's text decoder alone (no image): the closest existing model."""
    from pgmi import Engine
    from pgmi.synthetic import init_policy, paligemma_3b_config
    cfg = paligemma_3b_config()
    cfg["vision_config"]["num_hidden_layers"] = 0
    V = cfg["text_config"]["vocab_size"]
    out = {"prefill": {}, "decode": {}}
    for B, T in PREFILLS:
        eng = Engine(cfg, device=dev, max_batch=B, max_seq=T, max_kv=T + 8)
        eng.fill_synthetic(seed, init_policy)
        eng.prepare()
        kv = eng.new_kv(B, T + 8)
        ids, pos = torch.randint(3, 200000, (B, T), device=dev), torch.arange(T)[None]
        ms = timed(lambda: eng.lm_forward(kv, 0, pos, ids=ids, logits_rows=2), max(3, steps // 20), 3)
        out["prefill"][f"{B}x{T}"] = {"ms": round(ms, 3), "tok_s": round(B * T / ms * 1e3, 1)}
        del eng, kv
    weight_bytes = None
    for B in BATCHES:
        cap = CONTEXT + steps + warmup + 8
        eng = Engine(cfg, device=dev, max_batch=B, max_seq=CONTEXT, max_kv=cap)
        eng.fill_synthetic(seed, init_policy)
        eng.prepare()
        weight_bytes = sum(v.numel() * 2 for n, v in eng.views.items() if n.startswith("language_model"))
        kv = eng.new_kv(B, cap)
        ids = torch.randint(3, 200000, (B, CONTEXT), device=dev)
        eng.lm_forward(kv, 0, torch.arange(CONTEXT)[None], ids=ids, logits_rows=2)
        cur, lg = ids[:, 0].contiguous(), torch.empty((B, V), device=dev)
        at = [CONTEXT]

        def step():
            eng.decode(cur, kv, at[0], at[0] + 1, logits=lg, next_ids=cur, graph=True)
            at[0] += 1

        ms = timed(step, steps, max(3, warmup))
        out["decode"][f"{B}x{CONTEXT}"] = decode_entry(ms, B, weight_bytes)
        del eng, kv
    out["params_bytes"] = weight_bytes
    return out


def run(a) -> None:
    dev = torch.device("cuda", 0)
    torch.cuda.set_device(dev)
    steps, warmup = min(a.steps, 128), a.warmup
    for size in a.decoder.split(","):
        raw, leg = decoder_leg(size, steps, warmup, a.seed, dev)
        one = leg["decode"][f"1x{CONTEXT}"]
        ffs = [x["mlp"] for x in raw["layers"] if x["mlp"]]
        line = {"metric": f"layered decoder ({raw['architecture']} {size}) greedy decode tokens/s, batch 1", "value": one["tok_s"],
                "unit": "tokens/s", "n_gpus": 1, "steps": steps, "warmup": warmup, "ms_per_step": one["ms_per_step"],
                "higher_is_better": True, "dtype": "bf16", "data": "synthetic (random weights, random token ids)",
                "config": {"width": raw["width"], "layers": [x["type"] for x in raw["layers"]], "vocab": raw["vocab"],
                           "mixers": {x["type"]: x["mixer"] for x in raw["layers"]}, "streams": raw.get("streams", 1),
                           "ff": ffs[0]["ff"] if ffs[0]["kind"] == "dense" else ffs[0]}, **leg}
        gc.collect()
        if size == "2b":
            line["paligemma_text"] = gemma_leg(steps, warmup, a.seed, dev)
            gc.collect()
        print(json.dumps(line), flush=True)
