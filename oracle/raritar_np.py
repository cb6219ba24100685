"""oracle/raritar_np.py -- TEST INFRASTRUCTURE ONLY (never the product).

Plain, slow restatement (numpy, float64) of Raritar, one function per mechanism, token by token, sharing no code with
the product: one residual stream with a scaled update, one-number RMS norms, a short causal convolution added to what
a mixer reads, a bigram embedding, attention over a sliding window with kept first tokens (interleaved rotation with
scaled frequencies, normed values, capped scores, keys and values shared between layers), and a group-limited mixture
of experts with identity experts and a gated shared expert.
"""
from __future__ import annotations

import numpy as np

from oracle.decoder_np import F, Weights, gated_mlp, sigmoid, unit_rms


# ---------------------------------------------------------------- embedding, norm, convolution
def bigram_row(prev, cur, m):
    """Row of the bigram table; prev is None at a sequence's start."""
    return m["buckets"] if prev is None else (int(prev) * m["mul_prev"] + int(cur) * m["mul_cur"]) % m["buckets"]


def scalar_rms_norm(x, g, eps):
    return unit_rms(x, eps) * float(g)


def canon(earlier, h, w):
    """earlier [taps - 1, D], oldest first (updated in place): h plus the convolution of the last taps inputs."""
    window = np.concatenate([earlier, h[None]], 0)
    if len(earlier):
        earlier[:] = window[1:]
    return h + np.einsum("kd,dk->d", window, w)


# ---------------------------------------------------------------- attention
def rotary_frequencies(rot):
    """Angle per position of every rotated pair, after the wavelength-dependent scaling."""
    out = []
    for i in range(rot["dims"] // 2):
        f = float(rot["base"]) ** (-2.0 * i / rot["dims"])
        sc = rot.get("scaling")
        if sc:
            turn = 2.0 * np.pi / f
            if turn > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif turn >= sc["original"] / sc["high"]:
                s = (sc["original"] / turn - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return np.array(out, F)


def rotate(x, pos, rot):
    """x [heads, dim]: pairs (2i, 2i + 1) of the first rot.dims dimensions turned by pos * frequency i."""
    y = x.copy()
    a = pos * rotary_frequencies(rot)
    c, s = np.cos(a), np.sin(a)
    u, v = x[:, 0:rot["dims"]:2], x[:, 1:rot["dims"]:2]
    y[:, 0:rot["dims"]:2] = u * c - v * s
    y[:, 1:rot["dims"]:2] = v * c + u * s
    return y


def visible(i, mask):
    """Positions the query at i sees: the window's, and the first keep_first tokens."""
    j = np.arange(i + 1)
    return j[(i - j < mask["size"]) | (j < mask["keep_first"])]


def capped(s, cap):
    return cap * np.tanh(s / cap) if cap else s


def attend(q, k, v, scale, cap):
    """q [H, d], k [n, G, d], v [n, G, e] -> [H, e]."""
    H, G = q.shape[0], k.shape[1]
    out = np.zeros((H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = capped(k[:, g] @ q[h] * scale, cap)
        e = np.exp(s - s.max())
        out[h] = (e / e.sum()) @ v[:, g]
    return out


def attention(W, p, m, eps, state, i_layer, pos, h):
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate((W[p + "q"] @ h).reshape(H, d), pos, m["rot"])
    src = m.get("kv_from")
    if src is None:
        src = i_layer
        state[i_layer]["k"].append(rotate((W[p + "k"] @ h).reshape(G, d), pos, m["rot"]))
        state[i_layer]["v"].append(unit_rms((W[p + "v"] @ h).reshape(G, e), eps))
    js = visible(pos, m["mask"])
    o = attend(q, np.stack([state[src]["k"][j] for j in js]), np.stack([state[src]["v"][j] for j in js]), m["scale"],
               m["softcap"])
    return W[p + "o"] @ o.reshape(-1)


# ---------------------------------------------------------------- mixture of experts
def route(z, correction, r):
    """[(expert, weight)] of the chosen experts."""
    s = np.exp(z - z.max())
    s = s / s.sum()
    choice = s + correction
    n = r["groups"]["count"]
    best = choice.reshape(n, -1).max(1)
    kept = np.argsort(-best, kind="stable")[:r["groups"]["keep"]]
    allowed = np.full(choice.shape, -np.inf).reshape(n, -1)
    allowed[kept] = choice.reshape(n, -1)[kept]
    chosen = np.argsort(-allowed.reshape(-1), kind="stable")[:r["top"]]
    return [(int(e), s[e]) for e in chosen]


def experts(W, p, mlp, h):
    r = mlp["router"]
    y = np.zeros_like(h)
    for e, w in route(W[p + "router"] @ h, W[p + "correction"], r):
        y = y + w * (gated_mlp(W, p + f"e{e}.", h) if e < r["experts"] else h)
    return y + sigmoid(W[p + "shared.sg"] @ h)[0] * gated_mlp(W, p + "shared.", h)


# ---------------------------------------------------------------- the whole design
def new_state(cfg):
    return {"tokens": [], "layers": [{"k": [], "v": [], "conv": np.zeros((cfg["canon"]["taps"] - 1, cfg["width"]))}
                                     for _ in cfg["layers"]]}


def token_step(cfg, W, state, token, taps=None):
    """One token: logits [vocab]; taps (a list) receives the residual stream after every layer."""
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    pos = len(state["tokens"])
    prev = state["tokens"][-1] if pos else None
    state["tokens"].append(int(token))
    x = W["embed"][token] + W["bigram"][bigram_row(prev, token, cfg["embedding"]["bigram"])]
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = scalar_rms_norm(x, W[p + "norm1"], eps)
        h = canon(state["layers"][i]["conv"], h, W[p + "canon1"])
        x = x + mult * attention(W, p + "mix.", layer["mixer"], eps, state["layers"], i, pos, h)
        if layer["mlp"] is not None:
            x = x + mult * experts(W, p + "mlp.", layer["mlp"], scalar_rms_norm(x, W[p + "norm2"], eps))
        if taps is not None:
            taps.append(x)
    return W["head"] @ scalar_rms_norm(x, W["final.norm"], eps)


def run(cfg, W, tokens, state=None, taps=None):
    """Logits [len(tokens), vocab] of one sequence (state: continue from it)."""
    W = W if isinstance(W, Weights) else Weights(W)
    state = new_state(cfg) if state is None else state
    out = []
    for t in tokens:
        per = None if taps is None else []
        out.append(token_step(cfg, W, state, int(t), per))
        if taps is not None:
            taps.append(np.stack(per))
    return np.stack(out)


def greedy(cfg, W, tokens, n):
    """n greedily picked tokens after the prompt, and the logits each was picked from."""
    W = Weights(W)
    state = new_state(cfg)
    lg = run(cfg, W, tokens, state)[-1]
    toks, logits = [], []
    for _ in range(n):
        toks.append(int(lg.argmax()))
        logits.append(lg)
        if len(toks) < n:
            lg = token_step(cfg, W, state, toks[-1])
    return toks, np.stack(logits)


# ---------------------------------------------------------------- random models for the tests
def tensor_shapes(cfg):
    D, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, D), "bigram": (cfg["embedding"]["bigram"]["buckets"] + 1, D), "final.norm": (), "head": (V, D)}
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        out[p + "norm1"] = ()
        out[p + "canon1"] = (D, cfg["canon"]["taps"])
        out[p + "mix.q"] = (m["heads"] * m["dim"], D)
        if m.get("kv_from") is None:
            out[p + "mix.k"], out[p + "mix.v"] = (m["kv_heads"] * m["dim"], D), (m["kv_heads"] * m["vdim"], D)
        out[p + "mix.o"] = (D, m["heads"] * m["vdim"])
        if mlp is None:
            continue
        out[p + "norm2"] = ()
        r = mlp["router"]
        n = r["experts"] + r["identity"]
        parts = [(f"e{e}.", mlp["expert"]["ff"]) for e in range(r["experts"])] + [("shared.", mlp["shared"]["ff"])]
        for name, ff in parts:
            out.update({p + "mlp." + name + "gate": (ff, D), p + "mlp." + name + "up": (ff, D),
                        p + "mlp." + name + "down": (D, ff)})
        out.update({p + "mlp.router": (n, D), p + "mlp.correction": (n,), p + "mlp.shared.sg": (1, D)})
    return out


def bf16(w):
    u = np.ascontiguousarray(w, np.float32).view(np.uint32)
    u = (u + np.uint32(0x7FFF) + ((u >> np.uint32(16)) & np.uint32(1))) & np.uint32(0xFFFF0000)
    return u.view(np.float32).reshape(np.shape(w))


def route_margin(z, correction, r):
    """How far the nearest other choice of experts is: the smallest gap between a choice score that is taken (of the
    groups, then of the experts in them) and one that is left."""
    s = np.exp(z - z.max())
    choice = (s / s.sum() + correction).reshape(r["groups"]["count"], -1)
    best = np.sort(choice.max(1))[::-1]
    keep, top = r["groups"]["keep"], r["top"]
    gap = best[keep - 1] - best[keep] if keep < len(best) else np.inf
    kept = choice[np.argsort(-choice.max(1), kind="stable")[:keep]].reshape(-1)
    kept = np.sort(kept)[::-1]
    return min(gap, kept[top - 1] - kept[top] if top < len(kept) else np.inf)


KINDS = 5


def random_weights(cfg, seed):
    """float32 arrays holding bf16 values; scales chosen so that every mechanism moves the logits.  The last coordinates
    of the stream hold one of KINDS patterns by token, which no layer changes and which alone the routers read: a choice
    of experts is never a close call that rounding could turn."""
    rng = np.random.default_rng(seed)
    D, W = cfg["width"], {}
    T = max(KINDS, D // 6)
    patterns = np.sign(rng.standard_normal((KINDS, T))) * 2.0
    for n, shp in tensor_shapes(cfg).items():
        r = rng.standard_normal(shp)
        leaf = n.split(".", 1)[1] if n[0] == "l" else n
        if leaf in ("embed", "bigram"):
            w = r
            w[:, D - T:] = patterns[np.arange(shp[0]) % KINDS] if leaf == "embed" else 0.0
        elif "norm" in leaf:
            w = rng.uniform(0.85, 1.15, shp) if leaf == "norm2" else 1.0 + 0.2 * r
        elif leaf == "canon1":
            w = r * 0.4
        elif leaf == "mlp.correction":
            continue  # with the router
        elif leaf == "mlp.router":
            m = cfg["layers"][int(n[1:n.index(".")])]["mlp"]["router"]
            for _ in range(20000):
                w = np.zeros(shp)
                w[:, D - T:] = bf16(rng.standard_normal((shp[0], T)) * (1.2 / np.sqrt(T)))
                c = bf16(rng.standard_normal(shp[0]) * 0.2 - 0.2)
                # the norm divides the patterns by anything from 1.2 to 4.2, say: the choice is the same for all of it
                zs = [[w[:, D - T:] @ p / d for d in np.geomspace(1.2, 4.2, 9)] for p in patterns]
                sets = [{frozenset(e for e, _ in route(z, c, m)) for z in per} for per in zs]
                if all(len(x) == 1 for x in sets) and (len(set.union(*sets)) > 2 or m["top"] == shp[0]) and \
                        all(route_margin(z, c, m) > 0.003 for per in zs for z in per):
                    break
            else:
                raise ValueError("no router with a margin found")
            W[n.replace("router", "correction")] = c
        elif leaf.endswith("down") or leaf == "mix.o":
            w = r * ((2.5 if leaf.endswith("down") else 1.5) / np.sqrt(shp[-1]))
            w[D - T:] = 0.0
        else:
            w = r * (1.3 / np.sqrt(shp[-1]))
        W[n] = bf16(w)
    return W
