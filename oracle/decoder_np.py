"""oracle/decoder_np.py -- TEST INFRASTRUCTURE ONLY (checker side, never the product).

Plain, slow restatement (numpy, float64) of the layered decoder designs that libpgmi's decoder engine
runs (today: Tuvodra), one function per mechanism, written from the designs' equations.  It works
token by token where a mechanism carries a state, shares no code with the product and has no fast
path.  Weights are a dict name -> array under the checkpoint's tensor names.

A sequence's state is a plain list, one entry per layer, made by new_state() and updated in place.
"""
from __future__ import annotations

import numpy as np

F = np.float64


# ---------------------------------------------------------------- elementary functions
def sigmoid(x):
    x = np.asarray(x, F)
    e = np.exp(-np.abs(x))
    return np.where(x >= 0, 1.0 / (1.0 + e), e / (1.0 + e))


def silu(x):
    return np.asarray(x, F) * sigmoid(x)


def softplus(x):
    x = np.asarray(x, F)
    return np.maximum(x, 0.0) + np.log1p(np.exp(-np.abs(x)))


# ---------------------------------------------------------------- norms
def group_rms_norm(x, w, groups, eps):
    """x [..., D] in `groups` equal consecutive parts, each over its own root mean square; times w."""
    x = np.asarray(x, F)
    parts = x.reshape(x.shape[:-1] + (groups, x.shape[-1] // groups))
    y = parts / np.sqrt(np.mean(parts * parts, axis=-1, keepdims=True) + eps)
    return y.reshape(x.shape) * np.asarray(w, F)


def unit_rms(x, eps):
    """x over its root mean square along the last axis (no weight)."""
    x = np.asarray(x, F)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


# ---------------------------------------------------------------- hyper-connections
def streams_read(X, w_in):
    """X [S, D] -> the sublayer's input: sum over the streams of w_in[s] X[s]."""
    return np.einsum("s,sd->d", np.asarray(w_in, F), X)


def streams_write(X, y, mix, w_out):
    """New streams: X'[t] = sum_s mix[s, t] X[s] + w_out[t] y."""
    return np.einsum("st,sd->td", np.asarray(mix, F), X) + np.asarray(w_out, F)[:, None] * y[None, :]


# ---------------------------------------------------------------- selective scan
def causal_conv_step(taps, x, w, b):
    """One token of a per-channel causal convolution + silu.  taps [K-1, C]: the earlier inputs, oldest
    first (updated in place); w [C, K], its last column the current token's."""
    K = w.shape[1]
    window = np.concatenate([taps, x[None]], 0)
    y = np.einsum("kc,ck->c", window, np.asarray(w, F)) + np.asarray(b, F)
    if K > 1:
        taps[:] = window[1:]
    return silu(y)


def selective_scan_step(S, x, dt, A, B, C, D):
    """S [C, N] in place: S <- exp(dt A) S + dt x B; returns y [C] = S C + D x."""
    S[:] = np.exp(dt[:, None] * A) * S + (dt * x)[:, None] * B[None, :]
    return S @ C + D * x


def mamba_step(W, p, m, st, h):
    inner, R, N = m["inner"], m["dt_rank"], m["state"]
    xz = W[p + "in"] @ h
    x, z = xz[:inner], xz[inner:]
    x = causal_conv_step(st["taps"], x, W[p + "conv"], W[p + "conv.b"])
    q = W[p + "x"] @ x
    dt = softplus(W[p + "dt"] @ q[:R] + W[p + "dt.b"])
    y = selective_scan_step(st["S"], x, dt, -np.exp(W[p + "A_log"]), q[R:R + N], q[R + N:], W[p + "D"])
    return W[p + "o"] @ (y * silu(z))


# ---------------------------------------------------------------- minimal gated recurrence
def mingru_candidate(u):
    return np.where(u >= 0, u + 0.5, sigmoid(u))


def mingru_step(W, p, m, st, h):
    z = sigmoid(W[p + "z"] @ h + W[p + "z.b"])
    u = W[p + "x"] @ h + W[p + "x.b"]
    st["S"][:] = (1.0 - z) * st["S"] + z * mingru_candidate(u)
    return W[p + "o"] @ (st["S"] * silu(W[p + "g"] @ h))


# ---------------------------------------------------------------- windowed attention with a distance bias
def distance_bias(r1, r2, dist):
    """[heads, keys]: what a head takes off its scores, r1 ln(1 + r2 distance)."""
    return np.asarray(r1, F)[:, None] * np.log1p(np.asarray(r2, F)[:, None] * np.asarray(dist, F)[None, :])


def window_keys(i, size):
    """Positions the query at i sees: itself and the size - 1 before it."""
    return np.arange(max(0, i - size + 1), i + 1)


def attention_scores_out(q, k, v, scale, bias):
    """q [H, d], k [n, G, d], v [n, G, e], bias [H, n] -> [H, e] (query head h reads group h // (H/G))."""
    H, G = q.shape[0], k.shape[1]
    out = np.zeros((H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = k[:, g] @ q[h] * scale - bias[h]
        e = np.exp(s - s.max())
        out[h] = (e / e.sum()) @ v[:, g]
    return out


def attention_step(W, p, m, eps, st, h):
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit_rms((W[p + "q"] @ h + W[p + "q.b"]).reshape(H, d), eps)
    k = unit_rms((W[p + "k"] @ h + W[p + "k.b"]).reshape(G, d), eps)
    v = (W[p + "v"] @ h + W[p + "v.b"]).reshape(G, e)
    i = len(st["k"])
    st["k"].append(k)
    st["v"].append(v)
    js = window_keys(i, m["mask"]["size"])
    bias = distance_bias(W[p + "r1"], W[p + "r2"], i - js)
    o = attention_scores_out(q, np.stack([st["k"][j] for j in js]), np.stack([st["v"][j] for j in js]), m["scale"], bias)
    return W[p + "o"] @ o.reshape(-1)


# ---------------------------------------------------------------- feed-forward
def gated_mlp(W, p, h):
    return W[p + "down"] @ (silu(W[p + "gate"] @ h) * (W[p + "up"] @ h))


# ---------------------------------------------------------------- the whole design
def new_state(cfg):
    out = []
    for layer in cfg["layers"]:
        m = layer["mixer"]
        if layer["type"] == "mamba1":
            out.append({"taps": np.zeros((m["conv"] - 1, m["inner"])), "S": np.zeros((m["inner"], m["state"]))})
        elif layer["type"] == "mingru":
            out.append({"S": np.zeros(m["width"])})
        elif layer["type"] == "attention":
            out.append({"k": [], "v": []})
        else:
            raise ValueError(layer["type"])
    return out


def mixer_step(cfg, W, i, st, h):
    layer, p = cfg["layers"][i], f"l{i}.mix."
    if layer["type"] == "mamba1":
        return mamba_step(W, p, layer["mixer"], st, h)
    if layer["type"] == "mingru":
        return mingru_step(W, p, layer["mixer"], st, h)
    return attention_step(W, p, layer["mixer"], cfg["norm"]["eps"], st, h)


def token_step(cfg, W, state, token, taps=None):
    """One token through the model: logits [vocab]; taps (a list) receives the summed streams after every layer."""
    groups, eps = cfg["norm"]["groups"], cfg["norm"]["eps"]
    x = W["embed"][token] * cfg["embedding"]["scale"]
    X = np.repeat(x[None], cfg["streams"], 0)
    for i, layer in enumerate(cfg["layers"]):
        lp = f"l{i}."
        h = group_rms_norm(streams_read(X, W[lp + "hc1.in"]), W[lp + "norm1"], groups, eps)
        X = streams_write(X, mixer_step(cfg, W, i, state[i], h), W[lp + "hc1.mix"], W[lp + "hc1.out"])
        if layer["mlp"] is not None:
            h = group_rms_norm(streams_read(X, W[lp + "hc2.in"]), W[lp + "norm2"], groups, eps)
            X = streams_write(X, gated_mlp(W, lp + "mlp.", h), W[lp + "hc2.mix"], W[lp + "hc2.out"])
        if taps is not None:
            taps.append(X.sum(0))
    return W["embed"] @ group_rms_norm(X.sum(0), W["final.norm"], groups, eps)


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


class Weights(dict):
    """name -> float64 array."""

    def __init__(self, src):
        super().__init__((k, np.asarray(v, F)) for k, v in src.items())


# ---------------------------------------------------------------- random models for the tests
def tensor_shapes(cfg):
    D, V, S = cfg["width"], cfg["vocab"], cfg["streams"]
    out = {"embed": (V, D), "final.norm": (D,)}
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        subs = [1] + ([2] if layer["mlp"] is not None else [])
        for q in subs:
            out[p + f"norm{q}"] = (D,)
            out[p + f"hc{q}.in"], out[p + f"hc{q}.out"], out[p + f"hc{q}.mix"] = (S,), (S,), (S, S)
        x = p + "mix."
        if layer["type"] == "mamba1":
            C, N, R = m["inner"], m["state"], m["dt_rank"]
            out.update({x + "in": (2 * C, D), x + "conv": (C, m["conv"]), x + "conv.b": (C,), x + "x": (R + 2 * N, C),
                        x + "dt": (C, R), x + "dt.b": (C,), x + "A_log": (C, N), x + "D": (C,), x + "o": (D, C)})
        elif layer["type"] == "mingru":
            C = m["width"]
            out.update({x + "z": (C, D), x + "z.b": (C,), x + "x": (C, D), x + "x.b": (C,), x + "g": (C, D), x + "o": (D, C)})
        else:
            H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            out.update({x + "q": (H * d, D), x + "q.b": (H * d,), x + "k": (G * d, D), x + "k.b": (G * d,),
                        x + "v": (G * e, D), x + "v.b": (G * e,), x + "r1": (H,), x + "r2": (H,), x + "o": (D, H * e)})
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            out.update({p + "mlp.gate": (ff, D), p + "mlp.up": (ff, D), p + "mlp.down": (D, ff)})
    return out


def random_weights(cfg, seed):
    """float32 arrays holding bf16 values; scales chosen so that every mechanism moves the logits."""
    rng = np.random.default_rng(seed)
    W = {}
    for n, shp in tensor_shapes(cfg).items():
        r = rng.standard_normal(shp)
        leaf = n.split(".", 1)[1] if n.startswith("l") else n
        if n == "embed":
            w = r * 0.5
        elif "norm" in leaf:
            w = 1.0 + 0.2 * r
        elif leaf.endswith(".in") and leaf.startswith("hc"):
            w = 1.0 / shp[0] + 0.2 * r
        elif leaf.startswith("hc") and leaf.endswith(".out"):
            w = 1.0 + 0.3 * r
        elif leaf.startswith("hc") and leaf.endswith(".mix"):
            w = 0.8 * np.eye(shp[0]) + 0.15 * r
        elif leaf == "mix.A_log":
            w = rng.uniform(-2.0, 1.2, shp)
        elif leaf == "mix.dt.b":
            w = rng.uniform(-4.5, -0.5, shp)
        elif leaf == "mix.D":
            w = 1.0 + 0.3 * r
        elif leaf == "mix.conv":
            w = r * 0.5
        elif leaf == "mix.r1":
            w = rng.uniform(0.1, 1.0, shp)
        elif leaf == "mix.r2":
            w = rng.uniform(0.05, 1.5, shp)
        elif leaf == "mix.z.b":
            w = rng.uniform(-4.0, 0.5, shp)
        elif leaf.endswith(".b"):
            w = 0.3 * r
        elif leaf in ("mix.o", "mlp.down"):
            w = r * (0.8 / np.sqrt(shp[-1]))
        else:
            w = r * (1.1 / np.sqrt(shp[-1]))
        u = np.ascontiguousarray(w, np.float32).view(np.uint32)
        u = (u + np.uint32(0x7FFF) + ((u >> np.uint32(16)) & np.uint32(1))) & np.uint32(0xFFFF0000)
        W[n] = u.view(np.float32).reshape(shp)
    return W
