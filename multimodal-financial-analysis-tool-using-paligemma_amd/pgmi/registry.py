"""Model registry: config.json -> the class that runs it.

A checkpoint's family is found by config.json's "architecture" (layered decoders), or it is a PaliGemma
checkpoint ("architectures" / "model_type", or the vision_config + text_config pair of older ones).
Layered decoders register a reader that turns their config.json into a DecoderConfig.
"""
from __future__ import annotations

import json
import os
from typing import Callable, Dict

from .decoder import ATTENTION, MAMBA1, MINGRU, DecoderConfig, DecoderEngine, DecoderLayer


def _need(d: dict, key: str, where: str):
    if not isinstance(d, dict) or key not in d or d[key] is None:
        raise ValueError(f"config.json: {where} has no '{key}'")
    return d[key]


def tuvodra_config(cfg: dict) -> DecoderConfig:
    """Tuvodra: mamba1, windowed attention and minGRU mixers in any order around hyper-connected streams."""
    layers = []
    for i, entry in enumerate(_need(cfg, "layers", "the model")):
        where = f"layer {i}"
        kind, m = _need(entry, "type", where), _need(entry, "mixer", where)
        if kind == "mamba1":
            layer = DecoderLayer(MAMBA1, **{k: int(_need(m, k, where)) for k in ("conv", "dt_rank", "inner", "state")})
        elif kind == "mingru":
            layer = DecoderLayer(MINGRU, width=int(_need(m, "width", where)))
        elif kind == "attention":
            layer = DecoderLayer(ATTENTION, **{k: int(_need(m, k, where)) for k in ("heads", "kv_heads", "dim", "vdim")},
                                 window=int(_need(_need(m, "mask", where), "size", where)),
                                 scale=float(_need(m, "scale", where)), qk_norm=1, proj_bias=1, distance_bias=1)
        else:
            raise ValueError(f"config.json: {where} has the unknown mixer '{kind}'")
        mlp = entry.get("mlp")
        if mlp is not None:
            if _need(mlp, "kind", where) != "dense":
                raise ValueError(f"config.json: {where} has the unknown feed-forward '{mlp['kind']}'")
            layer.ff = int(_need(mlp, "ff", where))
        layers.append(layer)
    norm = _need(cfg, "norm", "the model")
    return DecoderConfig(vocab=int(_need(cfg, "vocab", "the model")), width=int(_need(cfg, "width", "the model")),
                         streams=int(_need(cfg, "streams", "the model")), norm_groups=int(_need(norm, "groups", "norm")),
                         norm_eps=float(_need(norm, "eps", "norm")),
                         embed_scale=float(_need(_need(cfg, "embedding", "the model"), "scale", "embedding")), layers=layers)


def _moe(mlp: dict, where: str) -> dict:
    """The mixture-of-experts fields of a layer."""
    r = _need(mlp, "router", where)
    groups, shared = r.get("groups"), mlp.get("shared")
    return dict(experts=int(_need(r, "experts", where)), identity=int(r.get("identity") or 0), top=int(_need(r, "top", where)),
                groups=int(_need(groups, "count", where)) if groups else 1,
                groups_keep=int(_need(groups, "keep", where)) if groups else 1,
                expert_ff=int(_need(_need(mlp, "expert", where), "ff", where)),
                shared_ff=int(_need(shared, "ff", where)) if shared else 0)


def raritar_config(cfg: dict) -> DecoderConfig:
    """Raritar: windowed attention with kept first tokens, rotary positions, capped scores and shared keys / values, and a
    mixture of experts, around one residual stream with an input convolution and a bigram embedding."""
    layers = []
    for i, entry in enumerate(_need(cfg, "layers", "the model")):
        where = f"layer {i}"
        kind, m = _need(entry, "type", where), _need(entry, "mixer", where)
        if kind != "attention":
            raise ValueError(f"config.json: {where} has the unknown mixer '{kind}'")
        mask, rot, kv = _need(m, "mask", where), _need(m, "rot", where), m.get("kv_from")
        layer = DecoderLayer(ATTENTION, **{k: int(_need(m, k, where)) for k in ("heads", "kv_heads", "dim", "vdim")},
                             window=int(_need(mask, "size", where)), keep_first=int(mask.get("keep_first") or 0),
                             scale=float(_need(m, "scale", where)), softcap=float(m.get("softcap") or 0.0), v_norm=1,
                             kv_from=-1 if kv is None else int(kv), rot_dims=int(_need(rot, "dims", where)),
                             rot_base=float(_need(rot, "base", where)))
        scaling = rot.get("scaling")
        if scaling:
            for k in ("factor", "low", "high", "original"):
                setattr(layer, "rot_" + k, float(_need(scaling, k, where)))
        mlp = entry.get("mlp")
        if mlp is not None:
            if _need(mlp, "kind", where) != "moe":
                raise ValueError(f"config.json: {where} has the unknown feed-forward '{mlp['kind']}'")
            for k, v in _moe(mlp, where).items():
                setattr(layer, k, v)
        layers.append(layer)
    pairs = _need(_need(cfg, "embedding", "the model"), "bigram", "embedding")
    buckets = int(_need(pairs, "buckets", "bigram"))
    if buckets < 1:
        raise ValueError("config.json: bigram needs at least one bucket")
    return DecoderConfig(vocab=int(_need(cfg, "vocab", "the model")), width=int(_need(cfg, "width", "the model")), streams=1,
                         norm_groups=1, norm_eps=float(_need(_need(cfg, "norm", "the model"), "eps", "norm")), embed_scale=1.0,
                         layers=layers, plain_residual=True, residual_mult=float(_need(cfg, "residual_mult", "the model")),
                         norm_scalar=True, canon_taps=int(_need(_need(cfg, "canon", "the model"), "taps", "canon")),
                         bigram_buckets=buckets, untied_head=True,
                         # only the row modulo the buckets matters: reduced factors cannot overflow 64 bits
                         bigram_mul_prev=int(_need(pairs, "mul_prev", "bigram")) % buckets,
                         bigram_mul_cur=int(_need(pairs, "mul_cur", "bigram")) % buckets)


DECODERS: Dict[str, Callable[[dict], DecoderConfig]] = {"Tuvodra": tuvodra_config, "Raritar": raritar_config}


def read_config(model_path: str) -> dict:
    with open(os.path.join(model_path, "config.json")) as f:
        return json.load(f)


def family(cfg: dict) -> str:
    """"decoder" or "paligemma"; ValueError for a config.json that is neither."""
    name = cfg.get("architecture")
    if name is not None:
        if name not in DECODERS:
            raise ValueError(f"unknown architecture '{name}' (known: {', '.join(sorted(DECODERS))})")
        return "decoder"
    if ("vision_config" in cfg and "text_config" in cfg) or cfg.get("model_type") == "paligemma":
        return "paligemma"
    raise ValueError("config.json names no architecture this library runs")


def decoder_config(cfg: dict) -> DecoderConfig:
    if family(cfg) != "decoder":
        raise ValueError("config.json is not a layered decoder's")
    return DECODERS[cfg["architecture"]](cfg)


def load_decoder(model_path: str, device=None, dtype: str = "bfloat16", max_batch: int = 64) -> DecoderEngine:
    """config.json + *.safetensors -> a prepared DecoderEngine."""
    eng = DecoderEngine(decoder_config(read_config(model_path)), device=device, dtype=dtype, max_batch=max_batch)
    eng.load_safetensors(model_path)
    eng.prepare()
    return eng
