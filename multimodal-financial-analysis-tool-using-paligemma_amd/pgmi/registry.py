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
                                 scale=float(_need(m, "scale", where)))
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


DECODERS: Dict[str, Callable[[dict], DecoderConfig]] = {"Tuvodra": tuvodra_config}


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
