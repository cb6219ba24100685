"""Small layered-decoder models for the tests: every size differs from its neighbours, many are no multiple of 8."""


def mamba(inner, state, dt_rank, conv, ff=None):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def attn(heads, kv_heads, dim, vdim, size, scale=None, ff=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                           "scale": dim ** -0.5 if scale is None else scale, "mask": {"size": size}},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def gru(width, ff=None):
    return {"type": "mingru", "mixer": {"width": width}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def model(layers, width=88, vocab=203, streams=3, groups=4, eps=3e-5, escale=2.5):
    return {"architecture": "Tuvodra", "vocab": vocab, "width": width, "streams": streams,
            "norm": {"groups": groups, "eps": eps}, "embedding": {"scale": escale}, "layers": layers}


# one mechanism each (one or two layers), sizes off every boundary
MECHANISMS = {
    "mamba_small": model([mamba(36, 3, 5, 2)], width=60, streams=1, groups=1),
    "mamba_conv1": model([mamba(40, 16, 1, 1)], width=72, streams=2, groups=3),
    "mamba_wide_state": model([mamba(52, 130, 12, 7)], width=64, streams=4, groups=8, vocab=97),
    "mamba_20": model([mamba(104, 20, 8, 4, ff=44)], width=80, streams=2, groups=5),
    "gru": model([gru(50)], width=56, streams=2, groups=7),
    "gru_mlp": model([gru(136, ff=61)], width=104, streams=3, groups=2),
    "attn_mha": model([attn(4, 4, 20, 28, 17)], width=60, streams=2, groups=3),
    "attn_gqa3": model([attn(6, 2, 64, 40, 33, ff=72)], width=96, streams=2, groups=4),
    "attn_mqa": model([attn(5, 1, 96, 128, 70)], width=100, streams=1, groups=5),
    "attn_gqa12": model([attn(12, 1, 32, 56, 9)], width=64, streams=5, groups=2),
    "attn_wide": model([attn(2, 2, 130, 72, 64)], width=120, streams=2, groups=6),
    "attn_plain_form": model([attn(2, 1, 264, 300, 21)], width=64, streams=2, groups=2),
    "attn_window1": model([attn(3, 3, 16, 16, 1)], width=48, streams=2, groups=2),
}

# all mixers, two orders, equal sizes avoided
MIXED = {
    "a": model([mamba(72, 12, 6, 3), gru(44), attn(6, 3, 24, 36, 40, ff=100), mamba(40, 9, 3, 5, ff=28), gru(68),
                attn(4, 1, 48, 16, 75)], width=84, streams=2, groups=3, vocab=211),
    "b": model([attn(8, 2, 32, 32, 130), attn(2, 1, 72, 64, 11, ff=90), gru(96, ff=64), mamba(128, 16, 8, 4)],
               width=128, streams=4, groups=8, vocab=160, eps=1e-6, escale=7.0),
}
