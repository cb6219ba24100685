"""Small Raritar models for the tests: every size differs from its neighbours, many are no multiple of 8."""


def moe(experts, ff, top, shared, identity=0, groups=(1, 1)):
    return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared},
            "router": {"experts": experts, "identity": identity, "top": top,
                       "groups": {"count": groups[0], "keep": groups[1]}}}


def layer(heads, kv_heads, dim, vdim, size, keep=0, rot=None, base=10000.0, scaling=None, scale=None, cap=30.0, kv_from=None,
          mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size, "keep_first": keep},
         "scale": dim ** -0.5 if scale is None else scale, "softcap": cap,
         "rot": {"base": base, "dims": dim if rot is None else rot}}
    if scaling is not None:
        m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


def model(layers, width=72, vocab=203, taps=4, buckets=67, mul=(5, 3), mult=0.6, eps=2e-5):
    return {"architecture": "Raritar", "vocab": vocab, "width": width, "canon": {"taps": taps}, "norm": {"eps": eps},
            "embedding": {"bigram": {"buckets": buckets, "mul_prev": mul[0], "mul_cur": mul[1]}}, "residual_mult": mult,
            "layers": layers}


# one mechanism each, sizes off every boundary
MECHANISMS = {
    "heads_gqa": model([layer(4, 2, 24, 40, 17, keep=3, rot=8)]),
    "heads_mha": model([layer(3, 3, 20, 28, 33, keep=5, rot=20)], width=60, taps=3),
    "heads_12_of_1": model([layer(12, 1, 64, 56, 9, keep=2, rot=32)], width=64),
    "heads_20_of_1": model([layer(20, 1, 16, 24, 40, keep=1, rot=6)], width=56),
    "heads_wide": model([layer(2, 2, 130, 72, 64, keep=7, rot=66)], width=96),
    "heads_96_128": model([layer(5, 1, 96, 128, 70, keep=65, rot=48)], width=100),
    "heads_plain_form": model([layer(2, 1, 264, 300, 21, keep=4, rot=100)], width=64),
    "heads_odd": model([layer(4, 2, 18, 22, 25, keep=6, rot=10)], width=61, vocab=101),
    "rotation_scaled": model([layer(4, 2, 32, 24, 200, rot=32, base=500.0, scaling=(3.0, 1.5, 6.0, 96))], width=80),
    "rotation_none_kept": model([layer(4, 1, 40, 40, 60, rot=2, base=50.0, scaling=(8.0, 1.0, 2.0, 5))]),
    "window_1": model([layer(3, 3, 16, 16, 1)], width=48),
    "window_1_kept": model([layer(3, 1, 16, 16, 1, keep=9)], width=48),
    "kept_more_than_window": model([layer(4, 2, 32, 32, 11, keep=90)]),
    "cap_low": model([layer(4, 2, 32, 48, 80, keep=2, cap=1.5, scale=0.8)]),
    "cap_high": model([layer(4, 2, 32, 48, 80, keep=2, cap=300.0, scale=0.5)]),
    "cap_none": model([layer(4, 2, 32, 48, 80, keep=2, cap=None, scale=0.4)]),
    "taps_1": model([layer(2, 1, 16, 24, 30)], taps=1),
    "taps_2": model([layer(2, 1, 16, 24, 30)], taps=2, width=68),
    "taps_7": model([layer(2, 1, 16, 24, 30)], taps=7),
    "taps_odd_width": model([layer(2, 1, 16, 24, 30)], taps=5, width=59),
    "pairs": model([layer(2, 1, 16, 16, 12)], buckets=1009, mul=(2 ** 31 - 1, 999983), mult=1.0),
    "pairs_one_bucket": model([layer(2, 1, 16, 16, 12)], buckets=1),
    "wide_row": model([layer(2, 1, 16, 16, 12)], width=4100, vocab=67),
    "wide_odd_row": model([layer(2, 1, 16, 16, 12)], width=1027, vocab=67),
    "shared_kv": model([layer(4, 2, 24, 40, 30, keep=4, rot=8), layer(4, 2, 24, 40, 9, keep=1, rot=8, cap=9.0, kv_from=0),
                        layer(6, 3, 16, 8, 50, rot=16), layer(6, 3, 16, 8, 50, keep=12, rot=16, kv_from=2),
                        layer(4, 2, 24, 40, 64, rot=8, scale=0.4, kv_from=0)]),
    "experts_top1": model([layer(2, 1, 16, 24, 30, mlp=moe(3, 20, 1, 28))]),
    "experts_few": model([layer(2, 1, 16, 24, 30, mlp=moe(4, 36, 2, 12))]),
    "experts_identity": model([layer(2, 1, 16, 24, 30, mlp=moe(6, 24, 4, 40, identity=3))], mult=0.35),
    "experts_grouped": model([layer(2, 1, 16, 24, 30, mlp=moe(13, 31, 3, 17, identity=2, groups=(5, 2)))]),
    "experts_many": model([layer(2, 1, 16, 24, 30, mlp=moe(70, 16, 5, 24, identity=10, groups=(8, 3)))], width=88),
    "experts_odd_width": model([layer(2, 1, 16, 24, 30, mlp=moe(5, 7, 2, 5, identity=1, groups=(2, 1)))], width=61),
    "experts_all": model([layer(2, 1, 16, 24, 30, mlp=moe(4, 9, 6, 33, identity=2))]),
}

MIXED = {
    "a": model([layer(6, 3, 24, 36, 40, keep=5, rot=12, mlp=moe(7, 44, 3, 52, identity=1, groups=(4, 2))),
                layer(6, 3, 24, 36, 23, keep=2, rot=12, cap=12.0, kv_from=0),
                layer(4, 1, 48, 16, 75, keep=30, base=3000.0, scaling=(4.0, 1.0, 4.0, 120), mlp=moe(5, 28, 2, 20)),
                layer(6, 3, 24, 36, 64, rot=12, kv_from=0, mlp=moe(9, 21, 4, 35, identity=3, groups=(3, 2)))],
               width=84, vocab=211),
    "b": model([layer(8, 2, 32, 32, 130, keep=10, rot=16), layer(2, 1, 72, 64, 11, keep=1, mlp=moe(8, 40, 2, 64)),
                layer(8, 2, 32, 32, 50, keep=70, rot=16, kv_from=0, mlp=moe(10, 24, 3, 16, identity=2, groups=(2, 1)))],
               width=128, vocab=160, taps=3, mult=0.8, eps=1e-6, buckets=301, mul=(17, 11)),
}
