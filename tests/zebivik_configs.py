"""Small Zebivik configurations (config.json dictionaries) for the tests.  They differ from each other in every size: attention
heads alone and in groups, keys above and below values, heads turned whole, in part and not at all, with and without slowed
frequencies, linear-attention heads of 3 to 150 channels under decays from 0 to 1, recurrent blocks wider and narrower than the
model, in one block and in many (of one channel too), behind one to seven taps, dense and mixed feed-forwards, layers without one,
one to eight groups of experts (of one expert and of more) with some or all kept, top from one to all, with and without a shared
expert, with and without a cap on the logits, scales on either side of one."""
import copy


def attention(heads, kv_heads, dim, vdim, scale, dims=None, base=10000.0, scaling=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if dims != 0:
        m["rot"] = {"dims": dim if dims is None else dims, "base": base}
        if scaling is not None:
            m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return m


def lightning(dim, vdim, *decay):
    return {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}


def side(left, right, left_scale=1.0, right_scale=1.0):
    return {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}


def rglru(width, blocks, conv):
    return {"width": width, "blocks": blocks, "conv": conv}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, top, ff, scale=1.0, groups=None, shared=None):
    router = {"experts": experts, "top": top, "scale": scale}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    out = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def layer(mixer, mlp):
    return {"type": "rglru" if "blocks" in mixer else "parallel", "mixer": mixer, "mlp": mlp}


def model(vocab, width, eps, mult, layers, softcap=None):
    d = {"architecture": "Zebivik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "layers": layers}
    if softcap is not None:
        d["logit_softcap"] = softcap
    return d


MIXED = model(211, 80, 1e-6, 0.7, [
    layer(side(attention(6, 2, 24, 40, 0.2, dims=16, scaling=(4.0, 1.0, 4.0, 64)), lightning(12, 20, 0.3, 0.9, 0.999), 0.8, 1.3), dense(96, 0.6)),
    layer(rglru(120, 5, 4), moe(15, 3, 48, 1.5, (5, 2), shared=40)),
    layer(rglru(48, 3, 2), None),
    layer(side(attention(3, 3, 32, 16, 0.31, base=500.0), lightning(40, 24, 0.97, 0.0), 1.4, 0.6), moe(6, 6, 24, 0.8)),
    layer(rglru(80, 1, 3), dense(56, 2.5)),
    layer(side(attention(5, 1, 16, 48, 0.25, dims=0), lightning(100, 70, 1.0), 1.0, 1.0), moe(8, 1, 32, 2.5, (2, 1), shared=64)),
], softcap=20.0)

# the sizes that the matrix-core attention, the grouped experts, the tiles of the linear attention and the gates' products are built for
MEDIUM = model(500, 192, 1e-5, 0.45, [
    layer(rglru(256, 2, 4), moe(16, 4, 64, 2.0, (4, 2), shared=128)),
    layer(side(attention(8, 4, 64, 64, 0.12, scaling=(8.0, 1.0, 4.0, 128)), lightning(64, 128, 0.5, 0.96, 0.9995), 1.2, 0.9), moe(8, 2, 128, 1.3, (2, 1))),
    layer(rglru(192, 24, 4), dense(256, 1.5)),
    layer(side(attention(4, 2, 128, 96, 0.09, dims=64, base=5000.0), lightning(128, 64, 0.99, 0.8), 0.7, 1.1), moe(16, 3, 64, 2.0, (8, 5), shared=64)),
], softcap=15.0)

# attention heads of 144 and of 300 elements, beyond the matrix-core kernels' common sizes and beyond their widest
WIDE = model(128, 64, 1e-5, 1.1, [
    layer(side(attention(2, 1, 40, 136, 0.15), lightning(16, 16, 0.9, 0.95)), moe(8, 3, 32, 1.0, (2, 1), shared=24)),
    layer(side(attention(2, 2, 300, 20, 0.05, dims=100), lightning(8, 24, 0.7), 0.5, 2.0), dense(72, 4.0)),
], softcap=50.0)

# sizes that are multiples of nothing, one head, one channel a block, one tap, one expert, groups of one
ODD = model(101, 50, 2e-5, 0.9, [
    layer(rglru(35, 5, 1), moe(7, 3, 11, 1.7)),
    layer(side(attention(3, 1, 6, 5, 0.3, dims=4), lightning(7, 9, 0.9, 0.2, 0.99), 1.1, 0.9), moe(1, 1, 13, 0.5, shared=7)),
    layer(rglru(22, 22, 7), moe(5, 2, 9, 1.2, (5, 3))),
    layer(side(attention(1, 1, 7, 9, 0.2, dims=0), lightning(1, 3, 0.5), 0.3, 1.7), None),
    layer(rglru(77, 7, 3), dense(17, 0.3))])

# recurrent blocks alone (nothing bounds the text)
ONLY_LRU = model(64, 32, 1e-5, 1.4, [layer(rglru(40, 2, 4), None), layer(rglru(24, 4, 3), moe(4, 2, 16, 1.0, (2, 1)))])
ONLY_PARALLEL = model(64, 32, 1e-5, 1.0, [layer(side(attention(4, 2, 16, 16, 0.3, base=100.0), lightning(10, 14, 0.9, 0.6), 1.3, 0.7), None),
                                          layer(side(attention(2, 1, 8, 24, 0.4), lightning(150, 33, 0.98)), None)])
# one mixer that remembers, for what must be carried far
ONLY_STATE = model(64, 32, 1e-5, 1.0, [layer(rglru(24, 3, 2), None)])
ONE_SIDE = model(64, 32, 1e-5, 1.0, [layer(side(attention(2, 1, 16, 16, 0.3), lightning(12, 10, 0.9999, 1.0), 1.0, 1.0), None)])

ALL = {"mixed": MIXED, "medium": MEDIUM, "wide": WIDE, "odd": ODD, "only_lru": ONLY_LRU, "only_parallel": ONLY_PARALLEL,
       "only_state": ONLY_STATE, "one_side": ONE_SIDE}


def with_layers(cfg, layers):
    c = copy.deepcopy(cfg)
    c["layers"] = copy.deepcopy(layers)
    return c
