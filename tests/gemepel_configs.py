"""Small Gemepel configurations (config.json dictionaries) for the tests.  They differ from each other in every size: one
to five heads, plain / rotated / value sizes and latent ranks that are all different inside a layer, query and key
latent sizes on either side of each other, several readers of one layer's keys, recurrent keys below and above
values and up to 150 channels, decays of ranks 1 to 40 and tau from 0.5 to 16, one to four groups of experts (of one
expert, of two and of more) with some or all kept, top from one to all, layers without a feed-forward, embeddings with and
without a table of token pairs."""
import copy


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base=10000.0, kv_from=None, dims=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
         "rot": {"base": base, "dims": rot_dim if dims is None else dims}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def gla(heads, dim, vdim, tau, rank):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": rank}


def moe(experts, top, ff, scale=1.0, groups=None):
    router = {"experts": experts, "top": top, "scale": scale}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": router}


def layer(mixer, mlp):
    return {"type": "gla" if "tau" in mixer else "latent_attention", "mixer": mixer, "mlp": mlp}


def model(vocab, width, eps, alpha, layers, scale=1.0, bigram=None):
    emb = {"scale": scale}
    if bigram is not None:
        emb["bigram"] = dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))
    return {"architecture": "Gemepel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha, "embedding": emb,
            "layers": layers}


MIXED = model(211, 80, 1e-6, 1.7, [
    layer(latent(3, 16, 8, 24, 20, 40, 0.2), moe(12, 3, 48, 1.5, (4, 2))),
    layer(gla(5, 12, 20, 4.0, 7), moe(6, 6, 24, 0.8, (1, 1))),
    layer(latent(5, 8, 8, 16, 36, 40, 0.31, kv_from=0), None),
    layer(gla(2, 40, 24, 16.0, 16), None),
    layer(latent(1, 32, 4, 40, 9, 20, 0.11, base=300.0), moe(8, 1, 32, 2.5, (2, 1))),
    layer(latent(2, 12, 8, 20, 50, 40, 0.25, kv_from=0), moe(9, 2, 40, 1.0, (3, 3))),
    layer(gla(1, 100, 70, 1.0, 40), moe(4, 2, 16, 3.0, (4, 2))),
], scale=0.7, bigram=(37, 5, 11))

# the sizes that the matrix-core attention, the grouped experts and the recurrence's wider forms are built for
MEDIUM = model(500, 192, 1e-5, 2.2, [
    layer(latent(4, 48, 32, 32, 64, 96, 0.11), moe(16, 4, 64, 2.0, (4, 2))),
    layer(gla(2, 64, 128, 16.0, 16), moe(8, 2, 128, 1.3, (2, 1))),
    layer(gla(3, 128, 64, 8.0, 16), moe(16, 3, 64, 2.0, (8, 5))),
    layer(latent(8, 16, 32, 64, 96, 96, 0.14, kv_from=0), moe(16, 4, 64, 2.0, (4, 2))),
    layer(latent(6, 32, 16, 24, 48, 64, 0.14, base=5000.0), None),
], scale=1.3, bigram=(101, 31, 3))

# latent heads of 144 and of 336: beyond the widest head of the matrix-core attention kernels
WIDE_LATENT = model(128, 64, 1e-5, 1.1, [
    layer(latent(2, 16, 16, 16, 24, 128, 0.1), moe(8, 3, 32, 1.0, (2, 1))),
    layer(latent(3, 8, 16, 24, 70, 128, 0.1, kv_from=0), None),
    layer(latent(2, 16, 16, 24, 40, 320, 0.05), moe(4, 2, 24, 2.0, (2, 1))),
], scale=0.9, bigram=(17, 3, 2))

# sizes that are multiples of nothing, one expert, one group of one expert each, a mixer that rotates nothing or a part
ODD = model(101, 50, 2e-5, 0.6, [
    layer(latent(3, 6, 2, 5, 7, 10, 0.3), moe(7, 3, 11, 1.7)),
    layer(gla(3, 7, 9, 2.0, 5), moe(1, 1, 13, 0.5)),
    layer(latent(1, 7, 0, 9, 11, 13, 0.2), moe(5, 2, 9, 1.2, (5, 3))),
    layer(latent(2, 5, 6, 3, 3, 9, 0.35, base=900.0, dims=4), None),
    layer(gla(1, 1, 3, 16.0, 1), moe(6, 2, 7, 1.0, (2, 2))),
    layer(latent(2, 3, 2, 7, 19, 10, 0.3, kv_from=0), None)], scale=2.1, bigram=(1, 7, 13))

# recurrences alone (nothing bounds the text), one of them with keys of more than 128 channels, no table of pairs
ONLY_GLA = model(64, 32, 1e-5, 1.4, [layer(gla(2, 10, 14, 16.0, 3), None), layer(gla(2, 150, 33, 0.5, 20), moe(4, 2, 16, 1.0, (2, 1)))])
ONLY_LATENT = model(64, 32, 1e-5, 2.0, [layer(latent(2, 8, 4, 6, 10, 12, 0.3, base=100.0), None)], bigram=(23, 2, 9))
# one recurrence under decays close to one, for what must be carried far
ONLY_STATE = model(64, 32, 1e-5, 1.0, [layer(gla(2, 12, 10, 16.0, 4), None)])

ALL = {"mixed": MIXED, "medium": MEDIUM, "wide_latent": WIDE_LATENT, "odd": ODD, "only_gla": ONLY_GLA, "only_latent": ONLY_LATENT,
       "only_state": ONLY_STATE}


def with_layers(cfg, layers):
    c = copy.deepcopy(cfg)
    c["layers"] = copy.deepcopy(layers)
    return c
