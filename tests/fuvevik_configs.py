"""Small Fuvevik configurations for the tests.  Between them every mechanism stands alone and beside the others, every
optional block of keys is on and off, and sizes that a model may happen to make equal or 1 (streams, heads and kv heads,
key and value size, the query factors of a layer and of the layer that reads its keys, experts and router outputs, chosen
and all of them, the experts' and the shared expert's limits) differ; several sizes are no multiples of 4, 8 or 16."""


def attn(heads, kv_heads, dim, vdim, scale, temp=None, kv_from=None):
    d = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if temp is not None:
        d["q_temp"] = {"coef": temp[0], "every": temp[1]}
    if kv_from is not None:
        d["kv_from"] = kv_from
    return d


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit, identity=None, shared=None):
    router = {"experts": experts, "top": top}
    if identity is not None:
        router["identity"] = identity
    d = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": router}
    if shared is not None:
        d["shared"] = {"ff": shared[0], "limit": shared[1]}
    return d


def model(width, vocab, streams, layers, eps=1e-5):
    return {"architecture": "Fuvevik", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps},
            "layers": [{"type": "attention", "mixer": mixer, "mlp": mlp} for mixer, mlp in layers]}


# one mechanism at a time
ATTN_ONLY = model(64, 97, 2, [(attn(6, 2, 16, 32, 0.4, temp=(0.8, 9)), None)])
ATTN_PLAIN = model(48, 50, 1, [(attn(3, 3, 20, 20, 0.3), None)])                   # one stream, no query factor; heads of 20: the vector units
ATTN_NARROW = model(64, 61, 3, [(attn(5, 1, 32, 16, 0.25, temp=(0.1, 1)), None)])   # the factor moves at every position; narrow values
DENSE_ONLY = model(56, 83, 4, [(attn(1, 1, 8, 8, 0.3), dense(144))], eps=1e-3)
MOE_ONLY = model(56, 83, 2, [(attn(2, 1, 8, 12, 0.3), moe(12, 3, 24, 1.25, identity=3, shared=(40, 2.0)))])
MOE_BARE = model(40, 61, 2, [(attn(2, 2, 8, 8, 0.4), moe(5, 1, 17, 0.8))])          # no identity experts, no shared expert, one expert a token
MOE_IDENTITY = model(40, 61, 3, [(attn(2, 2, 8, 8, 0.4), moe(2, 4, 16, 3.0, identity=5))])      # most outputs give the input back
MOE_ALL = model(48, 50, 2, [(attn(2, 1, 16, 16, 0.3), moe(3, 5, 32, 1.0, identity=2, shared=(16, 0.5)))])   # every output is chosen
MOE_MANY = model(32, 45, 2, [(attn(1, 1, 16, 16, 0.3), moe(66, 7, 8, 1.5, identity=4))])        # more router outputs than lanes
# streams of every compiled form: one a kernel of its own size, five to eight, more
FIVE_STREAMS = model(52, 61, 5, [(attn(2, 1, 16, 16, 0.3, temp=(0.5, 20)), dense(64)), (attn(2, 2, 16, 8, 0.3), moe(4, 2, 16, 1.0, identity=1))])
MANY_STREAMS = model(36, 53, 11, [(attn(2, 1, 16, 16, 0.3), dense(40)), (attn(2, 1, 16, 16, 0.2, temp=(0.3, 5), kv_from=0), None)])
# layers read the keys and values of another: other query heads, another factor and query factor than the layer that writes
SHARED_KV = model(64, 97, 4, [(attn(4, 2, 16, 8, 0.3, temp=(0.5, 30)), dense(96)), (attn(2, 1, 8, 8, 0.3, temp=(0.5, 12)), None),
                              (attn(2, 2, 16, 8, 0.25, kv_from=0), moe(4, 2, 16, 1.0, identity=1)),
                              (attn(6, 2, 16, 8, 0.35, temp=(1.0, 7), kv_from=0), None), (attn(3, 1, 8, 8, 0.5, kv_from=1), dense(33))])
# sizes that are multiples of nothing much: a width of 50, feed-forwards of 37 and 45, a vocabulary of 61
ODD_SIZES = model(50, 61, 3, [(attn(2, 1, 12, 10, 0.3, temp=(0.4, 11)), moe(6, 2, 37, 1.1, identity=1, shared=(45, 1.7))),
                              (attn(2, 2, 6, 10, 0.3), dense(37)), (attn(4, 1, 12, 10, 0.2, kv_from=0), moe(3, 3, 9, 2.0))])
# everything together
MIXED = model(72, 131, 4, [(attn(6, 2, 16, 24, 0.25, temp=(0.4, 50)), dense(160)),
                           (attn(6, 2, 32, 16, 0.2, temp=(0.7, 16)), moe(8, 3, 24, 1.5, identity=2, shared=(40, 2.0))),
                           (attn(4, 4, 24, 24, 0.3), moe(6, 2, 32, 1.0, shared=(16, 1.0))),
                           (attn(4, 2, 32, 16, 0.25, temp=(0.3, 33), kv_from=1), None),
                           (attn(8, 2, 32, 16, 0.15, temp=(0.6, 128), kv_from=1), moe(9, 4, 16, 2.0, identity=4))])
# softmax that picks one key, and more sharply with every step of the query factor
SHARP = model(64, 97, 3, [(attn(4, 2, 16, 16, 1.0, temp=(1.0, 19)), None), (attn(2, 2, 16, 16, 0.8, temp=(1.2, 64), kv_from=0), dense(48))])

ALL = {"attn_only": ATTN_ONLY, "attn_plain": ATTN_PLAIN, "attn_narrow": ATTN_NARROW, "dense_only": DENSE_ONLY, "moe_only": MOE_ONLY,
       "moe_bare": MOE_BARE, "moe_identity": MOE_IDENTITY, "moe_all": MOE_ALL, "moe_many": MOE_MANY, "five_streams": FIVE_STREAMS,
       "many_streams": MANY_STREAMS, "shared_kv": SHARED_KV, "odd_sizes": ODD_SIZES, "mixed": MIXED, "sharp": SHARP}
