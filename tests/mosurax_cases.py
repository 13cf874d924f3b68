"""Small Mosurax configurations for the tests: sizes that differ from each other and from whole tiles, loops at either end, every
kind of feed-forward."""


def attention(heads=6, kv_heads=3, dim=24, vdim=40, window=50, scale=0.2, mlp=None):
    return dict(type="attention", mlp=mlp, mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, mask=dict(size=window)))


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, shared=None):
    d = dict(kind="moe", router=dict(experts=experts, top=top), expert=dict(ff=ff))
    return d if shared is None else dict(d, shared=dict(ff=shared))


def config(layers, width=160, vocab=211, loop=None, cap=20.0, eps=1e-5, positions=256):
    d = dict(architecture="Mosurax", vocab=vocab, width=width, layers=layers, norm=dict(eps=eps), max_positions=positions, logit_softcap=cap)
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


CASES = {
    # a loop in the middle over both kinds of feed-forward, layers of different sizes in it
    "mixed": config([attention(mlp=dense(200)), attention(mlp=moe(12, 3, 48, 96)), attention(heads=4, kv_heads=1, dim=16, vdim=16, window=17, mlp=dense(72)),
                     attention(heads=2, kv_heads=2, dim=40, vdim=24, window=64, mlp=moe(5, 2, 64, 40))], loop=(1, 3, 2)),
    # looped from the first layer to the last, sizes that are no multiples of anything, no shared expert, one layer without a
    # feed-forward
    "odd": config([attention(heads=3, kv_heads=1, dim=9, vdim=11, window=33, mlp=moe(7, 4, 10)), attention(heads=2, kv_heads=1, dim=12, vdim=5, window=1),
                   attention(heads=1, kv_heads=1, dim=20, vdim=12, window=65, mlp=dense(50))], width=102, vocab=97, loop=(0, 3, 3), cap=5.0, eps=1e-6),
    # whole matrix tiles everywhere, one query head a key head, one expert a token, one pass
    "tiles": config([attention(heads=4, kv_heads=4, dim=64, vdim=128, window=90, scale=0.125, mlp=dense(512)),
                     attention(heads=8, kv_heads=2, dim=64, vdim=64, window=64, scale=0.15, mlp=moe(20, 1, 128, 192)),
                     attention(heads=4, kv_heads=2, dim=128, vdim=64, window=65, scale=0.1, mlp=moe(4, 4, 128, 64))], width=256, vocab=320, loop=(2, 3, 1)),
    # no loop; heads wider than the tiled prefill takes, more query heads on a key head than a matrix tile has rows
    "flat": config([attention(heads=20, kv_heads=1, dim=136, vdim=136, window=40, scale=0.08, mlp=moe(9, 2, 24, 24)), attention(window=4096, mlp=dense(64))],
                   width=128),
}
