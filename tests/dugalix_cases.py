"""Small Dugalix configurations for the tests: sizes that differ from each other and from whole tiles, every mixer and feed-forward,
and values that real models often make equal or 1."""


def rot(dims, base=1000.0, factor=None):
    return dict(base=base, dims=dims) if factor is None else dict(base=base, dims=dims, scaling=dict(factor=factor))


def attention(heads=6, kv_heads=3, dim=24, window=50, scale=0.3, dims=8, mlp=None):
    return dict(type="attention", mlp=mlp, mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=scale, mask=dict(size=window),
                                                      rot=rot(dims, 500.0)))


def memory(heads=4, dim=20, vdim=28, cap=3.0):
    return dict(heads=heads, dim=dim, vdim=vdim, gate_cap=cap)


def parallel(heads=6, kv_heads=2, dim=24, vdim=40, window=21, first=5, scale=0.25, dims=16, factor=4.0, right=None, scales=(1.3, 0.6), mlp=None):
    left = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, mask=dict(size=window, keep_first=first), rot=rot(dims, 2000.0, factor))
    return dict(type="parallel", mlp=mlp, mixer=dict(left=left, right=right or memory(), left_scale=scales[0], right_scale=scales[1]))


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, identity, top, ff, groups=(1, 1), shared=None):
    d = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, identity=identity, top=top, groups=dict(count=groups[0], keep=groups[1])))
    return d if shared is None else dict(d, shared=dict(ff=shared))


def config(layers, width=160, vocab=211, mult=0.8, eps=1e-5):
    return dict(architecture="Dugalix", vocab=vocab, width=width, layers=layers, norm=dict(eps=eps), residual_mult=mult)


CASES = {
    # both mixers, every feed-forward, one layer without any
    "mixed": config([parallel(mlp=moe(7, 2, 3, 48, (3, 2), 40)), attention(mlp=dense(200)), parallel(window=66, first=17, right=memory(3, 32, 24, 9.0)),
                     attention(window=17, heads=4, kv_heads=1, dim=40, dims=40, mlp=moe(9, 3, 2, 56, (2, 1), 72)),
                     parallel(heads=3, kv_heads=3, dim=16, vdim=16, first=0, factor=1.0, scales=(1.0, 1.0), mlp=dense(72))]),
    # sizes that are no multiples of anything, groups of one, a window of one token, no identities, no rotation at all, a negative factor
    "odd": config([attention(heads=3, kv_heads=1, dim=9, dims=6, window=1, mlp=moe(5, 0, 2, 10, (5, 3), 9)),
                   parallel(heads=2, kv_heads=1, dim=12, vdim=5, dims=10, window=1, first=1, right=memory(3, 7, 11, 2.0), scales=(-0.7, 0.4), mlp=dense(50)),
                   attention(heads=2, kv_heads=2, dim=11, dims=0, window=65, mlp=moe(3, 6, 2, 22, (3, 3))),
                   parallel(heads=1, kv_heads=1, dim=20, vdim=12, dims=20, window=9, first=30, right=memory(1, 13, 3, 5.0))], width=102, vocab=97, mult=1.0, eps=1e-6),
    # whole matrix tiles everywhere: weight streams, partials, tiled prefills, one expert a token
    "tiles": config([parallel(heads=4, kv_heads=2, dim=64, vdim=64, window=64, first=64, dims=64, scale=0.125, right=memory(4, 64, 64, 15.0), mlp=dense(512)),
                     attention(heads=8, kv_heads=2, dim=64, dims=32, window=64, scale=0.125, mlp=moe(12, 4, 1, 128, (4, 2), 128)),
                     parallel(heads=4, kv_heads=4, dim=64, vdim=128, dims=32, window=90, right=memory(2, 128, 128, 6.0), mlp=moe(4, 4, 4, 128, (2, 2), 128))],
                    width=256, vocab=320, mult=0.6),
    # heads wider than the tiled prefill takes, more query heads on a key head than a matrix tile has rows, more first tokens than a
    # prompt has, a memory wider than the chunked form takes
    "flat": config([attention(heads=20, kv_heads=1, dim=136, dims=48, window=4096, scale=0.08, mlp=moe(5, 4, 2, 24, (3, 1))),
                    parallel(heads=18, kv_heads=1, dim=40, vdim=136, window=30, first=400, right=memory(2, 200, 80, 12.0), mlp=dense(64))], width=128),
}
