"""Small Bulodra configurations for the tests: sizes that differ from each other and from whole tiles, every mixer and feed-forward,
and values that real models often make equal or 1."""

YARN = dict(factor=4.0, original=48, fast=6.0, slow=1.0)


def rot(dims, base=1000.0, scaling=None):
    return dict(base=base, dims=dims) if scaling is None else dict(base=base, dims=dims, scaling=scaling)


def capped(heads=6, kv_heads=3, dim=24, vdim=40, window=50, scale=0.9, cap=2.5, dims=8, mlp=None):
    return dict(type="attention_2", mlp=mlp, mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, softcap=cap, mask=dict(size=window),
                                                        rot=rot(dims, 500.0)))


def attention(heads=6, kv_heads=2, dim=40, vdim=24, scale=0.2, dims=24, scaling=YARN, mlp=None):
    return dict(type="attention", mlp=mlp, mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot=rot(dims, 2000.0, scaling)))


def latent(heads=5, dim=24, rot_dim=16, vdim=40, kv_rank=48, q_rank=72, scale=0.2, scaling=YARN, mlp=None):
    return dict(type="latent_attention", mlp=mlp, mixer=dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale,
                                                             rot=rot(rot_dim, 700.0, scaling)))


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, groups=(1, 1), shared=None, limit=1.2, scale=1.7):
    d = dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top, scale=scale, groups=dict(count=groups[0], keep=groups[1])))
    return d if shared is None else dict(d, shared=dict(ff=shared[0], limit=shared[1]))


def config(layers, width=160, vocab=211, mult=0.8, logit_scale=1.6, eps=1e-5, buckets=53, mul_prev=29, mul_cur=7):
    return dict(architecture="Bulodra", vocab=vocab, width=width, layers=layers, norm=dict(eps=eps), residual_mult=mult, logit_scale=logit_scale,
                embedding=dict(bigram=dict(buckets=buckets, mul_prev=mul_prev, mul_cur=mul_cur)))


CASES = {
    # every mixer, every feed-forward, one layer without any
    "mixed": config([capped(mlp=dense(200)), attention(mlp=moe(12, 3, 48, (3, 2), (40, 0.6))), latent(mlp=moe(6, 2, 56, (2, 1))), capped(window=17, kv_heads=1),
                     attention(heads=3, kv_heads=3, dim=16, vdim=16, dims=16, scaling=None, mlp=dense(72))]),
    # sizes that are no multiples of anything, groups of one expert, a window of one token, factors beyond the number of buckets
    "odd": config([attention(heads=3, kv_heads=1, dim=9, vdim=11, dims=6, mlp=moe(7, 4, 10, (7, 5), (9, 2.0))), capped(heads=2, kv_heads=1, dim=12, vdim=5, dims=10, window=1),
                   latent(heads=3, dim=7, rot_dim=6, vdim=5, kv_rank=13, q_rank=11, mlp=dense(50)), capped(heads=1, kv_heads=1, dim=20, vdim=12, dims=20, window=65,
                                                                                                      mlp=moe(9, 2, 22, (3, 3)))],
                  width=102, vocab=97, mult=1.0, logit_scale=1.0, eps=1e-6, buckets=31, mul_prev=1009, mul_cur=2003),
    # whole matrix tiles everywhere: weight streams, partials, tiled prefills, one expert a token
    "tiles": config([latent(heads=4, dim=64, rot_dim=32, vdim=64, kv_rank=128, q_rank=128, scale=0.12, mlp=dense(512)),
                     capped(heads=8, kv_heads=2, dim=64, vdim=64, window=64, dims=32, scale=0.5, mlp=moe(20, 1, 128, (5, 2), (128, 1.0))),
                     attention(heads=4, kv_heads=4, dim=64, vdim=128, dims=64, scale=0.125, mlp=moe(4, 4, 128, (2, 2), (64, 3.0)))], width=256, vocab=320, logit_scale=0.5),
    # heads wider than the tiled prefill takes, more query heads on a key head than a matrix tile has rows, a window no prompt fills
    "flat": config([attention(heads=20, kv_heads=1, dim=136, vdim=136, dims=48, scale=0.08, mlp=moe(9, 2, 24, (3, 1))),
                    latent(heads=20, dim=40, rot_dim=8, vdim=24, kv_rank=72, q_rank=40, mlp=dense(64)), capped(window=4096, cap=50.0, mlp=dense(64))], width=128),
}
