"""Plain, slow evaluation of the Bulodra design: a decoder with bigram embeddings whose layers mix with rotary grouped-query attention
(learned sinks, biases, norms on queries and keys), latent attention with query latents, or windowed soft-capped attention with a
gate a head, in front of dense or group-limited routed feed-forward parts; every sublayer reads the residual stream itself and is
normed behind.  One function per mechanism, every attention row one explicit softmax over its visible keys, every token's
experts one by one; nothing is shared with the product path.

`weights` maps tensor names to tensors; everything is computed in `dtype` (float64 unless told otherwise) on the CPU.  A whole
sequence goes in, logits and the residual stream behind every layer come out.  `oracle.hybrid.rounding` applies."""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

from . import hybrid as oh

F64 = torch.float64


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def bigram_rows(tokens: List[int], mul_prev: int, mul_cur: int, buckets: int) -> List[int]:
    """Row of the bigram table for every token: the pair (token before, token) hashed; the first token has the last row."""
    return [buckets if i == 0 else (tokens[i - 1] * mul_prev + t * mul_cur) % buckets for i, t in enumerate(tokens)]


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def frequencies(dims: int, base: float, scaling: Optional[dict] = None) -> Tuple[List[float], float]:
    """(rotation per position of every pair, factor on cos and sin); `scaling` stretches the slow pairs (YaRN)."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return f, 1.0

    def turns(t):           # the (fractional) pair index that turns t times over the original length
        return dims * math.log(scaling["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo = max(math.floor(turns(scaling["fast"])), 0)
    hi = min(math.ceil(turns(scaling["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / scaling["factor"] * ramp + fi * (1.0 - ramp))
    return out, 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_halves(x, rot: dict):
    """x [T, heads, n], row t at position t: dimension i turns with i + dims / 2, on the first dims dimensions."""
    dims = rot["dims"]
    f, factor = frequencies(dims, rot["base"], rot.get("scaling"))
    out, pos = x.clone(), torch.arange(x.shape[0], dtype=x.dtype)[:, None]
    for i in range(dims // 2):
        c, s = torch.cos(pos * f[i]) * factor, torch.sin(pos * f[i]) * factor
        u, v = x[..., i], x[..., i + dims // 2]
        out[..., i], out[..., i + dims // 2] = u * c - v * s, v * c + u * s
    return out


def attend(q, k, v, scale, window=None, cap=None, sink=None):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V].  Position i sees the keys up to itself, at most `window` of them; scores go
    through cap * tanh(s / cap); sink [H] adds exp(sink) to every denominator."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    o = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        for h in range(H):
            s = k[lo:i + 1, h // per] @ q[i, h] * scale
            if cap is not None:
                s = cap * torch.tanh(s / cap)
            if sink is not None:
                s = torch.cat([s, sink[h:h + 1]])
            e = torch.exp(s - s.max())
            p = e / e.sum()
            o[i, h] = p[:i + 1 - lo] @ v[lo:i + 1, h // per]
    return o


def _heads(h, w, name, n, bias=False):
    y = h @ w[name].T
    return oh._r(y + w[name + ".b"] if bias else y).view(h.shape[0], n, -1)


def biased_attention(h, w, m, eps):
    """w: 'q', 'k', 'v' with '.b', 'q.norm', 'k.norm', 'sink', 'o'."""
    H, G = m["heads"], m["kv_heads"]
    q, k, v = (_heads(h, w, n, c, bias=True) for n, c in (("q", H), ("k", G), ("v", G)))
    q = oh._r(rotate_halves(oh.rms_norm(q, w["q.norm"], eps), m["rot"]))
    k = oh._r(rotate_halves(oh.rms_norm(k, w["k.norm"], eps), m["rot"]))
    o = oh._r(attend(q, k, v, m["scale"], sink=w["sink"]))
    return oh.linear(o.reshape(h.shape[0], -1), w["o"])


def latent_attention(h, w, m, eps):
    """w: 'dq', 'dq.norm', 'uq', 'dkv', 'dkv.norm', 'uk', 'uv', 'sink', 'o'."""
    T, H, D, RK = h.shape[0], m["heads"], m["dim"], m["kv_rank"]
    cq = oh._r(oh.rms_norm(oh.linear(h, w["dq"]), w["dq.norm"], eps))
    q = oh.linear(cq, w["uq"]).view(T, H, D + m["rot_dim"])
    dkv = oh.linear(h, w["dkv"])
    c = oh._r(oh.rms_norm(dkv[:, :RK], w["dkv.norm"], eps))
    kr = oh._r(rotate_halves(dkv[:, None, RK:], m["rot"])).expand(T, H, -1)
    q = torch.cat([q[..., :D], oh._r(rotate_halves(q[..., D:], m["rot"]))], -1)
    k = torch.cat([oh.linear(c, w["uk"]).view(T, H, D), kr], -1)
    v = oh.linear(c, w["uv"]).view(T, H, m["vdim"])
    o = oh._r(attend(q, k, v, m["scale"], sink=w["sink"]))
    return oh.linear(o.reshape(T, -1), w["o"])


def capped_attention(h, w, m, eps):
    """w: 'q', 'k', 'v', 'g' (one row a head), 'o'."""
    H, G = m["heads"], m["kv_heads"]
    q, k, v = (_heads(h, w, n, c) for n, c in (("q", H), ("k", G), ("v", G)))
    q, k = (oh._r(unit_rms(rotate_halves(x, m["rot"]), eps)) for x in (q, k))
    o = attend(q, k, v, m["scale"], window=m["mask"]["size"], cap=m["softcap"])
    o = oh._r(o * sigmoid(oh.linear(h, w["g"]))[..., None])
    return oh.linear(o.reshape(h.shape[0], -1), w["o"])


MIXERS = {"attention": biased_attention, "latent_attention": latent_attention, "attention_2": capped_attention}


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def gelu_mlp(h, w):
    return oh.linear(oh._r(gelu_tanh(oh.linear(h, w["gate"])) * oh.linear(h, w["up"])), w["down"])


def clamped_swiglu(g, u, limit):
    g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


def expert(h, w, limit):
    return oh.linear(oh._r(clamped_swiglu(oh.linear(h, w["gate"]), oh.linear(h, w["up"]), limit)), w["down"])


margins: List[float] = []      # smallest gap of every route() call between what was just taken and what was just left out


def route(h, w, correction, r: dict):
    """-> per token [(expert, weight)]: sigmoid scores; groups ranked by their two best corrected scores, experts of the kept groups by
    their corrected score, weighted by the plain score times r['scale']."""
    s = sigmoid(h @ w.T)
    choice = s + correction
    E, groups = s.shape[1], r.get("groups") or dict(count=1, keep=1)
    size, keep = E // groups["count"], groups["keep"]
    out = []
    for t in range(h.shape[0]):
        rank = []
        for g in range(groups["count"]):
            best = sorted((float(choice[t, e]) for e in range(g * size, (g + 1) * size)), reverse=True)
            rank.append((sum(best[:2]), g))
        rank.sort(key=lambda x: (-x[0], x[1]))
        if keep < len(rank):
            margins.append(rank[keep - 1][0] - rank[keep][0])
        open_ = [e for _, g in rank[:keep] for e in range(g * size, (g + 1) * size)]
        open_.sort(key=lambda e: (-float(choice[t, e]), e))
        if r["top"] < len(open_):
            margins.append(float(choice[t, open_[r["top"] - 1]] - choice[t, open_[r["top"]]]))
        out.append([(e, s[t, e] * r["scale"]) for e in open_[:r["top"]]])
    return out


def moe_mlp(h, w, f):
    out = torch.zeros_like(h)
    for t, chosen in enumerate(route(h, w["router"], w["correction"], f["router"])):
        for e, p in chosen:
            out[t] += p * expert(h[t:t + 1], oh._sub(w, f"e{e}."), f["expert"]["limit"])[0]
    if f.get("shared"):
        out = out + expert(h, oh._sub(w, "shared."), f["shared"]["limit"])
    return out


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=F64):
    """-> (logits [T, vocab], [residual stream behind every layer])."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, m, big = cfg["norm"]["eps"], cfg["residual_mult"], cfg["embedding"]["bigram"]
    x = w["embed"][torch.tensor(tokens)] + w["bigram"][torch.tensor(bigram_rows(tokens, big["mul_prev"], big["mul_cur"], big["buckets"]))]
    trace = []
    for i, lay in enumerate(cfg["layers"]):
        p, f = f"l{i}.", lay["mlp"]
        x = x + m * oh.rms_norm(MIXERS[lay["type"]](oh._r(x), oh._sub(w, p + "mix."), lay["mixer"], eps), w[p + "norm1"], eps)
        if f is not None:
            h, sub = oh._r(x), oh._sub(w, p + "mlp.")
            x = x + m * oh.rms_norm(moe_mlp(h, sub, f) if f["kind"] == "moe" else gelu_mlp(h, sub), w[p + "norm2"], eps)
        trace.append(x)
    return oh.linear(oh._r(oh.rms_norm(x, w["final.norm"], eps)), w["head"]) * cfg["logit_scale"], trace


# ---------------------------------------------------------------------------------------------- random models
def tensor_shapes(cfg: dict) -> Dict[str, Tuple[int, ...]]:
    W = cfg["width"]
    out: Dict[str, Tuple[int, ...]] = {"embed": (cfg["vocab"], W), "bigram": (cfg["embedding"]["bigram"]["buckets"] + 1, W), "head": (cfg["vocab"], W),
                                       "final.norm": (W,)}

    def mlp(prefix, ff):
        out.update({prefix + "gate": (ff, W), prefix + "up": (ff, W), prefix + "down": (W, ff)})

    for i, lay in enumerate(cfg["layers"]):
        m, f, p = lay["mixer"], lay["mlp"], f"l{i}."
        H, D, V = m["heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = (W,)
        mix = {"o": (W, H * V)}
        if lay["type"] == "latent_attention":
            R, K, Q = m["rot_dim"], m["kv_rank"], m["q_rank"]
            mix.update({"dq": (Q, W), "dq.norm": (Q,), "uq": (H * (D + R), Q), "dkv": (K + R, W), "dkv.norm": (K,), "uk": (H * D, K), "uv": (H * V, K), "sink": (H,)})
        else:
            G = m["kv_heads"]
            mix.update({"q": (H * D, W), "k": (G * D, W), "v": (G * V, W)})
            if lay["type"] == "attention":
                mix.update({"q.b": (H * D,), "k.b": (G * D,), "v.b": (G * V,), "q.norm": (D,), "k.norm": (D,), "sink": (H,)})
            else:
                mix["g"] = (H, W)
        out.update({p + "mix." + n: s for n, s in mix.items()})
        if f is None:
            continue
        out[p + "norm2"] = (W,)
        if f["kind"] == "dense":
            mlp(p + "mlp.", f["ff"])
            continue
        for e in range(f["router"]["experts"]):
            mlp(f"{p}mlp.e{e}.", f["expert"]["ff"])
        out[p + "mlp.router"], out[p + "mlp.correction"] = (f["router"]["experts"], W), (f["router"]["experts"],)
        if f.get("shared"):
            mlp(p + "mlp.shared.", f["shared"]["ff"])
    return out


CODE_DIMS, CODES = 8, 12


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """bf16 weights whose every branch matters: matrices keep unit variance, norms spread around 1, sinks and biases are of the size of
    scores and activations, corrections reach below zero.  No token sits between two experts: the first CODE_DIMS columns of the
    embedding hold one of CODES sign patterns, nothing else writes to those columns of the residual, and the routers read only
    them, drawn until every pattern's choice of groups and experts is clear."""
    g = torch.Generator().manual_seed(seed)
    code = torch.randint(0, 2, (CODES, CODE_DIMS), generator=g) * 4.0 - 2.0
    shapes, out = tensor_shapes(cfg), {}
    for name, shape in shapes.items():
        r = torch.randn(shape, generator=g)
        last = name.split(".")[-1]
        if last in ("norm1", "norm2", "norm"):
            t = 1.0 + 0.2 * r
        elif last in ("embed", "bigram", "sink"):
            t = r
        elif last in ("b", "correction"):
            t = r * 0.5
        else:
            t = r / math.sqrt(shape[1])
        if last == "embed":
            t[:, :CODE_DIMS] = code[torch.arange(shape[0]) % CODES]
        elif last == "bigram":
            t[:, :CODE_DIMS] = 0.0
        elif last in ("norm1", "norm2"):
            t[:CODE_DIMS] = 0.0
        out[name] = t.to(torch.bfloat16)
    saved = list(margins)
    for i, lay in enumerate(cfg["layers"]):
        if lay["mlp"] is None or lay["mlp"]["kind"] != "moe":
            continue
        name, best = f"l{i}.mlp.router", None
        for _ in range(200):
            w = torch.zeros(shapes[name])
            w[:, :CODE_DIMS] = torch.randn((shapes[name][0], CODE_DIMS), generator=g) * 0.3
            w = w.to(torch.bfloat16)
            margins.clear()
            route(code.double(), w[:, :CODE_DIMS].double(), out[f"l{i}.mlp.correction"].double(), lay["mlp"]["router"])
            gap = min(margins, default=1.0)
            if best is None or gap > best[0]:
                best = (gap, w)
            if gap > 0.02:
                break
        out[name] = best[1]
    margins[:] = saved
    return out
