"""Plain, slow evaluation of the Dugalix design: a decoder whose layers mix either with windowed attention whose weights are sigmoids of
the scores and whose values are the keys, or with a windowed softmax attention that keeps the first tokens beside a matrix memory
with exponential gates; feed-forward parts are squared-relu layers, dense or routed among experts and identities; every sublayer is
normed in front and behind, and every mixer reads a blend of its token and the one in front.  One function per mechanism, every
attention row over its list of visible keys, the recurrence token by token, every token's experts one by one; nothing is shared with the
product path.

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


def norm(x, w, eps):
    """RMS norm; the weight is stored around zero."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * (1.0 + w)


def token_shift(h, mu):
    """Every token's row moved towards the row of the token in front (zeros in front of the first)."""
    front = torch.cat([torch.zeros_like(h[:1]), h[:-1]])
    return h + (front - h) * mu


def rotate(x, rot: dict):
    """x [T, heads, dim] at positions 0 .. T - 1: the pair (i, i + dims / 2) of the first `dims` dimensions turns by position * f_i."""
    n = rot["dims"]
    factor = (rot.get("scaling") or {}).get("factor", 1.0)
    out = x.clone()
    for t in range(x.shape[0]):
        for i in range(n // 2):
            a = t * rot["base"] ** (-2.0 * i / n) / factor
            c, s = math.cos(a), math.sin(a)
            u, v = x[t, :, i], x[t, :, i + n // 2]
            out[t, :, i], out[t, :, i + n // 2] = u * c - v * s, v * c + u * s
    return out


def visible(i: int, window: Optional[int] = None, first: int = 0) -> List[int]:
    """The positions that position i sees: the last `window` up to itself, and the first `first`."""
    return [j for j in range(i + 1) if window is None or i - j < window or j < first]


def attend(q, k, v, scale, window=None, first=0, offsets=None):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V].  Softmax over the visible keys; offsets [H]: sigmoid(score + offset) instead,
    key by key."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    o = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        keys = visible(i, window, first)
        for h in range(H):
            s = k[keys, h // per] @ q[i, h] * scale
            if offsets is not None:
                p = sigmoid(s + offsets[h])
            else:
                e = torch.exp(s - s.max())
                p = e / e.sum()
            o[i, h] = p @ v[keys, h // per]
    return o


def _heads(h, w, name, n, bias=False):
    y = h @ w[name].T
    return oh._r(y + w[name + ".b"] if bias else y).view(h.shape[0], n, -1)


def sigmoid_attention(h, w, m, eps):
    """w: 'q', 'k', 'pb' (one a head), 'o'.  The values are the keys as projected."""
    q, k = _heads(h, w, "q", m["heads"]), _heads(h, w, "k", m["kv_heads"])
    o = attend(oh._r(rotate(q, m["rot"])), oh._r(rotate(k, m["rot"])), k, m["scale"], window=m["mask"]["size"], offsets=w["pb"])
    return oh.linear(oh._r(o).reshape(h.shape[0], -1), w["o"])


def biased_attention(h, w, m):
    """w: 'q', 'k', 'v', 'o' with '.b'."""
    H, G = m["heads"], m["kv_heads"]
    q, k, v = (_heads(h, w, n, c, bias=True) for n, c in (("q", H), ("k", G), ("v", G)))
    o = attend(oh._r(rotate(q, m["rot"])), oh._r(rotate(k, m["rot"])), v, m["scale"], window=m["mask"]["size"], first=m["mask"]["keep_first"])
    return oh._r(oh._r(o).reshape(h.shape[0], -1) @ w["o"].T + w["o.b"])


def log_sigmoid(z):
    return -oh.softplus(-z)


def memory_recurrence(q, k, v, i, f):
    """q, k [T, H, D], v [T, H, V], log gates i, f [T, H] -> [T, H, V].  State S [D, V] and n [D] relative to e^m, from zero, m from zero."""
    T, H, D = q.shape
    o = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        S, n, m = torch.zeros(D, v.shape[2], dtype=q.dtype), torch.zeros(D, dtype=q.dtype), torch.zeros((), dtype=q.dtype)
        for t in range(T):
            new = torch.maximum(f[t, h] + m, i[t, h])
            keep, add = torch.exp(f[t, h] + m - new), torch.exp(i[t, h] - new)
            S = keep * S + add * torch.outer(k[t, h], v[t, h])
            n = keep * n + add * k[t, h]
            m = new
            o[t, h] = S.T @ q[t, h] / (torch.maximum((n @ q[t, h]).abs(), torch.exp(-m)) + 1e-6)
    return o


def matrix_memory(h, w, m, eps):
    """w: 'q', 'k', 'v', 'g', 'norm', 'o', and the gates' 'i', 'f' with '.b'."""
    T, H, cap = h.shape[0], m["heads"], m["gate_cap"]
    q, k, v = (_heads(h, w, n, H) for n in ("q", "k", "v"))
    i, f = (cap * torch.tanh((oh.linear(h, w[n]) + w[n + ".b"]) / cap) for n in ("i", "f"))
    o = oh._r(memory_recurrence(q * m["dim"] ** -0.5, k, v, i, log_sigmoid(f)))
    o = o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps)
    return oh.linear(oh._r(o.reshape(T, -1) * w["norm"] * sigmoid(oh.linear(h, w["g"]))), w["o"])


def parallel(h, w, m, eps):
    left, right = biased_attention(h, oh._sub(w, "left."), m["left"]), matrix_memory(h, oh._sub(w, "right."), m["right"], eps)
    return m["left_scale"] * left + m["right_scale"] * right


MIXERS = {"attention": sigmoid_attention, "parallel": parallel}


def feed_forward(h, w):
    """w: 'up', 'down'."""
    return oh.linear(oh._r(torch.clamp(oh.linear(h, w["up"]), min=0) ** 2), w["down"])


margins: List[float] = []      # smallest gap of every route() call between what was just taken and what was just left out


def route(h, w, correction, r: dict):
    """-> per token [(expert, weight)]: softmax over everything; groups ranked by their best corrected score, members of the kept
    groups by their corrected score, weighted by the plain one."""
    z = h @ w.T
    e = torch.exp(z - z.max(-1, keepdim=True).values)
    s = e / e.sum(-1, keepdim=True)
    choice = s + correction
    n, groups = s.shape[1], r.get("groups") or dict(count=1, keep=1)
    size, keep = n // groups["count"], groups["keep"]
    out = []
    for t in range(h.shape[0]):
        rank = sorted(((max(float(choice[t, e]) for e in range(g * size, (g + 1) * size)), g) for g in range(groups["count"])), key=lambda x: (-x[0], x[1]))
        if keep < len(rank):
            margins.append(rank[keep - 1][0] - rank[keep][0])
        open_ = sorted((e for _, g in rank[:keep] for e in range(g * size, (g + 1) * size)), key=lambda e: (-float(choice[t, e]), e))
        if r["top"] < len(open_):
            margins.append(float(choice[t, open_[r["top"] - 1]] - choice[t, open_[r["top"]]]))
        out.append([(e, s[t, e]) for e in open_[:r["top"]]])
    return out


def moe(h, w, f):
    """Experts 'e0' ..., behind them router.identity identities; 'shared' with 'shared.sg'."""
    out = torch.zeros_like(h)
    real = f["router"]["experts"]
    for t, chosen in enumerate(route(h, w["router"], w["correction"], f["router"])):
        for e, p in chosen:
            out[t] += p * (feed_forward(h[t:t + 1], oh._sub(w, f"e{e}."))[0] if e < real else h[t])
    if f.get("shared"):
        out = out + feed_forward(h, oh._sub(w, "shared.")) * sigmoid(h @ w["shared.sg"].T)
    return out


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=F64):
    """-> (logits [T, vocab], [residual stream behind every layer])."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][torch.tensor(tokens)]
    trace = []
    for i, lay in enumerate(cfg["layers"]):
        p, f = f"l{i}.", lay.get("mlp")
        h = oh._r(token_shift(oh._r(norm(x, w[p + "norm1"], eps)), w[p + "shift"]))
        x = x + m * norm(MIXERS[lay["type"]](h, oh._sub(w, p + "mix."), lay["mixer"], eps), w[p + "norm1b"], eps)
        if f is not None:
            h, sub = oh._r(norm(x, w[p + "norm2"], eps)), oh._sub(w, p + "mlp.")
            x = x + m * norm(moe(h, sub, f) if f["kind"] == "moe" else feed_forward(h, sub), w[p + "norm2b"], eps)
        trace.append(x)
    return oh.linear(oh._r(norm(x, w["final.norm"], eps)), w["head"]), trace


# ---------------------------------------------------------------------------------------------- random models
def tensor_shapes(cfg: dict) -> Dict[str, Tuple[int, ...]]:
    W = cfg["width"]
    out: Dict[str, Tuple[int, ...]] = {"embed": (cfg["vocab"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}

    def feed(prefix, ff):
        out.update({prefix + "up": (ff, W), prefix + "down": (W, ff)})

    for i, lay in enumerate(cfg["layers"]):
        m, f, p = lay["mixer"], lay["mlp"], f"l{i}."
        out.update({p + "norm1": (W,), p + "norm1b": (W,), p + "shift": (W,)})
        if lay["type"] == "attention":
            H, G, D = m["heads"], m["kv_heads"], m["dim"]
            mix = {"q": (H * D, W), "k": (G * D, W), "pb": (H,), "o": (W, H * D)}
        else:
            a, r = m["left"], m["right"]
            rows = {"q": a["heads"] * a["dim"], "k": a["kv_heads"] * a["dim"], "v": a["kv_heads"] * a["vdim"]}
            mix = {f"left.{n}": (c, W) for n, c in rows.items()}
            mix.update({f"left.{n}.b": (c,) for n, c in rows.items()})
            mix.update({"left.o": (W, a["heads"] * a["vdim"]), "left.o.b": (W,)})
            H, D, V = r["heads"], r["dim"], r["vdim"]
            mix.update({f"right.{n}": (c, W) for n, c in (("q", H * D), ("k", H * D), ("v", H * V), ("g", H * V), ("i", H), ("f", H))})
            mix.update({"right.i.b": (H,), "right.f.b": (H,), "right.norm": (H * V,), "right.o": (W, H * V)})
        out.update({p + "mix." + n: s for n, s in mix.items()})
        if f is None:
            continue
        out.update({p + "norm2": (W,), p + "norm2b": (W,)})
        if f["kind"] == "dense":
            feed(p + "mlp.", f["ff"])
            continue
        members = f["router"]["experts"] + f["router"].get("identity", 0)
        for e in range(f["router"]["experts"]):
            feed(f"{p}mlp.e{e}.", f["expert"]["ff"])
        out[p + "mlp.router"], out[p + "mlp.correction"] = (members, W), (members,)
        if f.get("shared"):
            feed(p + "mlp.shared.", f["shared"]["ff"])
            out[p + "mlp.shared.sg"] = (1, W)
    return out


CODE_DIMS, CODES = 8, 12


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """bf16 weights whose every branch matters: matrices keep unit variance, norms make unit rows, offsets, biases and gates are of the size
    of what they join, memories last for tens of tokens, corrections reach below zero.  No token sits between two experts: the first
    CODE_DIMS columns of the embedding hold one of CODES sign patterns, nothing else writes to those columns of the residual or reads
    them, except the routers, which read nothing else and are drawn until the choice of every pattern is clear.  The patterns are large, so
    that the rest of the residual hardly changes what the norm makes of them."""
    g = torch.Generator().manual_seed(seed)
    code = torch.randint(0, 2, (CODES, CODE_DIMS), generator=g) * 2.0 - 1.0
    amplitude = math.sqrt(6.0 * cfg["width"] / CODE_DIMS)     # the patterns add 6 to the mean square of a row, everything else 1 to 5
    shapes, out = tensor_shapes(cfg), {}
    for name, shape in shapes.items():
        r = torch.randn(shape, generator=g)
        last = name.split(".")[-1]
        if last in ("norm1", "norm1b", "norm2", "norm2b", "norm"):
            t = 0.2 * r + 1.0 if name.endswith("right.norm") else 0.2 * r if last.endswith("b") else 1.9 + 0.5 * r
        elif last == "shift":
            t = 0.4 + 0.3 * r
        elif last in ("embed", "pb"):
            t = r
        elif last == "b":
            t = r * 0.5 + (2.5 if name.endswith("f.b") else 0.0)
        elif last == "correction":
            t = r * 0.08 - 0.03
        else:
            t = r / math.sqrt(shape[1])
        if last == "embed":
            t[:, :CODE_DIMS] = code[torch.arange(shape[0]) % CODES] * amplitude
        elif last in ("norm1", "norm1b", "norm2b") or name == "final.norm":
            t[:CODE_DIMS] = -1.0
        elif last == "norm2":
            t[:CODE_DIMS] = 5.8 / amplitude - 1.0
        elif last in ("up", "sg"):
            t[:, :CODE_DIMS] = 0.0
        out[name] = t.to(torch.bfloat16)
    saved = list(margins)
    seen = torch.cat([code * s for s in (1.66, 1.8, 2.0, 2.25)]).double()
    for i, lay in enumerate(cfg["layers"]):
        if lay["mlp"] is None or lay["mlp"]["kind"] != "moe":
            continue
        name, best = f"l{i}.mlp.router", None
        for _ in range(300):
            w = torch.zeros(shapes[name])
            w[:, :CODE_DIMS] = torch.randn((shapes[name][0], CODE_DIMS), generator=g) * 0.4
            w = w.to(torch.bfloat16)
            margins.clear()
            picks = [{e for e, _ in t} for t in route(seen, w[:, :CODE_DIMS].double(), out[f"l{i}.mlp.correction"].double(), lay["mlp"]["router"])]
            changes = sum(p != picks[k % CODES] for k, p in enumerate(picks))
            gap = min(margins, default=1.0) - changes
            if best is None or gap > best[0]:
                best = (gap, w)
            if gap > 0.01:
                break
        out[name] = best[1]
    margins[:] = saved
    return out
