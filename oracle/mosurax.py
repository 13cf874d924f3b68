"""Plain, slow evaluation of the Mosurax design: a looped decoder with learned positions whose layers are windowed grouped-query
attention with a sink and an output gate, behind dense or routed feed-forward parts.  One function per mechanism, every
attention row one explicit softmax over its visible keys, every token's experts one by one; nothing is shared with the
product path.

`weights` maps tensor names to tensors; everything is computed in `dtype` (float64 unless told otherwise) on the CPU.  A whole
sequence goes in, logits and the residual stream behind every executed layer come out: there is no cache here, so prefill,
portions and token-by-token decoding of the product are all compared against the same rows.  `oracle.hybrid.rounding` applies."""
from __future__ import annotations

import math
from typing import Dict, List, Tuple

import torch

from . import hybrid as oh

F64 = torch.float64


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def sink_softmax(s):
    """exp(s_j) / (1 + sum exp(s)) along the last dimension: a key of score 0 that carries no value."""
    m = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def windowed_attention(q, k, v, window, scale):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H, V]; position i sees the `window` positions up to and with itself."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    o = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for i in range(T):
        lo = max(0, i - window + 1)
        for h in range(H):
            p = sink_softmax(k[lo:i + 1, h // per] @ q[i, h] * scale)
            o[i, h] = p @ v[lo:i + 1, h // per]
    return o


def attention_mixer(h, w, m):
    """w: 'q', 'k', 'v', 'g', 'o'; m: the mixer's sizes."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = oh.linear(h, w["q"]).view(T, H, m["dim"])
    k = oh.linear(h, w["k"]).view(T, G, m["dim"])
    v = oh.linear(h, w["v"]).view(T, G, m["vdim"])
    o = windowed_attention(q, k, v, m["mask"]["size"], m["scale"]).reshape(T, -1)
    return oh.linear(oh._r(o * sigmoid(oh.linear(h, w["g"]))), w["o"])


def gated_mlp(h, gate, up, down):
    return oh.linear(oh._r(oh.silu(oh.linear(h, gate)) * oh.linear(h, up)), down)


margins: List[float] = []      # smallest gap of every route() call between the last expert taken and the first one left out


def route(h, w, b, top):
    """The `top` largest of the logits w h + b per token and the softmax over those alone -> (weights, experts) [T, top]."""
    z, e = torch.sort(h @ w.T + b, dim=-1, descending=True)
    if top < z.shape[1]:
        margins.append(float((z[:, top - 1] - z[:, top]).min()))
    return torch.softmax(z[:, :top], -1), e[:, :top]


def moe_mlp(h, w, m):
    """w: 'router', 'router.b', 'e<i>.gate' ..., 'shared.gate' ... when there is a shared expert."""
    p, e = route(h, w["router"], w["router.b"], m["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for i in range(e.shape[1]):
            x = f"e{int(e[t, i])}."
            out[t] += p[t, i] * gated_mlp(h[t:t + 1], w[x + "gate"], w[x + "up"], w[x + "down"])[0]
    if m.get("shared"):
        out = out + gated_mlp(h, w["shared.gate"], w["shared.up"], w["shared.down"])
    return out


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def forward(cfg: dict, weights: Dict[str, torch.Tensor], tokens: List[int], dtype=F64):
    """-> (logits [T, vocab], [residual stream behind every executed layer])."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x0 = w["embed"][torch.tensor(tokens, dtype=torch.int64)] + w["pos"][:len(tokens)]
    x, trace = x0, []

    def norm(name):
        return oh._r(oh.rms_norm(x, w[name], eps))

    for i, t in oh.run_order(cfg):
        lay, p = cfg["layers"][i], f"l{i}."
        if t is not None:
            x = (x + x0 if t > 0 else x) + w["loop.step"][t]
        x = x + attention_mixer(norm(p + "norm1"), oh._sub(w, p + "mix."), lay["mixer"])
        if lay["mlp"] is not None:
            h, sub = norm(p + "norm2"), oh._sub(w, p + "mlp.")
            x = x + (moe_mlp(h, sub, lay["mlp"]) if lay["mlp"]["kind"] == "moe" else gated_mlp(h, sub["gate"], sub["up"], sub["down"]))
        trace.append(x)
    logits = oh.linear(norm("final.norm"), w["head"])
    return (soft_cap(logits, cfg["logit_softcap"]) if cfg.get("logit_softcap") else logits), trace


# ---------------------------------------------------------------------------------------------- random models
def tensor_shapes(cfg: dict) -> Dict[str, Tuple[int, ...]]:
    W = cfg["width"]
    out: Dict[str, Tuple[int, ...]] = {"embed": (cfg["vocab"], W), "pos": (cfg["max_positions"], W), "head": (cfg["vocab"], W), "final.norm": (W,)}
    if cfg.get("loop"):
        out["loop.step"] = (cfg["loop"]["times"], W)

    def mlp(prefix, ff):
        out.update({prefix + "gate": (ff, W), prefix + "up": (ff, W), prefix + "down": (W, ff)})

    for i, lay in enumerate(cfg["layers"]):
        m, f, p = lay["mixer"], lay["mlp"], f"l{i}."
        H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        out[p + "norm1"] = (W,)
        out.update({p + "mix." + n: s for n, s in (("q", (H * D, W)), ("k", (G * D, W)), ("v", (G * V, W)), ("g", (H * V, W)), ("o", (W, H * V)))})
        if f is None:
            continue
        out[p + "norm2"] = (W,)
        if f["kind"] == "dense":
            mlp(p + "mlp.", f["ff"])
            continue
        for e in range(f["router"]["experts"]):
            mlp(f"{p}mlp.e{e}.", f["expert"]["ff"])
        out[p + "mlp.router"], out[p + "mlp.router.b"] = (f["router"]["experts"], W), (f["router"]["experts"],)
        if f.get("shared"):
            mlp(p + "mlp.shared.", f["shared"]["ff"])
    return out


CODE_DIMS, CODES = 8, 12


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """bf16 weights whose every branch matters: matrices keep unit variance, norms spread around 1.  No token sits between two
    experts: the first CODE_DIMS columns of the embedding hold one of CODES sign patterns, nothing else writes to those columns of
    the residual, and the routers read only them, drawn until every pattern's choice is clear."""
    g = torch.Generator().manual_seed(seed)
    code = torch.randint(0, 2, (CODES, CODE_DIMS), generator=g) * 4.0 - 2.0
    shapes, out = tensor_shapes(cfg), {}
    for name, shape in shapes.items():
        r = torch.randn(shape, generator=g)
        last = name.split(".")[-1]
        if last in ("norm1", "norm2", "norm"):
            t = 1.0 + 0.2 * r
        elif last in ("embed", "pos"):
            t = r
        elif last in ("step", "b"):
            t = r * 0.5
        else:
            t = r / math.sqrt(shape[1])
        if last == "embed":
            t[:, :CODE_DIMS] = code[torch.arange(shape[0]) % CODES]
        elif last in ("pos", "step"):
            t[:, :CODE_DIMS] = 0.0
        elif last in ("o", "down"):
            t[:CODE_DIMS] = 0.0
        out[name] = t.to(torch.bfloat16)
    for name in (n for n in shapes if n.endswith(".router")):
        top, best = next(lay["mlp"]["router"]["top"] for i, lay in enumerate(cfg["layers"]) if name.startswith(f"l{i}.")), None
        c = code * out[name.replace("mlp.router", "norm2")][:CODE_DIMS].float()
        for _ in range(200):
            w = torch.zeros(shapes[name])
            w[:, :CODE_DIMS] = torch.randn((shapes[name][0], CODE_DIMS), generator=g)
            gap = float("inf")
            for s in (0.3, 0.6, 1.0):
                z = torch.sort(s * c @ w[:, :CODE_DIMS].T + out[name + ".b"].float(), dim=-1, descending=True).values
                if top < z.shape[1]:
                    gap = min(gap, float((z[:, top - 1] - z[:, top]).min()))
            if best is None or gap > best[0]:
                best = (gap, w)
        out[name] = best[1].to(torch.bfloat16)
    return out
