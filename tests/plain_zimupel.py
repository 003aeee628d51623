"""Zimupel, plainly: whole sequences in float64, a python loop over tokens for both recurrences, over queries, heads and
maps for the attention, over tokens and experts for the mixture.  One function per mechanism, written from the design's
equations; it shares nothing with the engine (which keeps pages and state slots, runs ragged batches and fuses steps).

``weights`` maps tensor names to tensors; ``cfg`` is the config.json dictionary.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F = torch.float64


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def stream_norm(x, w, eps):
    return rms(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ------------------------------------------------------------------------------------------------------ embedding
def embedding(W, eps, tokens):
    return stream_norm(W["embed"][torch.tensor(tokens)], W["embed.norm"], eps)


# ------------------------------------------------------------------------------------------- streams in place of one
def read_streams(X, w):
    """X [n, streams, width]: what a branch reads, sum_s w_s x_s."""
    return torch.einsum("s,nsc->nc", w, X)


def write_streams(X, mix, out, y):
    """Every stream from all the old ones and the branch's output: x_t <- sum_s mix[s, t] x_s + out[t] y."""
    return torch.einsum("st,nsc->ntc", mix, X) + out[None, :, None] * y[:, None, :]


# ---------------------------------------------------------------------------------------- a memory with a fixed decay
def rotate(x, rot: Optional[dict]):
    """x [n, heads, dim]: of every head's first ``dims`` elements, i and i + dims / 2 turn together."""
    if rot is None:
        return x
    n, dims, base = x.shape[0], int(rot["dims"]), float(rot["base"])
    out = x.clone()
    pos = torch.arange(n, dtype=F)
    for i in range(dims // 2):
        a = pos * base ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., i], x[..., i + dims // 2]
        out[..., i], out[..., i + dims // 2] = u * c - v * s, v * c + u * s
    return out


def fixed_decay_scan(q, k, v, decay):
    """q, k [n, H, d]; v [n, H, e]; decay [H].  Decay, write, then read."""
    n, H, d = q.shape
    a = torch.tensor(decay, dtype=F)[:, None, None]
    S = torch.zeros(H, d, v.shape[-1], dtype=F)
    out = torch.zeros(n, H, v.shape[-1], dtype=F)
    for t in range(n):
        S = a * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hde,hd->he", S, q[t])
    return out


def retention(W, p: str, m: dict, eps: float, h, cache):
    n, H, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = (h @ W[p + "q"].T).view(n, H, d), (h @ W[p + "k"].T).view(n, H, d), (h @ W[p + "v"].T).view(n, H, e)
    q, k = rotate(q, m.get("rot")), rotate(k, m.get("rot")) * d ** -0.5
    o = rms(fixed_decay_scan(q, k, v, m["decay"]), eps).reshape(n, H * e)
    return (o * silu(h @ W[p + "g"].T)) @ W[p + "o"].T


def lightning(W, p: str, m: dict, eps: float, h, cache):
    n, H, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k, v = (silu(h @ W[p + s].T).view(n, H, w) for s, w in (("q", d), ("k", d), ("v", e)))
    o = fixed_decay_scan(q, k, v, m["decay"]).reshape(n, H * e)
    return (rms(o, eps) * W[p + "norm"] * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


# ------------------------------------------------------------------------------------------ attention with two maps
# when a list: for every query, head and map of every attention, (query, head, map, the key with the largest weight,
# that weight) is appended
ATTENTION_PEAKS: Optional[list] = None


def keys_and_values(W, p: str, m: dict, h):
    n, G = h.shape[0], m["kv_heads"]
    k = (h @ W[p + "k"].T + W[p + "k.b"]).view(n, G, 2, m["dim"])
    v = (h @ W[p + "v"].T + W[p + "v.b"]).view(n, G, m["vdim"])
    return k, v


def map_weight(W, p: str, m: dict) -> float:
    """lambda: what the second map's output is taken off with."""
    first = float((W[p + "lq1"] * W[p + "lk1"]).sum())
    second = float((W[p + "lq2"] * W[p + "lk2"]).sum())
    return math.exp(first) - math.exp(second) + float(m["diff"])


def combine_maps(a1, a2, lam: float, diff: float, eps: float):
    return rms(a1 - lam * a2, eps) * (1.0 - diff)


def attention(W, p: str, m: dict, eps: float, h, cache):
    """``cache``: layer number -> its keys and values (this layer's own are put there by the caller)."""
    n, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    k, v = cache["kv"]
    q = (h @ W[p + "q"].T + W[p + "q.b"]).view(n, H, 2, d)
    out = torch.zeros(2, n, H, e, dtype=F)
    for i in range(n):
        for hd in range(H):
            g = hd // (H // G)
            for which in range(2):
                w = torch.softmax((k[: i + 1, g, which] @ q[i, hd, which]) * m["scale"], dim=0)
                out[which, i, hd] = w @ v[: i + 1, g]
                if ATTENTION_PEAKS is not None:
                    ATTENTION_PEAKS.append((i, hd, which, int(torch.argmax(w)), float(w.max())))
    o = combine_maps(out[0], out[1], map_weight(W, p, m), float(m["diff"]), eps)
    return o.reshape(n, H * e) @ W[p + "o"].T


# --------------------------------------------------------------------------------------------------- feed-forwards
# when a list: per layer and token, the smaller of two gaps between choice scores: the last chosen expert's and the
# best other one's (among those that may be chosen), and the last kept group's and the best dropped one's
ROUTER_GAPS: Optional[list] = None


def kept_experts(choice, groups: Optional[dict]) -> List[int]:
    """The experts that may be chosen: those of the groups whose two largest choice scores sum highest."""
    n = choice.shape[0]
    if groups is None:
        return list(range(n))
    size = n // int(groups["count"])
    score = [float(torch.topk(choice[g * size: (g + 1) * size], min(2, size)).values.sum()) for g in range(int(groups["count"]))]
    order = sorted(range(len(score)), key=lambda g: -score[g])
    keep = sorted(order[: int(groups["keep"])])
    if ROUTER_GAPS is not None and len(keep) < len(order):
        ROUTER_GAPS[-1] = min(ROUTER_GAPS[-1], score[order[len(keep) - 1]] - score[order[len(keep)]])
    return [g * size + i for g in keep for i in range(size)]


def route(W, p: str, f: dict, x):
    """[(expert, weight)] of one token."""
    r = f["router"]
    s = torch.sigmoid(W[p + "router"] @ x)
    choice = s + W[p + "correction"]
    if ROUTER_GAPS is not None:
        ROUTER_GAPS.append(math.inf)
    allowed = kept_experts(choice, r.get("groups"))
    order = sorted(allowed, key=lambda e: -float(choice[e]))
    top = order[: int(r["top"])]
    if ROUTER_GAPS is not None and len(order) > len(top):
        ROUTER_GAPS[-1] = min(ROUTER_GAPS[-1], float(choice[top[-1]] - choice[order[len(top)]]))
    total = float(s[top].sum()) + 1e-20
    return [(e, float(s[e]) / total) for e in top]


def expert(W, p: str, x):
    return W[p + "down"] @ (silu(W[p + "gate"] @ x) * (W[p + "up"] @ x))


def mixture(W, p: str, f: dict, h):
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, w in route(W, p, f, h[t]):
            out[t] += w * expert(W, f"{p}e{e}.", h[t])
    return out


def dense(W, p: str, f: dict, h):
    return (gelu_tanh(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


# ------------------------------------------------------------------------------------------------------- the model
def run_layer(W, cfg: dict, i: int, X, caches: dict):
    layer, eps, p = cfg["layers"][i], float(cfg["norm"]["eps"]), f"l{i}."
    kind, m = layer["type"], layer["mixer"]
    h = stream_norm(read_streams(X, W[p + "hc1.in"]), W[p + "norm1"], eps)
    cache = {}
    if kind == "attention":
        source = m.get("kv_from")
        if source is None:
            caches[i] = keys_and_values(W, p + "mix.", m, h)
        cache["kv"] = caches[i if source is None else int(source)]
    y = globals()[kind](W, p + "mix.", m, eps, h, cache)
    X = write_streams(X, W[p + "hc1.mix"], W[p + "hc1.out"], y)
    f = layer.get("mlp")
    if f is not None:
        h = stream_norm(read_streams(X, W[p + "hc2.in"]), W[p + "norm2"], eps)
        y = (dense if f["kind"] == "dense" else mixture)(W, p + "mlp.", f, h)
        X = write_streams(X, W[p + "hc2.mix"], W[p + "hc2.out"], y)
    return X


def finish_logits(z, scale: float, cap: Optional[float]):
    z = z * scale
    return z if not cap else cap * torch.tanh(z / cap)


@torch.no_grad()
def forward(weights: Dict[str, torch.Tensor], cfg: dict, tokens: List[int], streams: Optional[list] = None):
    """Logits [n, vocab], float64.  ``streams``: the sum of the streams after every layer is appended to it."""
    W = {k: v.to(F) for k, v in weights.items()}
    eps = float(cfg["norm"]["eps"])
    x = embedding(W, eps, tokens)
    X = x[:, None, :].repeat(1, int(cfg["streams"]), 1)
    caches: dict = {}
    for i in range(len(cfg["layers"])):
        X = run_layer(W, cfg, i, X, caches)
        if streams is not None:
            streams.append(X.sum(1))
    z = stream_norm(X.sum(1), W["final.norm"], eps) @ W["head"].T
    return finish_logits(z, float(cfg.get("logit_scale", 1.0)), cfg.get("logit_softcap"))
