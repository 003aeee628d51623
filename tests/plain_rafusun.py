"""Rafusun, plainly: whole sequences in float64, a python loop over tokens for both recurrences and over queries and
heads for the attention.  One function per mechanism, written from the design's equations; it shares nothing with the
engine (which keeps pages and state slots, runs ragged batches and fuses steps).

``weights`` maps tensor names to tensors; ``cfg`` is the config.json dictionary.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F = torch.float64
UNIT_EPS = 1e-6


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def stream_norm(x, w, eps):
    return rms(x, eps) * w


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ------------------------------------------------------------------------------------------------------ embedding
def bigram_row(previous: Optional[int], token: int, b: dict) -> int:
    """The row of the pair (previous token, token); a sequence's first token has the row after the last bucket."""
    if previous is None:
        return int(b["buckets"])
    return (previous * int(b["mul_prev"]) + token * int(b["mul_cur"])) % int(b["buckets"])


def embedding(W, cfg, tokens):
    e = cfg.get("embedding") or {}
    x = W["embed"][torch.tensor(tokens)] * float(e.get("scale", 1.0))
    if e.get("bigram") is not None:
        rows = [bigram_row(None if i == 0 else tokens[i - 1], t, e["bigram"]) for i, t in enumerate(tokens)]
        x = x + W["bigram"][torch.tensor(rows)]
    return x


# -------------------------------------------------------------------------------------------------- channel_delta
def short_convolution(x, w):
    """x [n, channels], w [channels, taps]; silu on the sum; zeros before the start."""
    n, taps = x.shape[0], w.shape[1]
    out = torch.zeros_like(x)
    for t in range(n):
        for j in range(taps):
            back = taps - 1 - j
            if t >= back:
                out[t] += w[:, j] * x[t - back]
    return silu(out)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + UNIT_EPS)


def channel_decay(W, p: str, H: int, d: int, h):
    """[n, H, d], in (0, 1)."""
    z = (h @ W[p + "a1"].T) @ W[p + "a2"].T + W[p + "dt_bias"]
    return torch.exp(-torch.exp(W[p + "A_log"])[None, :, None] * softplus(z).view(h.shape[0], H, d))


def delta_scan(q, k, v, beta, g):
    """q, k [n, H, d]; v [n, H, e]; beta [n, H]; g [n, H, d].  Decay, then write what the memory lacks, then read."""
    n, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=F)
    out = torch.zeros(n, H, v.shape[-1], dtype=F)
    for t in range(n):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hde,hd->he", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = torch.einsum("hde,hd->he", S, q[t])
    return out


def channel_delta(W, p: str, m: dict, eps: float, h):
    n, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    conv = lambda name: short_convolution(h @ W[p + name].T, W[p + name + ".conv"])
    q, k, v = conv("q").view(n, G, d), conv("k").view(n, G, d), conv("v").view(n, H, e)
    share = torch.arange(H) // (H // G)
    q, k = unit(q)[:, share] * d ** -0.5, unit(k)[:, share]
    beta = torch.sigmoid(h @ W[p + "b"].T)
    o = delta_scan(q, k, v, beta, channel_decay(W, p, H, d, h))
    gate = torch.sigmoid((h @ W[p + "g1"].T) @ W[p + "g2"].T).view(n, H, e)
    return (rms(o, eps) * W[p + "norm"] * gate).reshape(n, H * e) @ W[p + "o"].T


# ---------------------------------------------------------------------------------------------- parallel: the left
# when a list: for every query and head of every attention, (query, head, the key with the largest weight, that
# weight, what the sink takes) is appended
ATTENTION_PEAKS: Optional[list] = None


def rotate(x, rot: dict):
    """x [n, heads, dim]: the first dims elements of every head turn, neighbours (2i, 2i + 1) together."""
    n, dims, base = x.shape[0], int(rot["dims"]), float(rot["base"])
    out = x.clone()
    pos = torch.arange(n, dtype=F)
    for i in range(dims // 2):
        a = pos * base ** (-2.0 * i / dims)
        c, s = torch.cos(a)[:, None], torch.sin(a)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i], out[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def first_visible(i: int, mask: Optional[dict]) -> int:
    """The first key that the query at position i sees: its chunk's first position."""
    return 0 if mask is None else i // int(mask["size"]) * int(mask["size"])


def sink_softmax(s):
    """exp(s_j) / (1 + sum exp(s)): a sink of score 0 without a value."""
    top = max(float(s.max()), 0.0)
    e = torch.exp(s - top)
    return e / (math.exp(-top) + e.sum())


def chunked_attention(W, p: str, m: dict, eps: float, h):
    n, H, G, d, e = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ W[p + "q"].T).view(n, H, d)
    k = (h @ W[p + "k"].T).view(n, G, d)
    v = (h @ W[p + "v"].T).view(n, G, e)
    if m.get("rot") is not None:
        q, k = rotate(q, m["rot"]), rotate(k, m["rot"])
    q, k = rms(q, eps), rms(k, eps)
    cap = m.get("softcap")
    out = torch.zeros(n, H, e, dtype=F)
    for i in range(n):
        lo = first_visible(i, m.get("mask"))
        for hd in range(H):
            g = hd // (H // G)
            s = (k[lo: i + 1, g] @ q[i, hd]) * m["scale"]
            if cap:
                s = cap * torch.tanh(s / cap)
            w = sink_softmax(s)
            out[i, hd] = w @ v[lo: i + 1, g]
            if ATTENTION_PEAKS is not None:
                ATTENTION_PEAKS.append((i, hd, lo + int(torch.argmax(w)), float(w.max()), 1.0 - float(w.sum())))
    return out.reshape(n, H * e) @ W[p + "o"].T


# --------------------------------------------------------------------------------------------- parallel: the right
def token_before(h):
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def bonus_scan(r, k, v, w, u):
    """r, k, w [n, H, d]; v [n, H, e]; u [H, d].  Read the memory as it was plus the token's own write weighed by u;
    then decay and write."""
    n, H, d = r.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=F)
    out = torch.zeros(n, H, v.shape[-1], dtype=F)
    for t in range(n):
        kv = k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hde,hd->he", S + u[:, :, None] * kv, r[t])
        S = w[t][:, :, None] * S + kv
    return out


def time_mixing(W, p: str, m: dict, eps: float, h):
    n, H, d = h.shape[0], m["heads"], m["dim"]
    past = token_before(h)
    mix = lambda s: h + (past - h) * W[p + "mu." + s]
    r, k, v = ((mix(s) @ W[p + s].T).view(n, H, d) for s in ("r", "k", "v"))
    gate = silu(mix("g") @ W[p + "g"].T)
    z = torch.tanh(mix("w") @ W[p + "w1"].T) @ W[p + "w2"].T + W[p + "w0"]
    w = torch.exp(-torch.exp(z)).view(n, H, d)
    o = bonus_scan(r, k, v, w, W[p + "u"])
    return (rms(o, eps).reshape(n, H * d) * W[p + "norm"] * gate) @ W[p + "o"].T


def parallel(W, p: str, m: dict, eps: float, h):
    left = chunked_attention(W, p + "left.", m["left"], eps, h)
    right = time_mixing(W, p + "right.", m["right"], eps, h)
    return 0.5 * (rms(left, eps) * W[p + "left.out"] + rms(right, eps) * W[p + "right.out"])


# ------------------------------------------------------------------------------------------------------- the model
def gated_ff(W, p: str, h):
    return (gelu_tanh(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def run_layer(W, cfg: dict, i: int, x):
    layer, eps, alpha, p = cfg["layers"][i], float(cfg["norm"]["eps"]), float(cfg["postln_alpha"]), f"l{i}."
    b = globals()[layer["type"]](W, p + "mix.", layer["mixer"], eps, x)
    x = stream_norm(alpha * x + b * W[p + "ls1"], W[p + "norm1"], eps)
    if layer.get("mlp") is not None:
        b = gated_ff(W, p + "mlp.", x)
        x = stream_norm(alpha * x + b * W[p + "ls2"], W[p + "norm2"], eps)
    return x


@torch.no_grad()
def forward(weights: Dict[str, torch.Tensor], cfg: dict, tokens: List[int], streams: Optional[list] = None):
    """Logits [n, vocab], float64.  ``streams``: the residual stream after every layer is appended to it."""
    W = {k: v.to(F) for k, v in weights.items()}
    x = embedding(W, cfg, tokens)
    for i in range(len(cfg["layers"])):
        x = run_layer(W, cfg, i, x)
        if streams is not None:
            streams.append(x.clone())
    return stream_norm(x, W["final.norm"], float(cfg["norm"]["eps"])) @ W["head"].T
