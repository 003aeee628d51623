"""Small Rafusun configurations that differ from each other in every size and option, random weights for them, and
helpers to run them through the engine and the plain implementation."""
from __future__ import annotations

import copy
from typing import Dict

import torch

import plain_rafusun as P
from mesolix_cases import make_requests, relative_error  # noqa: F401  (shared test equipment)
from mesolix_cases import assert_matches as _assert_matches
from yalis_amd.config.runtime import EngineConfig
from yalis_amd.engine.factory import build_model, tensor_specs_for
from yalis_amd.engine.step import ModelRunner


def delta(heads, kv_heads, dim, vdim, conv):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def both(left, right):
    return {"type": "parallel", "mixer": {"left": left, "right": right}}


def att(heads, kv_heads, dim, vdim, scale, chunk=None, softcap=None, rot=None):
    """rot: (dims, base)."""
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk is not None:
        m["mask"] = {"size": chunk}
    if softcap is not None:
        m["softcap"] = softcap
    if rot is not None:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
    return m


def mixing(heads, dim):
    return {"heads": heads, "dim": dim}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def model(vocab, width, eps, alpha, layers, scale=1.0, bigram=None):
    out = []
    for layer, mlp in layers:
        entry = copy.deepcopy(layer)
        entry["mlp"] = copy.deepcopy(mlp)
        out.append(entry)
    embedding = {"scale": scale}
    if bigram is not None:
        embedding["bigram"] = {"buckets": bigram[0], "mul_prev": bigram[1], "mul_cur": bigram[2]}
    return {"architecture": "Rafusun", "vocab": vocab, "width": width, "postln_alpha": alpha, "norm": {"eps": eps},
            "embedding": embedding, "layers": out}


# what the ranks of the low-rank pairs are in the random weights (config.json does not name them)
RANKS = {"odd": (3, 5, 7), "mix": (16, 8, 12), "wide": (24, 40, 32)}  # (a1, g1, w1)

CONFIGS = {
    # nothing a multiple of 8; key heads shared by groups and values wider than keys in the delta rule; a chunk that is no
    # multiple of anything; values narrower than keys; a rotation of part of the head; layers with and without
    # feed-forward of both kinds; more pairs' buckets than tokens
    "odd": model(70, 42, 1e-5, 1.7, [
        (both(att(6, 2, 10, 6, 0.6, 11, 4.0, (6, 50.0)), mixing(3, 7)), dense(29)),
        (delta(4, 2, 6, 9, 3), None),
        (delta(3, 3, 10, 5, 1), dense(30)),
        (both(att(3, 3, 8, 12, 0.4, 20), mixing(2, 10)), None),
    ], scale=3.0, bigram=(211, 17, 5)),
    # one key head; no chunk, no cap, the whole head rotates; two chunk sizes; a pairs' table of one bucket only
    "mix": model(128, 64, 1e-6, 4.0, [
        (delta(2, 1, 16, 8, 5), dense(96)),
        (both(att(4, 1, 16, 16, 0.3, 32, 20.0, (16, 10000.0)), mixing(2, 32)), None),
        (both(att(2, 2, 24, 8, 0.5, None, None, (8, 300.0)), mixing(4, 8)), dense(64)),
        (delta(4, 4, 8, 24, 2), None),
        (both(att(4, 2, 16, 16, 0.4, 7, 9.0), mixing(1, 24)), dense(40)),
    ], scale=1.0, bigram=(1, 3, 1)),
    # sizes of whole wavefronts (the matrix-core attention, grouped and tiled products in bfloat16); chunks that end
    # inside pages and blocks of keys
    "wide": model(200, 128, 1e-6, 2.5, [
        (both(att(4, 2, 64, 64, 0.9, 100, 25.0, (32, 30000.0)), mixing(4, 64)), dense(256)),
        (delta(4, 2, 64, 32, 4), dense(128)),
        (both(att(2, 1, 128, 128, 1.1, 48, 50.0, (64, 10000.0)), mixing(2, 64)), None),
    ], scale=8.0, bigram=(97, 1000003, 7919)),
}
PAGE = {"odd": 16, "mix": 32, "wide": 64}
LENGTHS = {"odd": [1, 23, 50, 9, 37, 64], "mix": [70, 3, 41, 129, 18], "wide": [150, 40, 97, 2, 230]}


def random_weights(cfg: dict, seed: int, ranks=(16, 8, 12)) -> Dict[str, torch.Tensor]:
    """Float32 weights by tensor name; values that bfloat16 holds exactly, so that both engines and the plain
    implementation read the same numbers."""
    g = torch.Generator().manual_seed(seed)
    rank = dict(zip(("a", "g", "w"), ranks))
    out = {}
    for name, spec in tensor_specs_for(cfg).items():
        last = name.rsplit(".", 1)[-1]
        shape = list(spec.shape)
        if last in ("a1", "g1", "w1"):
            shape[0] = rank[last[0]]
        if last in ("a2", "g2", "w2"):
            shape[1] = rank[last[0]]
        offset = 0.0
        if last.startswith(("norm", "ls")) or last == "out":
            std, offset = 0.3, 1.0  # plain weights
        elif last == "conv":
            std = 0.5
        elif last in ("A_log", "dt_bias"):
            std, offset = 0.7, -1.0
        elif last == "w0":
            std, offset = 1.0, -1.0
        elif ".mu." in name:
            std, offset = 0.4, 0.5
        elif last == "u":
            std = 0.7
        elif name == "bigram":
            std = 0.7
        elif name == "embed":
            std = 1.0 / float(cfg["embedding"]["scale"])
        else:
            std = 1.5 / (shape[-1] ** 0.5)
        out[name] = (torch.randn(shape, generator=g) * std + offset).to(torch.bfloat16).float()
    return out


def make_runner(cfg, weights, dtype, device, ops, page_size, num_pages, max_seqs=4, max_len=512) -> ModelRunner:
    eng = EngineConfig(page_size=page_size, num_pages=num_pages, max_num_seqs=max_seqs, max_model_len=max_len,
                       max_num_batched_tokens=max_len, dtype=dtype, device=device)
    m = build_model(cfg, eng, ops=ops)
    wd = torch.float32 if dtype == "float32" else torch.bfloat16
    m.load({k: v.to(wd).to(device) for k, v in weights.items()})
    return ModelRunner(m, eng)


class Wanted(dict):
    """The plain logits by request, and what they were made of (for ``steady``)."""

    def __init__(self, logits, cfg, weights, reqs):
        super().__init__(logits)
        self.made_of = (cfg, weights, reqs)


def plain_logits(cfg, weights, reqs) -> Wanted:
    return Wanted({rid: P.forward(weights, cfg, toks) for rid, toks in reqs.items()}, cfg, weights, reqs)


# how far roundings of the size of bfloat16's may move a position's logits for it to be compared in bfloat16
STEADY = 0.04


def steady(want: Wanted) -> Dict[str, torch.Tensor]:
    """Which positions a bfloat16 engine can be held to.  A recurrence's read-out is divided by its own root mean square,
    so where the query happens to be nearly at right angles to all that a memory holds (a sequence's first tokens, small
    heads) a rounding decides its direction.  Every layer's input is disturbed by as much as its rounding would (twice),
    and positions whose logits then move by more than ``STEADY`` are left out."""
    cfg, weights, reqs = want.made_of
    layer = P.run_layer
    keep = {rid: torch.ones(len(toks), dtype=torch.bool) for rid, toks in reqs.items()}
    for seed in (1, 2):
        g = torch.Generator().manual_seed(seed)
        P.run_layer = lambda W, c, i, x: layer(W, c, i, x * (1.0 + 2.0 ** -8 * (2.0 * torch.rand(x.shape, generator=g, dtype=torch.float64) - 1.0)))
        try:
            for rid, toks in reqs.items():
                keep[rid] &= relative_error(P.forward(weights, cfg, toks), want[rid]) <= STEADY
        finally:
            P.run_layer = layer
    return keep


def assert_matches(got, want, bf16: bool, what: str) -> None:
    if bf16 and isinstance(want, Wanted):
        keep = steady(want)
        share = sum(int(k.sum()) for k in keep.values()) / sum(len(k) for k in keep.values())
        assert share >= 0.6, f"{what}: only {share:.0%} of the positions can be compared in bfloat16"
        _assert_matches(got, want, True, what, {rid: torch.where(k, float("inf"), 0.0) for rid, k in keep.items()})
        return
    _assert_matches(got, want, bf16, what)
