"""Small Zimupel configurations that differ from each other in every size and option, random weights for them, and
helpers to run them through the engine and the plain implementation."""
from __future__ import annotations

import copy
from typing import Dict

import torch

import plain_zimupel as P
from mesolix_cases import make_requests, relative_error  # noqa: F401  (shared test equipment)
from mesolix_cases import assert_matches as _assert_matches
from yalis_amd.config.runtime import EngineConfig
from yalis_amd.engine.factory import build_model, tensor_specs_for
from yalis_amd.engine.step import ModelRunner


def att(heads, kv_heads, dim, vdim, scale, diff, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def lightning(dim, vdim, decay):
    return {"type": "lightning", "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}}


def retention(dim, vdim, decay, rot=None):
    """rot: (dims, base)."""
    m = {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}
    if rot is not None:
        m["rot"] = {"dims": rot[0], "base": rot[1]}
    return {"type": "retention", "mixer": m}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, groups=None):
    """groups: (count, keep)."""
    router = {"experts": experts, "top": top}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "router": router, "expert": {"ff": ff}}


def model(vocab, width, eps, streams, layers, scale=1.0, cap=None):
    out = []
    for layer, mlp in layers:
        entry = copy.deepcopy(layer)
        entry["mlp"] = copy.deepcopy(mlp)
        out.append(entry)
    cfg = {"architecture": "Zimupel", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "logit_scale": scale, "layers": out}
    if cap is not None:
        cfg["logit_softcap"] = cap
    return cfg


CONFIGS = {
    # nothing a multiple of 8; keys shared by groups, values narrower and wider than a map's keys; a layer that reads another's
    # keys with a scale and a share of its own; a rotation of part of the head and none; a decay of one; groups
    # of two experts, no groups, no feed-forward
    "odd": model(70, 42, 1e-5, 3, [
        (att(6, 2, 5, 7, 0.6, 0.35), moe(6, 2, 10, (3, 2))),
        (lightning(7, 5, [0.5, 0.97, 0.9]), dense(29)),
        (att(6, 2, 5, 7, 0.9, 0.1, kv_from=0), None),
        (retention(10, 6, [0.9, 0.995], (6, 50.0)), moe(5, 1, 12)),
        (retention(6, 9, [1.0, 0.95, 0.8]), dense(18)),
    ], scale=0.7, cap=6.0),
    # one stream's worth of everything: a recurrent layer first, one key head, every expert chosen, one group kept of two,
    # a group per head, no cap
    "mix": model(128, 64, 1e-6, 5, [
        (retention(16, 24, [0.99, 0.9], (16, 10000.0)), moe(8, 3, 16, (2, 1))),
        (att(4, 1, 8, 16, 0.3, 0.5), dense(96)),
        (lightning(24, 12, [0.98, 0.8, 0.999, 0.9]), moe(4, 4, 24)),
        (att(3, 3, 12, 8, 0.4, 0.2), None),
        (att(4, 1, 8, 16, 0.2, 0.8, kv_from=1), moe(6, 1, 20, (6, 3))),
    ], scale=1.3),
    # sizes of whole wavefronts (the matrix-core attention with one and with several tokens a tile, the scan's chunks, grouped
    # products in bfloat16)
    "wide": model(200, 128, 1e-6, 2, [
        (att(4, 2, 32, 64, 0.25, 0.3), moe(8, 2, 64, (4, 2))),
        (lightning(64, 32, [0.9, 0.998]), dense(128)),
        (retention(32, 64, [0.97, 0.6, 0.995], (32, 30000.0)), None),
        (att(8, 1, 64, 128, 0.15, 0.5), dense(64)),
        (att(4, 2, 32, 64, 0.4, 0.6, kv_from=0), moe(6, 2, 32, (2, 1))),
    ], scale=0.5, cap=10.0),
}
PAGE = {"odd": 16, "mix": 32, "wide": 64}
# (seeds whose models are steady at most positions, see ``steady``)
SEEDS = {"odd": 30, "mix": 22, "wide": 3}
LENGTHS = {"odd": [1, 23, 50, 9, 37, 64], "mix": [70, 3, 41, 129, 18], "wide": [150, 40, 97, 2, 200]}


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """Float32 weights by tensor name; values that bfloat16 holds exactly, so that both engines and the plain
    implementation read the same numbers."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, spec in tensor_specs_for(cfg).items():
        last = name.rsplit(".", 1)[-1]
        offset = 0.0
        if last.startswith("norm"):
            std, offset = 0.3, 1.0
        elif ".hc" in name:
            std, offset = 0.15, {"in": 0.6, "out": 1.0, "mix": 0.0}[last]
            if last == "mix":
                offset = 0.8 * torch.eye(spec.shape[0])
        elif last in ("lq1", "lk1", "lq2", "lk2"):
            std = 0.6 / spec.shape[0] ** 0.25
        elif last == "b":
            std = 0.4
        elif last == "correction":
            std = 0.3
        elif last == "router":
            std = 2.0 / spec.shape[-1] ** 0.5
        elif name == "embed":
            std = 1.0
        elif last in ("o", "down"):  # (what a branch adds stays below what it is added to)
            std = 0.4 / (spec.shape[-1] ** 0.5)
        else:
            std = 1.5 / (spec.shape[-1] ** 0.5)
        out[name] = (torch.randn(spec.shape, generator=g) * std + offset).to(torch.bfloat16).float()
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
STEADY = 0.06
# and how far apart the last chosen expert (group) and the best one left out must be
CLEAR_CALL = 0.03


def router_gaps(cfg, weights, toks) -> torch.Tensor:
    P.ROUTER_GAPS = seen = []
    try:
        P.forward(weights, cfg, toks)
    finally:
        P.ROUTER_GAPS = None
    return torch.tensor(seen, dtype=torch.float64).view(-1, len(toks)).min(0).values if seen else torch.full((len(toks),), float("inf"), dtype=torch.float64)


def steady(want: Wanted) -> Dict[str, torch.Tensor]:
    """Which positions a bfloat16 engine can be held to: those whose routers' choices are no close calls, and whose logits
    barely move when every layer's input is disturbed by a few times its rounding (a read-out or a difference of two
    maps that is divided by its own root mean square can hang on a rounding where it happens to be small)."""
    cfg, weights, reqs = want.made_of
    layer = P.run_layer
    keep = {rid: router_gaps(cfg, weights, toks) >= CLEAR_CALL for rid, toks in reqs.items()}
    for seed in (1, 2, 3, 4):
        g = torch.Generator().manual_seed(seed)
        P.run_layer = lambda W, c, i, X, caches: layer(W, c, i, X * (1.0 + 2.0 ** -7 * (2.0 * torch.rand(X.shape, generator=g, dtype=torch.float64) - 1.0)), caches)
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
        assert share >= 0.5, f"{what}: only {share:.0%} of the positions can be compared in bfloat16"
        _assert_matches(got, want, True, what, {rid: torch.where(k, float("inf"), 0.0) for rid, k in keep.items()})
        return
    _assert_matches(got, want, bf16, what)
