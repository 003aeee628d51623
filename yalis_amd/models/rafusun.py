"""Rafusun: a small decoder whose config.json lists its layers one by one, each with one of two mixers and an
optional dense feed-forward, in blocks that norm the stream after every sum.

What the design fixes (everything else is read from config.json or a tensor's shape):
  * the stream starts as embed[token] * embedding.scale plus a row for the pair (token before, token) of the table
    "bigram": row (before * mul_prev + token * mul_cur) mod buckets, the last row for a sequence's first token;
  * a layer is  x = norm1(a x + ls1 * mixer(x));  x = norm2(a x + ls2 * ff(x))  with a = ``postln_alpha``, RMS norms
    with a plain weight, and a weight per element on each branch;
  * mixer "channel_delta": the gated delta rule behind short causal convolutions with silu, unit-length q and k
    (1e-6 under the root), a sigmoid write strength per head, a decay per head and key channel,
    exp(-exp(A_log) softplus(W_a2 W_a1 h + dt_bias)), a read-out normed per head and gated by the sigmoid of
    W_g2 W_g1 h;
  * mixer "parallel": two mixers read the same input, and the result is half the sum of their outputs, each normed over
    the width.  Left: grouped-head attention with interleaved rotary positions on the first ``rot.dims`` elements,
    queries and keys divided by their root mean square, scores squashed to softcap tanh(s / softcap), keys of the
    query's own chunk of ``mask.size`` positions only, and one added to the softmax's denominator.  Right: time mixing
    on a matrix per head, with inputs mixed with the token before's, a decay per channel and a bonus for the current
    token;
  * feed-forward "dense": down(gelu(gate h) * up h) with the tanh form of gelu;
  * logits = head N_final(x), a table of its own.

config.json: {"architecture": "Rafusun", "vocab", "width", "postln_alpha", "norm": {"eps"}, "embedding": {"scale",
"bigram": {"buckets", "mul_prev", "mul_cur"}}, "layers": [{"type", "mixer": {...}, "mlp": {"kind": "dense", "ff"} |
null}]}; tensors "embed", "bigram", "l<i>.norm1|norm2|ls1|ls2", "l<i>.mix.*", "l<i>.mlp.gate|up|down", "final.norm",
"head".
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from ..config.reader import ConfigError, KeyReader
from ..config.registry import register_architecture
from ..config.specs import LayerSpec, ModelSpec, PartSpec, RunEntry

ARCHITECTURE_NAME = "Rafusun"
MIXERS = ("channel_delta", "parallel")
UNIT_EPS = 1e-6  # under the root when the delta rule's q and k are made unit vectors
SINK_SCORE = 0.0  # exp of it joins every softmax's denominator
# the design names no longest sequence; tables by position are made for the engine's own limit
MAX_POSITIONS = 1 << 20


@dataclass(frozen=True)
class RafusunLayer:
    kind: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]]


@dataclass(frozen=True)
class RafusunConfig:
    vocab: int
    width: int
    eps: float
    alpha: float
    embedding_scale: float
    bigram: Optional[Dict[str, int]]
    layers: Tuple[RafusunLayer, ...]
    raw: Dict[str, Any]

    @staticmethod
    def _heads(r: KeyReader, where: str) -> Dict[str, Any]:
        out = {"heads": r.integer("heads", minimum=1), "kv_heads": r.integer("kv_heads", minimum=1), "dim": r.integer("dim", minimum=1),
               "vdim": r.integer("vdim", minimum=1)}
        if out["heads"] % out["kv_heads"]:
            raise ConfigError(f"{where}: heads={out['heads']} is not a multiple of kv_heads={out['kv_heads']}")
        return out

    @classmethod
    def _channel_delta(cls, m: Dict[str, Any], where: str) -> Dict[str, Any]:
        r = KeyReader(m, where=where)
        out = dict(cls._heads(r, where), conv=r.integer("conv", minimum=1))
        r.finish()
        return out

    @classmethod
    def _left(cls, m: Dict[str, Any], where: str) -> Dict[str, Any]:
        r = KeyReader(m, where=where)
        out = dict(cls._heads(r, where), scale=r.number("scale", positive=True), softcap=r.number("softcap", default=None, positive=True))
        mask = r.mapping("mask", default=None)  # (left out: every earlier key is seen)
        out["chunk"] = None
        if mask is not None:
            mr = KeyReader(mask, where=where + " mask")
            out["chunk"] = mr.integer("size", minimum=1)
            mr.finish()
        rot = r.mapping("rot", default=None)
        out["rot"] = None
        if rot is not None:
            rr = KeyReader(rot, where=where + " rot")
            dims = rr.integer("dims", minimum=2)
            if dims % 2 or dims > out["dim"]:
                raise ConfigError(f"{where} rot: dims={dims} must be even and at most dim={out['dim']}")
            out["rot"] = {"dims": dims, "base": rr.number("base", positive=True)}
            rr.finish()
        r.finish()
        return out

    @staticmethod
    def _right(m: Dict[str, Any], where: str) -> Dict[str, Any]:
        r = KeyReader(m, where=where)
        out = {"heads": r.integer("heads", minimum=1), "dim": r.integer("dim", minimum=1)}
        r.finish()
        return out

    @classmethod
    def _parallel(cls, m: Dict[str, Any], where: str) -> Dict[str, Any]:
        r = KeyReader(m, where=where)
        out = {"left": cls._left(r.mapping("left"), where + " left"), "right": cls._right(r.mapping("right"), where + " right")}
        r.finish()
        return out

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], strict: bool = False) -> "RafusunConfig":
        r = KeyReader(raw)
        vocab, width = r.integer("vocab", minimum=1), r.integer("width", minimum=1)
        eps = KeyReader(r.mapping("norm"), where="config.json norm").number("eps", positive=True)
        alpha = r.number("postln_alpha")
        scale, bigram = 1.0, None
        embedding = r.mapping("embedding", default=None)  # (left out: the rows as they are, and no pairs)
        if embedding is not None:
            er = KeyReader(embedding, where="config.json embedding")
            scale = er.number("scale", default=1.0, positive=True)
            pairs = er.mapping("bigram", default=None)
            if pairs is not None:
                pr = KeyReader(pairs, where="config.json embedding bigram")
                bigram = {"buckets": pr.integer("buckets", minimum=1), "mul_prev": pr.integer("mul_prev", minimum=0),
                          "mul_cur": pr.integer("mul_cur", minimum=0)}
                pr.finish()
            er.finish()
        listed = r.raw_value("layers", None)
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        readers = {"channel_delta": cls._channel_delta, "parallel": cls._parallel}
        layers = []
        for i, entry in enumerate(listed):
            where = f"config.json layers[{i}]"
            if not isinstance(entry, dict):
                raise ConfigError(f"{where} must be an object")
            er = KeyReader(entry, where=where)
            kind = er.string("type")
            if kind not in readers:
                raise ConfigError(f"{where}: mixer type {kind!r} is not one of this design's {MIXERS}")
            m = readers[kind](er.mapping("mixer"), where + " mixer")
            mlp = er.mapping("mlp", default=None)
            if mlp is not None:
                fr = KeyReader(mlp, where=where + " mlp")
                fr.require_value("kind", ["dense"], default="dense")
                mlp = {"ff": fr.integer("ff", minimum=1)}
                fr.finish()
            er.finish()
            layers.append(RafusunLayer(kind, m, mlp))
        r.taken.add("architecture")
        r.finish(strict=strict)
        return cls(vocab, width, eps, alpha, scale, bigram, tuple(layers), dict(raw))

    def to_dict(self) -> Dict[str, Any]:
        return dict(self.raw)


def _mixer(cfg: RafusunConfig, layer: RafusunLayer, prefix: str) -> PartSpec:
    m = layer.mixer
    if layer.kind == "channel_delta":
        return PartSpec("channel_delta_rule", {
            "prefix": prefix, "hidden_size": cfg.width, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
            "value_dim": m["vdim"], "conv_taps": m["conv"], "unit_eps": UNIT_EPS, "out_norm_eps": cfg.eps})
    left, right = m["left"], m["right"]
    attention = PartSpec("attention", {
        "prefix": f"{prefix}.left", "hidden_size": cfg.width, "num_heads": left["heads"], "num_kv_heads": left["kv_heads"],
        "head_dim": left["dim"], "value_dim": left["vdim"], "scale": left["scale"], "names": {"q": "q", "k": "k", "v": "v", "o": "o"},
        "window": left["chunk"], "chunked": left["chunk"] is not None, "softcap": left["softcap"], "sink_score": SINK_SCORE,
        "qk_norm": {"eps": cfg.eps},
        "position": None if left["rot"] is None else PartSpec("rotary", {
            "rotary_dim": left["rot"]["dims"], "theta": left["rot"]["base"], "pairing": "interleaved", "scaling": None})})
    time_mixing = PartSpec("time_mixing", {"prefix": f"{prefix}.right", "hidden_size": cfg.width, "num_heads": right["heads"],
                                           "head_dim": right["dim"], "out_norm_eps": cfg.eps})
    return PartSpec("side_by_side", {"left": attention, "right": time_mixing, "left_norm": f"{prefix}.left.out",
                                     "right_norm": f"{prefix}.right.out", "hidden_size": cfg.width, "eps": cfg.eps, "scale": 0.5})


def build_rafusun_spec(cfg: RafusunConfig) -> ModelSpec:
    def norm(name: str, **more: Any) -> PartSpec:
        return PartSpec("rmsnorm", dict({"name": name, "size": cfg.width, "eps": cfg.eps, "unit_offset": False}, **more))

    layers = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}"
        ffn = ffn_norm = None
        if layer.mlp is not None:
            ffn = PartSpec("gated_mlp", {"prefix": f"{p}.mlp", "hidden_size": cfg.width, "intermediate_size": layer.mlp["ff"],
                                         "activation": "gelu_tanh", "names": {"gate": "gate", "up": "up", "down": "down"}})
            ffn_norm = norm(f"{p}.norm2", branch_weight=f"{p}.ls2")
        layers.append(LayerSpec.of(p, "post_norm", mixer=_mixer(cfg, layer, f"{p}.mix"), mixer_norm=norm(f"{p}.norm1", branch_weight=f"{p}.ls1"),
                                   feed_forward=ffn, feed_forward_norm=ffn_norm).with_params(residual_scale=cfg.alpha))
    table = {"name": "embed", "vocab_size": cfg.vocab, "hidden_size": cfg.width, "scale": cfg.embedding_scale}
    if cfg.bigram is None:
        embedding = PartSpec("token_embedding", table)
    else:
        embedding = PartSpec("token_pair_embedding", dict(table, pair_name="bigram", **cfg.bigram))
    spec = ModelSpec(
        architecture=ARCHITECTURE_NAME,
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        max_positions=MAX_POSITIONS,
        embedding=embedding,
        layers=tuple(layers),
        run_order=tuple(RunEntry(layer=i) for i in range(len(layers))),
        final_norm=norm("final.norm"),
        head=PartSpec("lm_head", {"name": "head", "tied_to": None, "vocab_size": cfg.vocab, "hidden_size": cfg.width}),
    )
    spec.validate()
    return spec


register_architecture(ARCHITECTURE_NAME, RafusunConfig, build_rafusun_spec)
