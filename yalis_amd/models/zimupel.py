"""Zimupel: a small decoder whose config.json lists its layers one by one, each with one of three mixers and an optional
dense or routed feed-forward, on a stream that is kept as several copies.

What the design fixes (everything else is read from config.json or a tensor's shape):
  * the stream starts as the RMS norm of embed[token] with the weight "embed.norm", as ``streams`` equal copies; for either
    branch q of a layer (1 the mixer, 2 the feed-forward) u = sum_s hc_q.in[s] x_s, y = branch(norm_q(u)), and
    x_t <- sum_s hc_q.mix[s, t] x_s + hc_q.out[t] y; the model ends with the norm of the copies' sum;
  * mixer "retention": a matrix per head with a constant decay per head (``decay``), rotary positions on the first ``rot.dims``
    elements of q and k, pairs (i, i + dims / 2), k times dim^-1/2, a read-out normed per head without a weight and gated by silu;
  * mixer "lightning": the same recurrence on silu of all three projections, the heads' read-outs normed together with a
    weight and gated by the sigmoid;
  * mixer "attention": differential attention with grouped heads, biases on q, k and v, no positions; a layer with
    ``kv_from`` reads an earlier layer's keys and values;
  * feed-forward "dense": down(gelu(gate h) * up h) with the tanh form of gelu; "moe": sigmoid scores, a correction for the
    choice alone, groups of experts of which the best are kept, weights the chosen scores' shares; an expert is
    down(silu(gate h) * up h);
  * logits = cap tanh(scale (head N_final(sum_s x_s)) / cap), a table of its own.

config.json: {"architecture": "Zimupel", "vocab", "width", "streams", "norm": {"eps"}, "logit_scale", "logit_softcap", "layers":
[{"type", "mixer": {...}, "mlp": {"kind": "dense", "ff"} | {"kind": "moe", "router": {"experts", "top", "groups": {"count",
"keep"}}, "expert": {"ff"}} | null}]}; tensors "embed", "embed.norm", "l<i>.norm1|norm2", "l<i>.hc1|hc2.in|out|mix",
"l<i>.mix.*", "l<i>.mlp.*", "final.norm", "head".
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from ..config.reader import ConfigError, KeyReader
from ..config.registry import register_architecture
from ..config.specs import LayerSpec, ModelSpec, PartSpec, RunEntry

ARCHITECTURE_NAME = "Zimupel"
MIXERS = ("retention", "attention", "lightning")
MAX_STREAMS = 16  # copies of the stream the kernel between two branches holds
# the design names no longest sequence; tables by position are made for the engine's own limit
MAX_POSITIONS = 1 << 20


@dataclass(frozen=True)
class ZimupelLayer:
    kind: str
    mixer: Dict[str, Any]
    mlp: Optional[Dict[str, Any]]


@dataclass(frozen=True)
class ZimupelConfig:
    vocab: int
    width: int
    eps: float
    streams: int
    logit_scale: float
    logit_softcap: Optional[float]
    layers: Tuple[ZimupelLayer, ...]
    raw: Dict[str, Any]

    @staticmethod
    def _recurrent(r: KeyReader, where: str) -> Dict[str, Any]:
        out = {"heads": r.integer("heads", minimum=1), "dim": r.integer("dim", minimum=1), "vdim": r.integer("vdim", minimum=1)}
        decay = r.raw_value("decay", None)
        if not isinstance(decay, list) or len(decay) != out["heads"] or not all(
                isinstance(d, (int, float)) and not isinstance(d, bool) and 0.0 <= d <= 1.0 for d in decay):
            raise ConfigError(f"{where}: 'decay' must list a number between 0 and 1 for each of the {out['heads']} heads")
        return dict(out, decay=tuple(float(d) for d in decay))

    @classmethod
    def _retention(cls, m: Dict[str, Any], where: str) -> Dict[str, Any]:
        r = KeyReader(m, where=where)
        out = dict(cls._recurrent(r, where), rot=None)
        rot = r.mapping("rot", default=None)  # (left out: nothing rotates)
        if rot is not None:
            rr = KeyReader(rot, where=where + " rot")
            dims = rr.integer("dims", minimum=2)
            if dims % 2 or dims > out["dim"]:
                raise ConfigError(f"{where} rot: dims={dims} must be even and at most dim={out['dim']}")
            out["rot"] = {"dims": dims, "base": rr.number("base", positive=True)}
            rr.finish()
        r.finish()
        return out

    @classmethod
    def _lightning(cls, m: Dict[str, Any], where: str) -> Dict[str, Any]:
        r = KeyReader(m, where=where)
        out = cls._recurrent(r, where)
        r.finish()
        return out

    @staticmethod
    def _attention(m: Dict[str, Any], where: str) -> Dict[str, Any]:
        r = KeyReader(m, where=where)
        out = {"heads": r.integer("heads", minimum=1), "kv_heads": r.integer("kv_heads", minimum=1), "dim": r.integer("dim", minimum=1),
               "vdim": r.integer("vdim", minimum=1), "scale": r.number("scale", positive=True), "diff": r.number("diff"),
               "kv_from": r.integer("kv_from", default=None, minimum=0)}
        if out["heads"] % out["kv_heads"]:
            raise ConfigError(f"{where}: heads={out['heads']} is not a multiple of kv_heads={out['kv_heads']}")
        r.finish()
        return out

    @staticmethod
    def _mlp(f: Dict[str, Any], where: str) -> Dict[str, Any]:
        r = KeyReader(f, where=where)
        if r.require_value("kind", ["dense", "moe"], default="dense") == "dense":
            out: Dict[str, Any] = {"kind": "dense", "ff": r.integer("ff", minimum=1)}
            r.finish()
            return out
        router = KeyReader(r.mapping("router"), where=where + " router")
        expert = KeyReader(r.mapping("expert"), where=where + " expert")
        out = {"kind": "moe", "experts": router.integer("experts", minimum=1), "top": router.integer("top", minimum=1),
               "ff": expert.integer("ff", minimum=1), "groups": None}
        groups = router.mapping("groups", default=None)  # (left out: every expert can be chosen)
        reach = out["experts"]
        if groups is not None:
            gr = KeyReader(groups, where=where + " router groups")
            count, keep = gr.integer("count", minimum=1), gr.integer("keep", minimum=1)
            if out["experts"] % count or keep > count:
                raise ConfigError(f"{where} router groups: {out['experts']} experts in count={count} equal groups, keep={keep}")
            gr.finish()
            out["groups"] = {"count": count, "keep": keep}
            reach = keep * (out["experts"] // count)
        if out["top"] > reach:
            raise ConfigError(f"{where}: top={out['top']} of {reach} experts that can be chosen")
        router.finish()
        expert.finish()
        r.finish()
        return out

    @classmethod
    def from_dict(cls, raw: Dict[str, Any], strict: bool = False) -> "ZimupelConfig":
        r = KeyReader(raw)
        vocab, width = r.integer("vocab", minimum=1), r.integer("width", minimum=1)
        eps = KeyReader(r.mapping("norm"), where="config.json norm").number("eps", positive=True)
        streams = r.integer("streams", minimum=1)
        if streams > MAX_STREAMS:
            raise ConfigError(f"config.json: streams={streams}, at most {MAX_STREAMS} are offered")
        scale, cap = r.number("logit_scale", default=1.0), r.number("logit_softcap", default=None, positive=True)
        listed = r.raw_value("layers", None)
        if not isinstance(listed, list) or not listed:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        readers = {"retention": cls._retention, "attention": cls._attention, "lightning": cls._lightning}
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
            source = m.get("kv_from")
            if source is not None:
                if source >= i or layers[source].kind != "attention" or layers[source].mixer["kv_from"] is not None:
                    raise ConfigError(f"{where}: kv_from={source} must name an earlier attention layer with keys and values of its own")
                for key in ("heads", "kv_heads", "dim", "vdim"):
                    if m[key] != layers[source].mixer[key]:
                        raise ConfigError(f"{where}: kv_from={source}, whose {key}={layers[source].mixer[key]} is not this layer's {m[key]}")
            mlp = er.mapping("mlp", default=None)
            layers.append(ZimupelLayer(kind, m, None if mlp is None else cls._mlp(mlp, where + " mlp")))
            er.finish()
        r.taken.add("architecture")
        r.finish(strict=strict)
        return cls(vocab, width, eps, streams, scale, cap, tuple(layers), dict(raw))

    def to_dict(self) -> Dict[str, Any]:
        return dict(self.raw)


def _mixer(cfg: ZimupelConfig, layer: ZimupelLayer, prefix: str) -> PartSpec:
    m = layer.mixer
    common = {"prefix": prefix, "hidden_size": cfg.width, "num_heads": m["heads"], "head_dim": m["dim"], "value_dim": m["vdim"]}
    if layer.kind == "attention":
        return PartSpec("attention", dict(
            common, num_kv_heads=m["kv_heads"], scale=m["scale"], window=None, position=None, names={"q": "q", "k": "k", "v": "v", "o": "o"},
            projection_bias={"q": "q.b", "k": "k.b", "v": "v.b"},
            differential={"q1": "lq1", "k1": "lk1", "q2": "lq2", "k2": "lk2", "offset": m["diff"], "eps": cfg.eps}))
    common.update(decay=list(m["decay"]), out_norm_eps=cfg.eps)
    if layer.kind == "lightning":
        return PartSpec("lightning_attention", common)
    rot = m["rot"]
    return PartSpec("retention", dict(common, position=None if rot is None else PartSpec("rotary", {
        "rotary_dim": rot["dims"], "theta": rot["base"], "pairing": "half", "scaling": None})))


def _feed_forward(cfg: ZimupelConfig, f: Optional[Dict[str, Any]], prefix: str) -> Optional[PartSpec]:
    if f is None:
        return None
    common = {"prefix": prefix, "hidden_size": cfg.width, "intermediate_size": f["ff"]}
    if f["kind"] == "dense":
        return PartSpec("gated_mlp", dict(common, activation="gelu_tanh", names={"gate": "gate", "up": "up", "down": "down"}))
    return PartSpec("routed_moe", dict(common, experts=f["experts"], top=f["top"], activation="silu", scores="sigmoid_share", weighs="output",
                                       choice_correction="correction", groups=f["groups"]))


def build_zimupel_spec(cfg: ZimupelConfig) -> ModelSpec:
    def norm(name: str) -> PartSpec:
        return PartSpec("rmsnorm", {"name": name, "size": cfg.width, "eps": cfg.eps, "unit_offset": False})

    def streams(prefix: str) -> PartSpec:
        return PartSpec("mixed_streams", {"prefix": prefix, "streams": cfg.streams})

    layers, order = [], []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}"
        ff = _feed_forward(cfg, layer.mlp, f"{p}.mlp")
        layers.append(LayerSpec.of(
            p, "mixed_streams", mixer_streams=streams(f"{p}.hc1"), mixer_norm=norm(f"{p}.norm1"), mixer=_mixer(cfg, layer, f"{p}.mix"),
            feed_forward_streams=None if ff is None else streams(f"{p}.hc2"), feed_forward_norm=None if ff is None else norm(f"{p}.norm2"),
            feed_forward=ff))
        order.append(RunEntry(layer=i, cache_from=layer.mixer.get("kv_from")))
    spec = ModelSpec(
        architecture=ARCHITECTURE_NAME,
        hidden_size=cfg.width,
        vocab_size=cfg.vocab,
        max_positions=MAX_POSITIONS,
        embedding=PartSpec("normed_token_embedding", {"name": "embed", "norm_name": "embed.norm", "eps": cfg.eps, "vocab_size": cfg.vocab,
                                                      "hidden_size": cfg.width, "streams": cfg.streams}),
        layers=tuple(layers),
        run_order=tuple(order),
        final_norm=norm("final.norm"),
        head=PartSpec("lm_head", {"name": "head", "tied_to": None, "vocab_size": cfg.vocab, "hidden_size": cfg.width, "scale": cfg.logit_scale,
                                  "softcap": cfg.logit_softcap}),
    )
    spec.validate()
    return spec


register_architecture(ARCHITECTURE_NAME, ZimupelConfig, build_zimupel_spec)
