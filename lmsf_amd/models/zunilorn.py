"""Zunilorn as a ModelSpec: a decoder whose residual is several streams, with a loop over some of its layers.

n streams all begin as the token's row of the embedding table. Every layer: a sublayer reads a weighted sum of the
streams, RMS-normed; its result, times one constant of the model and a number per stream, joins the streams, which are
mixed by a matrix of the sublayer on the same occasion (parts/block.py: ``stream_residual``); first the mixer, then the
feed-forward. Layers ``loop.start`` to ``loop.stop`` - 1 run ``loop.times`` times in a row with the same weights and a cache
or state per pass. The mixer is one of
- "mamba2": a recurrence of matrices with one decay a head (parts/recurrent.py: ``state_space``);
- "attention": softmax attention with rotation of half-split pairs and YaRN scaling, a soft cap, a sink a head and a
  gate of one number a head (parts/flex_attention.py).
The feed-forward is dense and gated, both operands of the activation bounded, with biases (parts/mlp.py, "bounded"); or
experts of that form without biases, chosen by a softmax router with corrected scores, the last of its outputs experts
that return their input, with a shared expert behind a gate of one number a token (parts/routed_moe.py); or absent. The
logits are the embedding table times the normed sum of the streams, bounded by a soft cap. The reference has no such
architecture; its model files hard-wire Llama's block (core/src/model_executor/models/llama/llama.rs:276-385).

config.json: "architecture": "Zunilorn", "vocab", "width", "streams", "residual_mult", "norm": {"eps"}, "logit_softcap",
"loop"?: {"start", "stop", "times"}, and "layers", a list of {"type", "mixer", "mlp"} with
  mamba2:    {"heads", "vdim", "state", "groups", "conv", "norm_groups"}
  attention: {"heads", "kv_heads", "dim", "vdim", "scale", "softcap"?, "rot": {"base", "dims", "scaling"?: {"factor",
              "original", "fast", "slow"}}}
  mlp: null | {"kind": "dense", "ff", "limit"} | {"kind": "moe", "expert": {"ff", "limit"}, "router": {"experts", "top",
               "identity"?, "scale"?}, "shared"?: {"ff", "limit"}}
Optional: "max_position_embeddings", "torch_dtype", "eos_token_id", "bos_token_id".

Checkpoint names: embed, final.norm; per layer l<i>.{norm1, norm2}, l<i>.{hc1, hc2}.{in, out, mix}, l<i>.mix.{in, conv,
conv.b, dt_bias, A_log, D, norm, o} or l<i>.mix.{q, k, v, sink, g, o}, l<i>.mlp.{gate, up, down} with ".b" each, or
l<i>.mlp.{router, correction, e<k>.{gate, up, down}, shared.{gate, up, down, sg}}.
"""
import json
from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple

from ..config.model_config import ArchConfig, ConfigError
from ..config.registry import register_architecture
from ..parts.base import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

DEFAULT_MAX_POSITIONS = 131072
MAX_STREAMS = 32
MAX_STATE = 1024
_NUMBER = (int, float)


def _need(d: Any, key: str, where: str, kind=(int,), positive: bool = True, at_least: Optional[int] = None):
    if not isinstance(d, dict) or key not in d:
        raise ConfigError("config.json: %s lacks %r" % (where, key))
    v = d[key]
    if isinstance(v, bool) or not isinstance(v, kind):
        raise ConfigError("config.json: %s.%s is %r" % (where, key, v))
    if at_least is not None:
        if v < at_least:
            raise ConfigError("config.json: %s.%s must be >= %d, is %r" % (where, key, at_least, v))
    elif positive and not v > 0:
        raise ConfigError("config.json: %s.%s must be > 0, is %r" % (where, key, v))
    return v


@dataclass(frozen=True)
class ZunilornConfig(ArchConfig):
    width: int = 0
    streams: int = 1
    residual_mult: float = 1.0
    norm_eps: float = 1e-5
    logit_softcap: float = 0.0      # 0: logits as they are
    loop_start: int = 0
    loop_stop: int = 0              # start == stop: no loop
    loop_times: int = 1
    layers_json: str = "[]"         # the "layers" list as it was read (text: the dataclass is frozen and hashable)

    ARCHITECTURE = "Zunilorn"

    @property
    def layers(self) -> Tuple[Dict[str, Any], ...]:
        return tuple(json.loads(self.layers_json))

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "ZunilornConfig":
        where = "the configuration"
        vocab, width = _need(d, "vocab", where), _need(d, "width", where)
        streams = _need(d, "streams", where)
        mult = _need(d, "residual_mult", where, _NUMBER, positive=False) if "residual_mult" in d else 1.0
        eps = _need(d.get("norm"), "eps", "norm", _NUMBER)
        cap = _need(d, "logit_softcap", where, _NUMBER) if d.get("logit_softcap") is not None else 0.0
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        start, stop, times = 0, 0, 1
        if d.get("loop") is not None:
            start = _need(d["loop"], "start", "loop", at_least=0)
            stop = _need(d["loop"], "stop", "loop", at_least=0)
            times = _need(d["loop"], "times", "loop")
        eos = d.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos]))
        cfg = cls(architecture=cls.ARCHITECTURE, vocab_size=int(vocab),
                  max_position_embeddings=int(d.get("max_position_embeddings") or DEFAULT_MAX_POSITIONS),
                  torch_dtype=str(d.get("torch_dtype") or "bfloat16"), eos_token_ids=eos_ids,
                  bos_token_id=None if d.get("bos_token_id") is None else int(d["bos_token_id"]),
                  width=int(width), streams=int(streams), residual_mult=float(mult), norm_eps=float(eps),
                  logit_softcap=float(cap), loop_start=int(start), loop_stop=int(stop), loop_times=int(times),
                  layers_json=json.dumps(layers))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        layers = self.layers
        if self.streams > MAX_STREAMS:
            raise ConfigError("config.json: streams %d: at most %d" % (self.streams, MAX_STREAMS))
        if not (0 <= self.loop_start <= self.loop_stop <= len(layers)):
            raise ConfigError("config.json: loop %d to %d does not lie within the %d layers"
                              % (self.loop_start, self.loop_stop, len(layers)))
        for i, layer in enumerate(layers):
            where = "layers[%d]" % i
            kind = layer.get("type") if isinstance(layer, dict) else None
            m = layer.get("mixer") if isinstance(layer, dict) else None
            at = where + ".mixer"
            if kind == "mamba2":
                for key in ("heads", "vdim", "state", "groups", "conv", "norm_groups"):
                    _need(m, key, at)
                if m["heads"] % m["groups"]:
                    raise ConfigError("config.json: %s.heads %d is not a multiple of groups %d" % (at, m["heads"], m["groups"]))
                if m["heads"] * m["vdim"] % m["norm_groups"]:
                    raise ConfigError("config.json: %s: %d heads of %d do not split into norm_groups %d"
                                      % (at, m["heads"], m["vdim"], m["norm_groups"]))
                if m["state"] > MAX_STATE:
                    raise ConfigError("config.json: %s.state %d: at most %d" % (at, m["state"], MAX_STATE))
            elif kind == "attention":
                heads, kv = _need(m, "heads", at), _need(m, "kv_heads", at)
                if heads % kv:
                    raise ConfigError("config.json: %s.heads %d is not a multiple of kv_heads %d" % (at, heads, kv))
                dim = _need(m, "dim", at)
                _need(m, "vdim", at)
                _need(m, "scale", at, _NUMBER)
                if m.get("softcap") is not None:
                    _need(m, "softcap", at, _NUMBER)
                rot = m.get("rot")
                _need(rot, "base", at + ".rot", _NUMBER)
                dims = _need(rot, "dims", at + ".rot")
                if dims % 2 or dims > dim:
                    raise ConfigError("config.json: %s.rot.dims %d must be even and at most %d" % (at, dims, dim))
                if rot.get("scaling") is not None:
                    for key in ("factor", "original", "fast", "slow"):
                        _need(rot["scaling"], key, at + ".rot.scaling", _NUMBER)
            else:
                raise ConfigError("config.json: %s.type %r is not supported (mamba2, attention)" % (where, kind))
            mlp = layer.get("mlp")
            if mlp is None:
                continue
            mk = mlp.get("kind") if isinstance(mlp, dict) else None
            at = where + ".mlp"
            if mk == "dense":
                _need(mlp, "ff", at)
                _need(mlp, "limit", at, _NUMBER)
            elif mk == "moe":
                for key in ("expert", "shared"):
                    if key == "expert" or mlp.get(key) is not None:
                        _need(mlp.get(key), "ff", "%s.%s" % (at, key))
                        _need(mlp.get(key), "limit", "%s.%s" % (at, key), _NUMBER)
                r = mlp.get("router")
                e, top = _need(r, "experts", at + ".router"), _need(r, "top", at + ".router")
                same = _need(r, "identity", at + ".router", at_least=0) if r.get("identity") is not None else 0
                if r.get("scale") is not None:
                    _need(r, "scale", at + ".router", _NUMBER, positive=False)
                if top > e + same or top > 64:
                    raise ConfigError("config.json: %s.router: %d of %d experts (at most 64 a token)" % (at, top, e + same))
            else:
                raise ConfigError("config.json: %s.kind %r is not supported (dense, moe)" % (at, mk))

    def to_dict(self) -> Dict[str, Any]:
        out = {"architecture": self.ARCHITECTURE, "vocab": self.vocab_size, "width": self.width, "streams": self.streams,
               "residual_mult": self.residual_mult, "norm": {"eps": self.norm_eps},
               "logit_softcap": self.logit_softcap or None, "layers": list(self.layers),
               "max_position_embeddings": self.max_position_embeddings, "torch_dtype": self.torch_dtype,
               "eos_token_id": list(self.eos_token_ids) or None, "bos_token_id": self.bos_token_id}
        if self.loop_stop > self.loop_start:
            out["loop"] = {"start": self.loop_start, "stop": self.loop_stop, "times": self.loop_times}
        return out


def layer_runs(cfg: ZunilornConfig) -> List[int]:
    """The layers in the order in which they run."""
    a, b = cfg.loop_start, cfg.loop_stop
    return list(range(a)) + list(range(a, b)) * cfg.loop_times + list(range(b, len(cfg.layers)))


def _mixer_spec(kind: str, m: Dict[str, Any], W: int, eps: float) -> PartSpec:
    if kind == "mamba2":
        return PartSpec("state_space", {
            "prefix": "mix", "hidden_size": W, "heads": m["heads"], "vdim": m["vdim"], "state": m["state"],
            "groups": m["groups"], "conv": m["conv"], "norm_groups": m["norm_groups"], "eps": eps})
    rot = m["rot"]
    sc = rot.get("scaling")
    scaling = None if sc is None else {"rope_type": "yarn", "factor": sc["factor"], "beta_fast": sc["fast"],
                                       "beta_slow": sc["slow"], "original_max_position_embeddings": sc["original"]}
    return PartSpec("flex_attention", {
        "prefix": "mix", "hidden_size": W, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
        "v_head_dim": m["vdim"], "scale": m["scale"], "softcap": m.get("softcap") or 0.0, "sink": True, "head_gate": True,
        "weights_f32": True,
        "position": PartSpec("rotary", {"head_dim": m["dim"], "rotary_dim": rot["dims"], "theta": rot["base"],
                                        "scaling": scaling, "style": "neox", "angles": "float64"})})


def _ffn_spec(mlp: Optional[Dict[str, Any]], W: int) -> PartSpec:
    def gated(prefix: str, sizes: Dict[str, Any], bias: bool) -> PartSpec:
        return PartSpec("gated_mlp", {"prefix": prefix, "hidden_size": W, "intermediate_size": sizes["ff"],
                                      "activation": "bounded", "limit": sizes["limit"], "bias": bias, "bias_name": "b",
                                      "gate_name": "gate", "up_name": "up", "down_name": "down", "bare_names": True})

    if mlp is None:
        return PartSpec("none", {})
    if mlp["kind"] == "dense":
        return gated("mlp", mlp, True)
    r, shared = mlp["router"], mlp.get("shared")
    return PartSpec("routed_moe", {
        "prefix": "mlp", "hidden_size": W, "expert_size": mlp["expert"]["ff"], "limit": mlp["expert"]["limit"],
        "num_experts": r["experts"], "identity": r.get("identity") or 0, "top": r["top"], "scores": "softmax",
        "renormalize": True, "route_scale": 1.0 if r.get("scale") is None else r["scale"], "correction_name": "correction",
        "weight_on": "output", "shared": gated("shared", shared, False) if shared is not None else None,
        "shared_gate": "shared.sg" if shared is not None else None})


def build_zunilorn_spec(cfg: ZunilornConfig) -> ModelSpec:
    W = cfg.width

    def norm(name: str, kind: str = "group_rms_norm") -> PartSpec:
        return PartSpec(kind, {"prefix": name, "size": W, "eps": cfg.norm_eps, "weight_name": ""})

    layers = []
    for i, layer in enumerate(cfg.layers):
        mlp = layer.get("mlp")
        norms = {"input": norm("norm1")}
        if mlp is not None:
            norms["post_mixer"] = norm("norm2")
        layers.append(LayerSpec(
            prefix="l%d" % i, block=PartSpec("stream_residual", {"streams": cfg.streams, "scale": cfg.residual_mult}),
            mixer=_mixer_spec(layer["type"], layer["mixer"], W, cfg.norm_eps), feed_forward=_ffn_spec(mlp, W), norms=norms))
    return ModelSpec(
        embedding=PartSpec("stream_embedding", {"prefix": "embed", "vocab_size": cfg.vocab_size, "hidden_size": W,
                                                "streams": cfg.streams, "weight_name": ""}),
        layers=tuple(layers), schedule=tuple(ScheduleEntry(i) for i in layer_runs(cfg)),
        final_norm=norm("final.norm", "stream_sum_norm"),
        head=PartSpec("lm_head", {"prefix": "head", "vocab_size": cfg.vocab_size, "hidden_size": W, "weight_name": "embed",
                                  "softcap": cfg.logit_softcap}),
        vocab_size=cfg.vocab_size, hidden_size=W)


# a layer without a feed-forward may still carry the norm and the streams' numbers of one
register_architecture("Zunilorn", "zunilorn", ZunilornConfig, build_zunilorn_spec,
                      tolerated_tensors=(".norm2", ".hc2.in", ".hc2.out", ".hc2.mix"))
