"""Gurapel as a ModelSpec: a decoder with learned position vectors, norms on the sublayers' outputs alone, and experts.

x_0 = scale * embed[token] + pos[position]. Every layer is x += norm1(mixer(x)), then, where it has a feed-forward,
x += norm2(ffn(x)): the sublayers read the stream as it is, the norms are RMS norms whose stored weight w acts as 1 + w
(parts/block.py: ``output_norm``). The mixer is one of
- "parallel": two mixers side by side on the same input, each output RMS-normed over the width, the mean of the two
  (parts/parallel.py): "left" softmax attention within a window without rotation, with a norm over every query and key
  head, a soft cap and a logarithmic distance bias (parts/flex_attention.py), "right" Griffin's gated linear recurrence
  (parts/recurrent.py);
- "delta": the gated delta rule with one decay a head (parts/delta_rule.py).
The feed-forward is a mixture of gated experts, the ``top`` of the router's logits weighted by the softmax over the chosen
alone (parts/routed_moe.py), or absent. The logits are head . final_norm(x). The reference has no such architecture; its
model files hard-wire Llama's block (core/src/model_executor/models/llama/llama.rs:276-385).

config.json: "architecture": "Gurapel", "vocab", "width", "norm": {"eps"}, "embedding": {"scale"}, "max_positions" (rows of
the table of position vectors; without it the checkpoint's header gives them), and "layers", a list of
{"type", "mixer", "mlp"} with
  parallel: {"left": {"heads", "kv_heads", "dim", "vdim", "scale", "softcap"?, "mask": {"size"}},
             "right": {"width", "blocks", "conv"}}
  delta:    {"heads", "kv_heads", "dim", "vdim", "conv"}
  mlp:      null | {"kind": "moe", "expert": {"ff"}, "router": {"experts", "top"}}
Optional: "max_position_embeddings", "torch_dtype", "eos_token_id", "bos_token_id".

Checkpoint names: embed, pos, final.norm, head; per layer l<i>.{norm1, norm2}, l<i>.mix.left.{q, k, v, q.norm, k.norm, r1,
r2, o, out}, l<i>.mix.right.{y, y.b, x, x.b, conv, conv.b, ra, ra.b, ri, ri.b, lam, o, out} or l<i>.mix.{q, k, v, q.conv,
k.conv, v.conv, b, a, A_log, dt_bias, g, norm, o}, and l<i>.mlp.{router, e<k>.{gate, up, down}}.
"""
import json
from dataclasses import dataclass
from typing import Any, Dict, Tuple

from ..config.model_config import ArchConfig, ConfigError
from ..config.registry import register_architecture
from ..parts.base import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

_NUMBER = (int, float)
RECURRENCE_DECAY = 8.0          # log a = -8 r softplus(lam)
UNIT_NORM_EPS = 1e-6            # inside the root of the delta rule's unit vectors


def _need(d: Any, key: str, where: str, kind=(int,), positive: bool = True):
    if not isinstance(d, dict) or key not in d:
        raise ConfigError("config.json: %s lacks %r" % (where, key))
    v = d[key]
    if isinstance(v, bool) or not isinstance(v, kind):
        raise ConfigError("config.json: %s.%s is %r" % (where, key, v))
    if positive and not v > 0:
        raise ConfigError("config.json: %s.%s must be > 0, is %r" % (where, key, v))
    return v


def _check_heads(m: Any, where: str) -> None:
    heads, kv = _need(m, "heads", where), _need(m, "kv_heads", where)
    if heads % kv:
        raise ConfigError("config.json: %s.heads %d is not a multiple of kv_heads %d" % (where, heads, kv))
    _need(m, "dim", where)
    _need(m, "vdim", where)


@dataclass(frozen=True)
class GurapelConfig(ArchConfig):
    width: int = 0
    norm_eps: float = 1e-5
    embedding_scale: float = 1.0
    layers_json: str = "[]"         # the "layers" list as it was read (text: the dataclass is frozen and hashable)
    position_rows: int = 0          # rows of the table of position vectors

    ARCHITECTURE = "Gurapel"

    @property
    def layers(self) -> Tuple[Dict[str, Any], ...]:
        return tuple(json.loads(self.layers_json))

    @staticmethod
    def complete_from_checkpoint(d: Dict[str, Any], folder: str) -> Dict[str, Any]:
        """Where config.json does not say how many position vectors there are, the tensor's rows do."""
        if "max_positions" in d:
            return d
        from ..weights.loader import header_shapes
        try:
            shape = header_shapes(folder).get("pos")
        except Exception:  # noqa: BLE001 - no checkpoint (random weights): from_dict names the missing key
            return d
        return dict(d, max_positions=int(shape[0])) if shape else d

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "GurapelConfig":
        vocab = _need(d, "vocab", "the configuration")
        width = _need(d, "width", "the configuration")
        eps = _need(d.get("norm"), "eps", "norm", _NUMBER)
        scale = _need(d.get("embedding"), "scale", "embedding", _NUMBER, positive=False)
        rows = _need(d, "max_positions", "the configuration")
        layers = d.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        eos = d.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos]))
        # (a request can be no longer than there are position vectors)
        longest = min(int(rows), int(d.get("max_position_embeddings") or rows))
        cfg = cls(architecture=cls.ARCHITECTURE, vocab_size=int(vocab), max_position_embeddings=longest,
                  torch_dtype=str(d.get("torch_dtype") or "bfloat16"), eos_token_ids=eos_ids,
                  bos_token_id=None if d.get("bos_token_id") is None else int(d["bos_token_id"]),
                  width=int(width), norm_eps=float(eps), embedding_scale=float(scale), layers_json=json.dumps(layers),
                  position_rows=int(rows))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        for i, layer in enumerate(self.layers):
            where = "layers[%d]" % i
            kind = layer.get("type") if isinstance(layer, dict) else None
            m = layer.get("mixer") if isinstance(layer, dict) else None
            at = where + ".mixer"
            if kind == "parallel":
                left, right = (m or {}).get("left"), (m or {}).get("right")
                _check_heads(left, at + ".left")
                _need(left, "scale", at + ".left", _NUMBER)
                if left.get("softcap") is not None:
                    _need(left, "softcap", at + ".left", _NUMBER)
                _need(left.get("mask"), "size", at + ".left.mask")
                C, blocks = _need(right, "width", at + ".right"), _need(right, "blocks", at + ".right")
                _need(right, "conv", at + ".right")
                if C % blocks:
                    raise ConfigError("config.json: %s.right.width %d does not split into %d blocks" % (at, C, blocks))
            elif kind == "delta":
                _check_heads(m, at)
                _need(m, "conv", at)
                if m["dim"] > 256:
                    raise ConfigError("config.json: %s.dim %d: keys of at most 256 entries" % (at, m["dim"]))
            else:
                raise ConfigError("config.json: %s.type %r is not supported (parallel, delta)" % (where, kind))
            mlp = layer.get("mlp")
            if mlp is None:
                continue
            if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
                raise ConfigError("config.json: %s.mlp.kind %r is not supported (moe)"
                                  % (where, mlp.get("kind") if isinstance(mlp, dict) else mlp))
            _need(mlp.get("expert"), "ff", where + ".mlp.expert")
            e, top = (_need(mlp.get("router"), k, where + ".mlp.router") for k in ("experts", "top"))
            if top > e:
                raise ConfigError("config.json: %s.mlp.router: %d of %d experts" % (where, top, e))

    def to_dict(self) -> Dict[str, Any]:
        out = {"architecture": self.ARCHITECTURE, "vocab": self.vocab_size, "width": self.width,
               "norm": {"eps": self.norm_eps}, "embedding": {"scale": self.embedding_scale},
               "max_positions": self.position_rows, "layers": list(self.layers), "torch_dtype": self.torch_dtype,
               "eos_token_id": list(self.eos_token_ids) or None, "bos_token_id": self.bos_token_id}
        if self.max_position_embeddings < self.position_rows:
            out["max_position_embeddings"] = self.max_position_embeddings
        return out


def _mixer_spec(kind: str, m: Dict[str, Any], W: int, eps: float) -> PartSpec:
    if kind == "delta":
        return PartSpec("gated_delta", {
            "prefix": "mix", "hidden_size": W, "heads": m["heads"], "kv_heads": m["kv_heads"], "dim": m["dim"],
            "vdim": m["vdim"], "conv": m["conv"], "decay_rank": None, "gate_rank": None, "gate_activation": "silu",
            "eps": eps, "unit_eps": UNIT_NORM_EPS})
    left, right = m["left"], m["right"]
    return PartSpec("parallel_pair", {
        "prefix": "mix", "hidden_size": W, "eps": eps, "scale": 0.5,
        "left": PartSpec("flex_attention", {
            "hidden_size": W, "num_heads": left["heads"], "num_kv_heads": left["kv_heads"], "head_dim": left["dim"],
            "v_head_dim": left["vdim"], "scale": left["scale"], "softcap": left.get("softcap") or 0.0,
            "window": left["mask"]["size"], "unit_norm_eps": eps, "head_norm_weights": True, "distance_bias": True,
            "weights_f32": True}),
        "right": PartSpec("gated_linear_recurrence", {"hidden_size": W, "width": right["width"], "blocks": right["blocks"],
                                                      "conv": right["conv"], "decay": RECURRENCE_DECAY})})


def build_gurapel_spec(cfg: GurapelConfig) -> ModelSpec:
    W = cfg.width

    def norm(name: str) -> PartSpec:
        return PartSpec("group_rms_norm", {"prefix": name, "size": W, "eps": cfg.norm_eps, "weight_name": "",
                                           "weight_offset": 1.0})

    layers = []
    for i, layer in enumerate(cfg.layers):
        mlp = layer.get("mlp")
        norms = {"post_mixer": norm("norm1")}
        ffn = PartSpec("none", {})
        if mlp is not None:
            norms["post_ffn"] = norm("norm2")
            ffn = PartSpec("routed_moe", {
                "prefix": "mlp", "hidden_size": W, "expert_size": mlp["expert"]["ff"],
                "num_experts": mlp["router"]["experts"], "top": mlp["router"]["top"], "scores": "softmax",
                "renormalize": True, "weight_on": "output"})
        layers.append(LayerSpec(prefix="l%d" % i, block=PartSpec("output_norm"),
                                mixer=_mixer_spec(layer["type"], layer["mixer"], W, cfg.norm_eps), feed_forward=ffn,
                                norms=norms))
    return ModelSpec(
        embedding=PartSpec("positioned_embedding", {
            "prefix": "embed", "vocab_size": cfg.vocab_size, "hidden_size": W, "positions": cfg.position_rows,
            "scale": cfg.embedding_scale, "position_name": "pos"}),
        layers=tuple(layers), schedule=tuple(ScheduleEntry(i) for i in range(len(layers))), final_norm=norm("final.norm"),
        head=PartSpec("lm_head", {"prefix": "head", "vocab_size": cfg.vocab_size, "hidden_size": W, "weight_name": "head"}),
        vocab_size=cfg.vocab_size, hidden_size=W)


# a layer without a feed-forward may still carry the norm of one
register_architecture("Gurapel", "gurapel", GurapelConfig, build_gurapel_spec, tolerated_tensors=(".norm2",))
