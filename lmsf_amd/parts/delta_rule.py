"""The gated delta rule: a matrix memory of fixed size per request that every token corrects.

q = W_q h and k = W_k h (G heads of ``dim``), v = W_v h (H heads of ``vdim``; head h reads q/k head h // (H / G)); each
passes a short causal convolution over time per channel and SiLU; q and k are made unit vectors per head,
x / sqrt(sum x^2 + 1e-6), q also times dim^-1/2. beta = sigmoid(W_b h), one per head. The decay is
g = exp(-exp(A_log_h) softplus(a + dt_bias)): one per head and key channel, a = W_a2 (W_a1 h) through ``decay_rank``
numbers, or (``decay_rank`` None) one per head, a = W_a h. Per head, token by token:

    S <- g S (rows of S times g);   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q

(the read-out sees the token's own write). Every head's o over its root mean square, times a weight over vdim shared
by the heads, times an activation (``gate_activation``: sigmoid or silu) of a gate as wide as the heads' values,
W_g2 (W_g1 h) through ``gate_rank`` numbers or (None) W_g h; then W_o. A request's state: S [H, dim, vdim] float32 and the
convolutions' last taps - 1 inputs. What enters the recurrence beside the projections and the convolutions (unit
norms, beta, the decays with their softplus and exponentials, S) is float32 (csrc/delta_rule.hip). The reference has no
mixer with state (core/src/model_executor/layers/attention.rs:91-231 is its only mixer).
"""
from typing import Dict, Optional

import torch

from .base import CacheBinding, Mixer, Runtime, StateSpec, register_part
from .linear import FusedLinear, Linear
from .recurrent import FloatVector, ShortConv


@register_part("mixer", "gated_delta")
class GatedDelta(Mixer):
    graph_safe = True
    recordable = False

    def __init__(self, prefix: str, rt: Runtime, hidden_size: int, heads: int, kv_heads: int, dim: int, vdim: int,
                 conv: int, decay_rank: Optional[int], gate_rank: Optional[int], eps: float, unit_eps: float = 1e-6,
                 gate_activation: str = "sigmoid", names: Optional[Dict[str, str]] = None):
        super().__init__(prefix, rt)
        self.H, self.G, self.d, self.dv, self.taps = int(heads), int(kv_heads), int(dim), int(vdim), int(conv)
        if self.H % self.G:
            raise ValueError("%s: heads %d is not a multiple of kv_heads %d" % (prefix, self.H, self.G))
        if self.d > 256:
            raise ValueError("%s: keys of %d entries (at most 256)" % (prefix, self.d))
        self.eps, self.unit_eps = float(eps), float(unit_eps)
        self.per_head, self.full_gate = decay_rank is None, gate_rank is None
        self.ra = 0 if self.per_head else int(decay_rank)
        if gate_activation not in ("sigmoid", "silu"):
            raise ValueError("%s: gate_activation %r (sigmoid, silu)" % (prefix, gate_activation))
        self.gate_activation = gate_activation
        nm = dict(q="q", k="k", v="v", conv="conv", b="b", a="a", a1="a1", a2="a2", dt_bias="dt_bias", a_log="A_log", g="g",
                  g1="g1", g2="g2", norm="norm", out="o")
        nm.update(names or {})
        H, G, d, dv = self.H, self.G, self.d, self.dv
        self.n_qkv = 2 * G * d + H * dv
        self.gate_width = H * dv if self.full_gate else int(gate_rank)
        # one product for everything that reads the layer's input and may be rounded: q | k | v (| a1) | g or g1
        self.proj = FusedLinear(prefix, rt, hidden_size, [(nm["q"], G * d), (nm["k"], G * d), (nm["v"], H * dv)] +
                                ([] if self.per_head else [(nm["a1"], self.ra)]) +
                                [(nm["g"] if self.full_gate else nm["g1"], self.gate_width)], bare_names=True,
                                pad_rows_to=8)
        # and one, with a float32 result, for what enters the recurrence straight from it: beta (and the decay per head)
        self.beta = FusedLinear(prefix, rt, hidden_size, [(nm["b"], H)] + ([(nm["a"], H)] if self.per_head else []),
                                bare_names=True, pad_rows_to=8)
        self.conv = ShortConv(prefix, rt, [("%s.%s" % (nm[x], nm["conv"]), n) for x, n in
                                           (("q", G * d), ("k", G * d), ("v", H * dv))], self.taps, activation="silu")
        self.a2 = None if self.per_head else FusedLinear(prefix, rt, self.ra, [(nm["a2"], H * d)], bare_names=True,
                                                         pad_rows_to=8)
        self.g2 = None if self.full_gate else Linear(prefix, rt, nm["g2"], self.gate_width, H * dv, bare_names=True)
        self.dt_bias = FloatVector("%s.%s" % (prefix, nm["dt_bias"]), rt, (H if self.per_head else H * d,), init="zeros")
        self.a_log = FloatVector("%s.%s" % (prefix, nm["a_log"]), rt, (H,), init="const:0.0")
        self.norm = FloatVector("%s.%s" % (prefix, nm["norm"]), rt, (dv,), init="ones")
        self.o = Linear(prefix, rt, nm["out"], H * dv, hidden_size, bare_names=True)
        sizer = getattr(rt.ops, "gated_delta_state_floats", None)
        self.memory_floats = int(sizer(H, d, dv)) if sizer is not None else H * d * dv

    def children(self):
        return [p for p in (self.proj, self.beta, self.conv, self.a2, self.g2, self.dt_bias, self.a_log, self.norm, self.o)
                if p is not None]

    def state_spec(self) -> Optional[StateSpec]:
        return StateSpec((self.memory_floats + self.conv.state_floats,), torch.float32)

    def forward(self, h: torch.Tensor, ctx, binding: CacheBinding) -> torch.Tensor:
        ops = self.rt.ops
        H, G, d, dv = self.H, self.G, self.d, self.dv
        st = binding.state
        p = self.proj.forward(h)                                              # [N, q | k | v (| a1) | g or g1 | padding]
        qkv = self.conv.forward(p[:, :self.n_qkv], ctx, st[:, self.memory_floats:] if self.taps > 1 else None)
        gate = p[:, self.n_qkv + self.ra:self.n_qkv + self.ra + self.gate_width]
        b = ops.linear_wide(h, self.beta.weight, None)                        # float32: beta before its sigmoid (and a)
        if self.per_head:
            a = b[:, H:2 * H]
        else:
            a = ops.linear_wide(p[:, self.n_qkv:self.n_qkv + self.ra], self.a2.weight, None)   # float32: it enters the decay
        if self.g2 is not None:
            gate = self.g2.forward(gate)
        raw = ops.gated_delta(qkv, 0, G * d, 2 * G * d, a, self.dt_bias.weight, self.a_log.weight, b, st, ctx, H, G, d,
                              dv, d ** -0.5, self.unit_eps, per_head=self.per_head)
        o = ops.head_rms_gate(raw, H, dv, self.eps, self.norm.weight, gate, self.rt.dtype, self.gate_activation)
        return self.o.forward(o)
