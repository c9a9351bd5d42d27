"""Gated feed-forward: y = (act(x Wg^T) * (x Wu^T)) Wd^T; act is SiLU, GELU or the tanh form of GELU; or, "bounded",
the activation g sigmoid(1.702 g) (u + 1) with g = min(x Wg^T, limit), u = x Wu^T within [-limit, limit].

core/src/model_executor/models/llama/llama.rs:223-274: gate and up are one fused product of 2 I
rows (gate first), then silu_and_mul (vllm/kernels/activation_kernels.cu:26-42), then down.
"""
import torch

from .base import FeedForward, Runtime, register_part
from .linear import FusedLinear, Linear


@register_part("feed_forward", "gated_mlp")
class GatedMLP(FeedForward):
    graph_safe = True

    def __init__(self, prefix: str, rt: Runtime, hidden_size: int, intermediate_size: int, activation: str = "silu",
                 bias: bool = False, gate_name: str = "gate_proj", up_name: str = "up_proj",
                 down_name: str = "down_proj", bare_names: bool = False, bias_name: str = "bias", limit: float = 0.0):
        super().__init__(prefix, rt)
        if activation not in ("silu", "gelu", "gelu_tanh", "bounded"):
            raise ValueError("gated_mlp activation %r unknown (silu, gelu, gelu_tanh, bounded)" % activation)
        self.activation, self.limit = activation, float(limit)
        if (activation == "bounded") != (self.limit > 0):
            raise ValueError("gated_mlp: a limit > 0 goes with the activation 'bounded'")
        if activation == "bounded":      # (the recorded step program has no such activation)
            self.recordable = False
        self.gate_up = FusedLinear(prefix, rt, hidden_size,
                                   [(gate_name, intermediate_size), (up_name, intermediate_size)], bias=bias,
                                   bare_names=bare_names, bias_name=bias_name)
        self.down = Linear(prefix, rt, down_name, intermediate_size, hidden_size, bias=bias, bare_names=bare_names,
                           bias_name=bias_name)

    def children(self):
        return [self.gate_up, self.down]

    may_return_pending = True
    accepts_normed = True

    def forward(self, h: torch.Tensor, pending_ok: bool = False):
        if self.limit > 0:
            a = self.rt.ops.linear_gated(h, self.gate_up.weight, self.gate_up.bias, self.activation, limit=self.limit)
        else:
            a = self.rt.ops.linear_gated(h, self.gate_up.weight, self.gate_up.bias, self.activation)
        return self.down.forward(a, pending_ok=pending_ok)


@register_part("feed_forward", "plain_mlp")
class PlainMLP(FeedForward):
    """y = W_down act(W_up x), one matrix in and one out; act is the square of relu. The reference's feed-forward is the
    gated one above."""

    graph_safe = True
    recordable = False

    def __init__(self, prefix: str, rt: Runtime, hidden_size: int, intermediate_size: int,
                 activation: str = "relu_squared", up_name: str = "up", down_name: str = "down", bare_names: bool = True):
        super().__init__(prefix, rt)
        if activation != "relu_squared":
            raise ValueError("plain_mlp activation %r unknown (relu_squared)" % activation)
        self.up = Linear(prefix, rt, up_name, hidden_size, intermediate_size, bare_names=bare_names)
        self.down = Linear(prefix, rt, down_name, intermediate_size, hidden_size, bare_names=bare_names)

    def children(self):
        return [self.up, self.down]

    def forward(self, h: torch.Tensor):
        return self.down.forward(self.rt.ops.relu_squared(self.up.forward(h)))
