"""Mixers whose memory of a request is a state of fixed size: the selective scan, a matrix memory with
exponential gates, a gated linear recurrence and a recurrence of matrices with one decay a head, and the short causal
convolution that both they and some attention layers put behind a projection.

A request's state is one row of float32 numbers in the engine's state slots (``StateSpec``); a mixer says how
many it needs and gets ``binding.state`` [slots, that many]. The engine clears a row when a request takes it, so
"zeros before the sequence's start" and "the state starts at zero" need no code here. Everything that enters a
recurrence is float32 (csrc/recurrent.hip, csrc/linear_recurrence.hip, csrc/state_space.hip); the projections run in the run's dtype. The reference has no mixer
with state (its only one is attention over a paged cache, core/src/model_executor/layers/attention.rs:91-231).
"""
from typing import Callable, Dict, Optional, Sequence, Tuple

import torch

from .base import CacheBinding, Mixer, Part, Runtime, StateSpec, TensorDecl, register_part
from .linear import FusedLinear, Linear


class ShortConv(Part):
    """Causal convolution over time, a filter of ``taps`` per channel: y_t = sum_j w[:, j] u_(t - taps + 1 + j)
    (+ bias), zeros before a request's start. ``sources``: (checkpoint name under the prefix, channels) of the
    filters, laid side by side as one [C, taps] tensor; ``bias_name``: the name of a bias of C entries, or None.
    The last taps - 1 inputs of every request are its state: ``state_floats`` numbers."""

    graph_safe = True
    recordable = False

    def __init__(self, prefix: str, rt: Runtime, sources: Sequence[Tuple[str, int]], taps: int,
                 bias_name: Optional[str] = None, activation: Optional[str] = None):
        super().__init__(prefix, rt)
        self.sources = [(str(n), int(c)) for n, c in sources]
        self.channels = sum(c for _, c in self.sources)
        self.taps = int(taps)
        if self.taps < 1:
            raise ValueError("%s: a convolution needs at least one tap" % prefix)
        self.bias_name = bias_name
        self.activation = activation
        self.state_floats = self.channels * (self.taps - 1)
        self.weight: Optional[torch.Tensor] = None
        self.bias: Optional[torch.Tensor] = None

    def _full(self, name: str) -> str:
        return "%s.%s" % (self.prefix, name)

    def checkpoint_tensors(self) -> Dict[str, TensorDecl]:
        out = {self._full(n): TensorDecl((c, self.taps), init="normal:0.3") for n, c in self.sources}
        if self.bias_name:
            out[self._full(self.bias_name)] = TensorDecl((self.channels,), init="zeros")
        return out

    def load_weights(self, fetch: Callable[[str], torch.Tensor]) -> None:
        parts = [fetch(self._full(n)) for n, _ in self.sources]
        self.weight = (parts[0] if len(parts) == 1 else torch.cat(parts, 0)).to(self.rt.dtype).contiguous()
        if self.bias_name:
            self.bias = fetch(self._full(self.bias_name)).to(self.rt.dtype).contiguous()

    def forward(self, u: torch.Tensor, ctx, state: Optional[torch.Tensor]) -> torch.Tensor:
        return self.rt.ops.short_conv(u, self.weight, self.bias, state, ctx, self.activation)


class FloatVector(Part):
    """A checkpoint tensor that is kept in float32 whatever the run's dtype (what enters a recurrence); ``transform``:
    what is kept is this function of it."""

    graph_safe = True

    def __init__(self, name: str, rt: Runtime, shape: Tuple[int, ...], init: str = "normal",
                 transform: Optional[Callable[[torch.Tensor], torch.Tensor]] = None):
        super().__init__(name, rt)
        self.transform = transform
        self.shape, self.init = tuple(shape), init
        self.weight: Optional[torch.Tensor] = None

    def checkpoint_tensors(self) -> Dict[str, TensorDecl]:
        return {self.prefix: TensorDecl(self.shape, init=self.init, keeps_float32=True)}

    def load_weights(self, fetch: Callable[[str], torch.Tensor]) -> None:
        w = fetch(self.prefix).to(torch.float32)
        self.weight = (self.transform(w) if self.transform is not None else w).contiguous()


@register_part("mixer", "selective_scan")
class SelectiveScan(Mixer):
    """Mamba's mixer. [x | z] = W_in h; x <- silu(conv(x) + b); [dt | B | C] = W_x x; dt <- softplus(W_dt dt + b_dt);
    A = -exp(A_log);  S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n;  y_c = sum_n S[c, n] C_n + D_c x_c;
    out = W_o (y * silu(z)). State of a request: S [inner, state] and the convolution's last taps - 1 inputs."""

    graph_safe = True
    recordable = False

    def __init__(self, prefix: str, rt: Runtime, hidden_size: int, inner: int, state: int, dt_rank: int, conv: int,
                 names: Optional[Dict[str, str]] = None):
        super().__init__(prefix, rt)
        self.inner, self.n, self.rank, self.taps = int(inner), int(state), int(dt_rank), int(conv)
        if min(self.inner, self.n, self.rank, self.taps) < 1:
            raise ValueError("%s: sizes must be positive" % prefix)
        nm = dict(in_proj="in", conv="conv", conv_bias="conv.b", x_proj="x", dt_proj="dt", a_log="A_log", d="D", out="o")
        nm.update(names or {})
        self.in_proj = Linear(prefix, rt, nm["in_proj"], hidden_size, 2 * self.inner, bare_names=True)
        self.conv = ShortConv(prefix, rt, [(nm["conv"], self.inner)], self.taps, bias_name=nm["conv_bias"],
                              activation="silu")
        self.x_proj = Linear(prefix, rt, nm["x_proj"], self.inner, self.rank + 2 * self.n, bare_names=True)
        self.dt_proj = Linear(prefix, rt, nm["dt_proj"], self.rank, self.inner, bias=True, bare_names=True, bias_name="b")
        self.a_log = FloatVector("%s.%s" % (prefix, nm["a_log"]), rt, (self.inner, self.n), init="const:0.0")
        self.d = FloatVector("%s.%s" % (prefix, nm["d"]), rt, (self.inner,), init="ones")
        self.o = Linear(prefix, rt, nm["out"], self.inner, hidden_size, bare_names=True)
        self.scan_floats = self.inner * self.n

    def children(self):
        return [self.in_proj, self.conv, self.x_proj, self.dt_proj, self.a_log, self.d, self.o]

    def state_spec(self) -> Optional[StateSpec]:
        return StateSpec((self.scan_floats + self.conv.state_floats,), torch.float32)

    def forward(self, h: torch.Tensor, ctx, binding: CacheBinding) -> torch.Tensor:
        ops = self.rt.ops
        st = binding.state
        xz = self.in_proj.forward(h)                                            # [N, 2 inner]
        x = self.conv.forward(xz[:, :self.inner], ctx, st[:, self.scan_floats:] if self.taps > 1 else None)
        low = self.x_proj.forward(x)                                            # [N, rank + 2 n]: dt, B, C
        dt = ops.linear_wide(low[:, :self.rank], self.dt_proj.weight, self.dt_proj.bias)   # float32: a step size
        y = ops.selective_scan(x, dt, low, self.rank, self.rank + self.n, xz[:, self.inner:], self.a_log.weight,
                               self.d.weight, st, ctx)
        return self.o.forward(y)


@register_part("mixer", "matrix_memory")
class MatrixMemory(Mixer):
    """The matrix memory of xLSTM (mLSTM). q = W_q h * dim^-1/2, k = W_k h, v = W_v h per head; log gates
    i = cap tanh((W_i h + b_i) / cap), f = logsigmoid(cap tanh((W_f h + b_f) / cap)); with a running maximum m that
    starts at 0:  m' = max(f + m, i);  S <- exp(f + m - m') S + exp(i - m') k v^T;  n likewise with k alone;
    o = S^T q / (max(|n . q|, exp(-m')) + 1e-6). Every head's o over its root mean square, times a weight over all
    heads, times sigmoid(W_g h), then W_o. State of a request: S, n and m of every head."""

    graph_safe = True
    recordable = False

    def __init__(self, prefix: str, rt: Runtime, hidden_size: int, heads: int, dim: int, vdim: int, gate_cap: float,
                 eps: float, names: Optional[Dict[str, str]] = None):
        super().__init__(prefix, rt)
        self.H, self.d, self.dv = int(heads), int(dim), int(vdim)
        self.cap, self.eps = float(gate_cap), float(eps)
        if not self.cap > 0:
            raise ValueError("%s: gate_cap must be > 0" % prefix)
        nm = dict(q="q", k="k", v="v", g="g", i="i", f="f", norm="norm", out="o")
        nm.update(names or {})
        H, d, dv = self.H, self.d, self.dv
        self.qkvg = FusedLinear(prefix, rt, hidden_size, [(nm["q"], H * d), (nm["k"], H * d), (nm["v"], H * dv),
                                                          (nm["g"], H * dv)], bare_names=True)
        self.gates = FusedLinear(prefix, rt, hidden_size, [(nm["i"], H), (nm["f"], H)], bias=True, bare_names=True,
                                 bias_name="b")
        self.norm = FloatVector("%s.%s" % (prefix, nm["norm"]), rt, (H * dv,), init="ones")
        self.o = Linear(prefix, rt, nm["out"], H * dv, hidden_size, bare_names=True)
        sizer = getattr(rt.ops, "mlstm_state_floats", None)
        self.state_floats = int(sizer(H, d, dv)) if sizer is not None else H * d * (dv + 1) + H

    def children(self):
        return [self.qkvg, self.gates, self.norm, self.o]

    def state_spec(self) -> Optional[StateSpec]:
        return StateSpec((self.state_floats,), torch.float32)

    def forward(self, h: torch.Tensor, ctx, binding: CacheBinding) -> torch.Tensor:
        ops = self.rt.ops
        H, d, dv = self.H, self.d, self.dv
        p = self.qkvg.forward(h)
        gates = ops.linear_wide(h, self.gates.weight, self.gates.bias)                         # float32 [N, 2 H]
        o = ops.mlstm(p[:, :H * d], p[:, H * d:2 * H * d], p[:, 2 * H * d:2 * H * d + H * dv], gates,
                      p[:, 2 * H * d + H * dv:], self.norm.weight, binding.state, ctx, H, d, dv, d ** -0.5, self.cap,
                      self.eps)
        return self.o.forward(o)


@register_part("mixer", "gated_linear_recurrence")
class GatedLinearRecurrence(Mixer):
    """Griffin's recurrent block with a real-gated linear recurrence. Two branches of C = ``width`` channels,
    y = gelu_tanh(W_y h + b_y) and u = conv(W_x h + b_x) + b_c (no activation). u is cut into ``blocks`` equal parts, each
    with its own square matrices: r = sigmoid(W_r u + b_r), i = sigmoid(W_i u + b_i). log a = -decay * r * softplus(lam);
    S <- a S + sqrt(1 - a^2) i u; out = W_o (S * y). State of a request: S [C] and the convolution's last taps - 1 inputs."""

    graph_safe = True
    recordable = False

    def __init__(self, prefix: str, rt: Runtime, hidden_size: int, width: int, blocks: int, conv: int, decay: float = 8.0,
                 names: Optional[Dict[str, str]] = None):
        super().__init__(prefix, rt)
        self.C, self.blocks, self.taps, self.decay = int(width), int(blocks), int(conv), float(decay)
        if self.blocks < 1 or self.C % self.blocks:
            raise ValueError("%s: %d channels do not split into %d blocks" % (prefix, self.C, self.blocks))
        nm = dict(y="y", x="x", bias="b", conv="conv", conv_bias="conv.b", r="ra", r_bias="ra.b", i="ri", i_bias="ri.b",
                  lam="lam", out="o")
        nm.update(names or {})
        self.proj = FusedLinear(prefix, rt, hidden_size, [(nm["y"], self.C), (nm["x"], self.C)], bias=True,
                                bare_names=True, bias_name=nm["bias"])
        self.conv = ShortConv(prefix, rt, [(nm["conv"], self.C)], self.taps, bias_name=nm["conv_bias"])
        self.o = Linear(prefix, rt, nm["out"], self.C, hidden_size, bare_names=True)
        self.names = {k: "%s.%s" % (prefix, nm[k]) for k in ("r", "r_bias", "i", "i_bias", "lam")}
        self.wr: Optional[torch.Tensor] = None       # [blocks, C / blocks, C / blocks]
        self.wi: Optional[torch.Tensor] = None
        self.br: Optional[torch.Tensor] = None       # float32 [C]
        self.bi: Optional[torch.Tensor] = None
        self.rate: Optional[torch.Tensor] = None     # float32 [C]: decay * softplus(lam)

    def children(self):
        return [self.proj, self.conv, self.o]

    def checkpoint_tensors(self) -> Dict[str, TensorDecl]:
        c = self.C // self.blocks
        nm = self.names
        return {nm["r"]: TensorDecl((self.blocks, c, c)), nm["i"]: TensorDecl((self.blocks, c, c)),
                nm["r_bias"]: TensorDecl((self.blocks, c), init="zeros", keeps_float32=True),
                nm["i_bias"]: TensorDecl((self.blocks, c), init="zeros", keeps_float32=True),
                nm["lam"]: TensorDecl((self.C,), init="const:-2.0", keeps_float32=True)}

    def load_weights(self, fetch: Callable[[str], torch.Tensor]) -> None:
        nm = self.names
        self.wr, self.wi = (fetch(nm[k]).to(self.rt.dtype).contiguous() for k in ("r", "i"))
        self.br, self.bi = (fetch(nm[k]).to(torch.float32).reshape(-1).contiguous() for k in ("r_bias", "i_bias"))
        self.rate = (self.decay * torch.nn.functional.softplus(fetch(nm["lam"]).to(torch.float32))).contiguous()

    def tensors(self):
        return [t for t in (self.wr, self.wi, self.br, self.bi, self.rate) if t is not None]

    def state_spec(self) -> Optional[StateSpec]:
        return StateSpec((self.C + self.conv.state_floats,), torch.float32)

    def forward(self, h: torch.Tensor, ctx, binding: CacheBinding) -> torch.Tensor:
        st = binding.state
        p = self.proj.forward(h)                                                # [N, y | x]
        u = self.conv.forward(p[:, self.C:], ctx, st[:, self.C:] if self.taps > 1 else None)
        o = self.rt.ops.linear_recurrence(u, self.wr, self.br, self.wi, self.bi, self.rate, p[:, :self.C], st, ctx)
        return self.o.forward(o)


@register_part("mixer", "state_space")
class StateSpace(Mixer):
    """Mamba-2's mixer. inner = heads * vdim; [z | x | B | C | dt] = W_in h with B and C of ``groups`` groups of ``state``
    entries and one dt a head; [x | B | C] <- silu(conv(.) + b); dt <- softplus(dt + dt_bias). Per head, with B and C of
    its group: S <- exp(-exp(A_log) dt) S + dt B x^T, y = S^T C + D x. The heads' y, concatenated, times silu(z), then an
    RMS norm in ``norm_groups`` equal parts times a weight, then W_o. State of a request: S of every head and the
    convolution's last taps - 1 inputs."""

    graph_safe = True
    recordable = False

    def __init__(self, prefix: str, rt: Runtime, hidden_size: int, heads: int, vdim: int, state: int, groups: int, conv: int,
                 eps: float, norm_groups: int = 1, names: Optional[Dict[str, str]] = None):
        super().__init__(prefix, rt)
        self.H, self.dv, self.n, self.G, self.taps = int(heads), int(vdim), int(state), int(groups), int(conv)
        self.norm_groups, self.eps = int(norm_groups), float(eps)
        self.inner = self.H * self.dv
        if min(self.H, self.dv, self.n, self.G, self.taps, self.norm_groups) < 1 or self.H % self.G \
                or self.inner % self.norm_groups or self.n > 1024:
            raise ValueError("%s: %d heads of %d x %d (states of at most 1,024 rows) in %d groups, normed in %d parts"
                             % (prefix, self.H, self.n, self.dv, self.G, self.norm_groups))
        nm = dict(in_proj="in", conv="conv", conv_bias="conv.b", dt_bias="dt_bias", a_log="A_log", d="D", norm="norm",
                  out="o")
        nm.update(names or {})
        self.channels = self.inner + 2 * self.G * self.n
        self.n_main = self.inner + self.channels          # z | x | B | C: a product in the run's type; dt's is float32
        self.in_proj = Linear(prefix, rt, nm["in_proj"], hidden_size, self.n_main + self.H, bare_names=True, pad_rows_to=8)
        self.conv = ShortConv(prefix, rt, [(nm["conv"], self.channels)], self.taps, bias_name=nm["conv_bias"],
                              activation="silu")
        self.dt_bias = FloatVector("%s.%s" % (prefix, nm["dt_bias"]), rt, (self.H,), init="zeros")
        self.rate = FloatVector("%s.%s" % (prefix, nm["a_log"]), rt, (self.H,), init="const:0.0", transform=torch.exp)
        self.d = FloatVector("%s.%s" % (prefix, nm["d"]), rt, (self.H,), init="ones")
        self.norm = FloatVector("%s.%s" % (prefix, nm["norm"]), rt, (self.inner,), init="ones")
        self.o = Linear(prefix, rt, nm["out"], self.inner, hidden_size, bare_names=True)
        sizer = getattr(rt.ops, "state_space_state_floats", None)
        floats = int(sizer(self.H, self.n, self.dv)) if sizer is not None else self.H * self.n * self.dv
        self.state_floats = (floats + 3) // 4 * 4         # (the convolution's part begins at a multiple of 16 bytes)

    def children(self):
        return [self.in_proj, self.conv, self.dt_bias, self.rate, self.d, self.norm, self.o]

    def state_spec(self) -> Optional[StateSpec]:
        total = self.state_floats + self.conv.state_floats
        return StateSpec(((total + 3) // 4 * 4,), torch.float32)

    def forward(self, h: torch.Tensor, ctx, binding: CacheBinding) -> torch.Tensor:
        ops = self.rt.ops
        st = binding.state
        w = self.in_proj.weight
        p = ops.linear(h, w[:self.n_main])                                       # [N, z | x | B | C]
        dt = ops.linear_wide(h, w[self.n_main:], None)                           # float32 [N, >= H]: step sizes
        u = self.conv.forward(p[:, self.inner:], ctx, st[:, self.state_floats:] if self.taps > 1 else None)
        b_at = self.inner
        y = ops.state_space(u, 0, b_at, b_at + self.G * self.n, dt, self.dt_bias.weight, self.rate.weight, self.d.weight, st, ctx,
                            self.H, self.G, self.n, self.dv)
        return self.o.forward(ops.gated_group_norm(y, p[:, :self.inner], self.norm.weight, self.norm_groups, self.eps))
