"""A plain, slow implementation of the Gurapel design: whole sequences, no cache, recurrences token by token, one
function per mechanism. It shares nothing with the package: it reads a configuration dictionary and a dictionary of
tensors by checkpoint name. ``dtype`` float64 gives the yardstick, float32 what float32 rounding costs; ``storage``
(a torch dtype, None, or a pair (dtype, generator) for another draw of the rounding errors) rounds what an engine may
keep in 16 bits: the operands and results of the projections, the convolutions and the activations between them.

Notation: T tokens, width W. x_0 = scale * E[token] + P[position]; a layer is x += n1(mixer(x)); x += n2(ffn(x)), both
sublayers reading the stream as it is, every n an RMS norm whose stored weight w acts as 1 + w.
"""
import math

import torch


def _rt(x, storage):
    """Round to the storage type and back. ``storage`` may be (type, generator): the value is first moved by up to
    half a bfloat16 step at random, which gives another draw of the rounding errors."""
    if storage is None:
        return x
    if isinstance(storage, tuple):
        storage, gen = storage
        x = x * (1.0 + (torch.rand(x.shape, generator=gen, dtype=torch.float32).to(x.dtype) - 0.5) * 2.0 ** -8)
    return x.to(storage).to(x.dtype)


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_one_plus(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def linear(x, w, storage, bias=None):
    y = _rt(x, storage) @ w.T
    return _rt(y if bias is None else y + bias, storage)


def linear_wide(x, w, storage):
    """A product whose result stays as it is (it enters a recurrence or a router)."""
    return _rt(x, storage) @ w.T


# ---------------------------------------------------------------- embedding


def embed(cfg, tw, tokens, dtype):
    ids = torch.tensor(tokens, dtype=torch.long)
    return tw["embed"].to(dtype)[ids] * cfg["embedding"]["scale"] + tw["pos"].to(dtype)[:len(tokens)]


# ---------------------------------------------------------------- short convolution


def short_conv(u, w, bias=None):
    """Causal filter per channel, zeros before the start. u [T, C], w [C, taps]; the last tap is the current token's."""
    T, C = u.shape
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, C, dtype=u.dtype), u], 0)
    y = torch.zeros_like(u)
    for j in range(taps):
        y = y + padded[j:j + T] * w[:, j][None, :]
    return y if bias is None else y + bias


# ---------------------------------------------------------------- attention


def distance_bias(r1, r2, diff):
    """What is taken off a score at distance ``diff`` >= 0, per head: r1 ln(1 + r2 diff) [H, ...]."""
    shape = (-1,) + (1,) * diff.dim()
    return r1.view(shape) * torch.log(1.0 + r2.view(shape) * diff.clamp(min=0).to(r1.dtype)[None])


def attention(m, tw, p, h, eps, storage):
    T = h.shape[0]
    dt = h.dtype
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = linear(h, tw[p + ".q"], storage).view(T, H, d)
    k = linear(h, tw[p + ".k"], storage).view(T, G, d)
    v = linear(h, tw[p + ".v"], storage).view(T, G, dv)
    q = _rt(rms(q, eps) * tw[p + ".q.norm"].to(dt), storage)
    k = _rt(rms(k, eps) * tw[p + ".k.norm"].to(dt), storage)
    pos = torch.arange(T)
    diff = pos[:, None] - pos[None, :]
    seen = (diff >= 0) & (diff < m["mask"]["size"])
    off = distance_bias(tw[p + ".r1"].to(dt), tw[p + ".r2"].to(dt), diff)
    out = torch.zeros(T, H, dv, dtype=dt)
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * m["scale"]
        s = m["softcap"] * torch.tanh(s / m["softcap"]) - off[hd]
        out[:, hd] = torch.softmax(s.masked_fill(~seen, float("-inf")), -1) @ v[:, g]
    return linear(out.reshape(T, H * dv), tw[p + ".o"], storage)


# ---------------------------------------------------------------- the gated linear recurrence


def block_linear(u, w, b):
    """u [T, C] cut into w.shape[0] equal parts, each through its own square matrix [out, in]; b [blocks, C / blocks]."""
    n, c, _ = w.shape
    parts = [u[:, i * c:(i + 1) * c] @ w[i].T + b[i] for i in range(n)]
    return torch.cat(parts, -1)


def gated_linear_recurrence(u, r_pre, i_pre, lam):
    """S_t = a_t S_(t-1) + sqrt(1 - a_t^2) sigmoid(i_pre) u with log a = -8 sigmoid(r_pre) softplus(lam); S_0 = 0.
    u, r_pre, i_pre [T, C]; returns every S_t."""
    log_a = -8.0 * torch.sigmoid(r_pre) * torch.nn.functional.softplus(lam)[None, :]
    a = torch.exp(log_a)
    b = torch.sqrt(-torch.expm1(2.0 * log_a)) * torch.sigmoid(i_pre) * u
    S = torch.zeros(u.shape[1], dtype=u.dtype)
    out = torch.zeros_like(u)
    for t in range(u.shape[0]):
        S = a[t] * S + b[t]
        out[t] = S
    return out


def griffin(m, tw, p, h, storage):
    dt = h.dtype
    y = _rt(gelu_tanh(linear(h, tw[p + ".y"], storage, tw[p + ".y.b"])), storage)
    x = linear(h, tw[p + ".x"], storage, tw[p + ".x.b"])
    u = _rt(short_conv(x, tw[p + ".conv"], tw[p + ".conv.b"]), storage)
    S = gated_linear_recurrence(u, block_linear(u, tw[p + ".ra"], tw[p + ".ra.b"]),
                                block_linear(u, tw[p + ".ri"], tw[p + ".ri.b"]), tw[p + ".lam"].to(dt))
    return linear(S * y, tw[p + ".o"], storage)


def parallel(m, tw, p, h, eps, storage):
    a = attention(m["left"], tw, p + ".left", h, eps, storage)
    b = griffin(m["right"], tw, p + ".right", h, storage)
    return 0.5 * (rms(a, eps) * tw[p + ".left.out"] + rms(b, eps) * tw[p + ".right.out"])


# ---------------------------------------------------------------- delta rule


def delta_rule(q, k, v, beta, decay):
    """Per head, token by token: S <- decay_t S; u = beta_t (v_t - S^T k_t); S <- S + k_t u^T; o_t = S^T q_t.
    q, k [T, H, d]; v [T, H, dv]; beta, decay [T, H]. S starts at zero."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = S * decay[t][:, None, None]
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta(m, tw, p, h, eps, storage):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]

    def branch(name):
        return _rt(silu(short_conv(linear(h, tw[p + "." + name], storage), tw[p + "." + name + ".conv"])), storage)

    q, k, v = branch("q").view(T, G, d), branch("k").view(T, G, d), branch("v").view(T, H, dv)
    q, k = unit(q) * d ** -0.5, unit(k)
    rep = H // G
    beta = torch.sigmoid(linear_wide(h, tw[p + ".b"], storage))
    step = torch.nn.functional.softplus(linear_wide(h, tw[p + ".a"], storage) + tw[p + ".dt_bias"])
    decay = torch.exp(-torch.exp(tw[p + ".A_log"])[None, :] * step)
    o = delta_rule(q.repeat_interleave(rep, 1), k.repeat_interleave(rep, 1), v, beta, decay)
    gate = silu(linear(h, tw[p + ".g"], storage)).view(T, H, dv)
    o = _rt(rms(o, eps) * tw[p + ".norm"] * gate, storage)
    return linear(o.reshape(T, H * dv), tw[p + ".o"], storage)


# ---------------------------------------------------------------- feed-forward


def choose_experts(logits, top):
    """logits [T, E] -> (the ``top`` largest experts, the softmax over their logits alone)."""
    z, chosen = torch.topk(logits, top, -1)
    return chosen, torch.softmax(z, -1)


def expert(tw, p, h, storage):
    a = _rt(silu(linear(h, tw[p + ".gate"], storage)) * linear(h, tw[p + ".up"], storage), storage)
    return linear(a, tw[p + ".down"], storage)


def moe(mlp, tw, p, h, storage):
    chosen, weight = choose_experts(linear_wide(h, tw[p + ".router"], storage), mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for k, e in enumerate(chosen[t].tolist()):
            out[t] = out[t] + weight[t, k] * expert(tw, "%s.e%d" % (p, e), h[t:t + 1], storage)[0]
    return _rt(out, storage)


# ---------------------------------------------------------------- the model


def forward(cfg, tw, tokens, dtype=torch.float64, storage=None, want_layers=False):
    """Logits [T, vocab] of one whole sequence (and the stream after every layer)."""
    tw = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tw.items()}
    eps = cfg["norm"]["eps"]
    x = embed(cfg, tw, tokens, dtype)
    streams = []
    for i, layer in enumerate(cfg["layers"]):
        p = "l%d" % i
        h = _rt(x, storage)
        if layer["type"] == "parallel":
            a = parallel(layer["mixer"], tw, p + ".mix", h, eps, storage)
        elif layer["type"] == "delta":
            a = delta(layer["mixer"], tw, p + ".mix", h, eps, storage)
        else:
            raise ValueError(layer["type"])
        x = x + norm_one_plus(_rt(a, storage), tw[p + ".norm1"], eps)
        if layer.get("mlp") is not None:
            x = x + norm_one_plus(moe(layer["mlp"], tw, p + ".mlp", _rt(x, storage), storage), tw[p + ".norm2"], eps)
        streams.append(x.clone())
    logits = linear_wide(norm_one_plus(x, tw["final.norm"], eps), tw["head"], storage)
    return (logits, torch.stack(streams)) if want_layers else logits
