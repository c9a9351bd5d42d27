"""A plain, slow implementation of the Zunilorn design: whole sequences, no cache, the recurrence token by token, one
function per mechanism. It shares nothing with the package: it reads a configuration dictionary and a dictionary of
tensors by checkpoint name. ``dtype`` float64 gives the yardstick, float32 what float32 rounding costs; ``storage``
(a torch dtype, None, or a pair (dtype, generator) for another draw of the rounding errors) rounds what an engine may
keep in 16 bits: the operands and results of the projections, the convolution, cached keys and values and the
activations between the products.

Notation: T tokens, width W, n streams X [n, T, W], all equal to E[token] at the start. A sublayer f with the vectors a, b
[n] and the matrix M [n, n] of its own: y = f(norm(sum_s a_s X_s)); X_t <- sum_s M[s, t] X_s + c b_t y, c one constant of
the model. The model ends with the sum of the streams, a norm, the embedding table as head, and a soft cap.
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


def silu(z):
    return z * torch.sigmoid(z)


def linear(x, w, storage, bias=None):
    y = _rt(x, storage) @ w.T
    return _rt(y if bias is None else y + bias, storage)


def linear_wide(x, w, storage):
    """A product whose result stays as it is (it enters a recurrence, a router, or is a gate)."""
    return _rt(x, storage) @ w.T


# ---------------------------------------------------------------- several streams


def read_streams(X, a):
    """X [n, T, W], a [n] -> sum_s a_s X_s."""
    return (X * a.view(-1, 1, 1)).sum(0)


def write_streams(X, M, b, y, c):
    """X_t <- sum_s M[s, t] X_s + c b_t y, all from the old X."""
    return torch.einsum("st,sij->tij", M, X) + c * b.view(-1, 1, 1) * y[None]


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


# ---------------------------------------------------------------- the recurrence with one decay a head


def state_space(x, B, C, dt, A_log, D):
    """Token by token, per head h with the B and C of its group: S <- exp(-exp(A_log_h) dt_h) S + dt_h B x^T;
    y = S^T C + D_h x. x [T, H, dv]; B, C [T, G, N]; dt [T, H] > 0; S [H, N, dv] starts at zero."""
    T, H, dv = x.shape
    G, N = B.shape[1:]
    group = [h // (H // G) for h in range(H)]
    S = torch.zeros(H, N, dv, dtype=x.dtype)
    out = torch.zeros_like(x)
    rate = torch.exp(A_log)
    for t in range(T):
        Bt, Ct = B[t][group], C[t][group]
        S = torch.exp(-rate * dt[t])[:, None, None] * S + (dt[t][:, None] * Bt)[:, :, None] * x[t][:, None, :]
        out[t] = (S * Ct[:, :, None]).sum(1) + D[:, None] * x[t]
    return out


def gated_group_norm(y, z, w, parts, eps):
    """(y silu(z)) cut into equal parts, each over its own root mean square, times w."""
    y = y * silu(z)
    T, n = y.shape
    return rms(y.view(T, parts, n // parts), eps).reshape(T, n) * w


def mamba2(m, tw, p, h, eps, storage):
    T = h.shape[0]
    H, dv, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * dv
    w = tw[p + ".in"]
    z = linear(h, w[:inner], storage)
    u = linear(h, w[inner:2 * inner + 2 * G * N], storage)
    dt = linear_wide(h, w[2 * inner + 2 * G * N:], storage)
    u = _rt(silu(short_conv(u, tw[p + ".conv"], tw[p + ".conv.b"])), storage)
    dt = torch.nn.functional.softplus(dt + tw[p + ".dt_bias"])
    x, B, C = u[:, :inner], u[:, inner:inner + G * N], u[:, inner + G * N:]
    y = state_space(x.view(T, H, dv), B.view(T, G, N), C.view(T, G, N), dt, tw[p + ".A_log"], tw[p + ".D"])
    return linear(gated_group_norm(y.reshape(T, inner), z, tw[p + ".norm"], m["norm_groups"], eps), tw[p + ".o"], storage)


# ---------------------------------------------------------------- attention


def frequencies(rot):
    """Turns per position of every pair, and the factor on cosines and sines."""
    n, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / n) for i in range(n // 2)]
    sc = rot.get("scaling")
    if sc is None:
        return f, 1.0

    def place(t):
        return n * math.log(sc["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(place(sc["fast"])), 0), min(math.ceil(place(sc["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * r + fi * (1.0 - r))
    return out, 0.1 * math.log(sc["factor"]) + 1.0


def rotate(x, rot):
    """x [T, heads, d]: entries i and i + dims / 2 of every head turned by the position times the pair's frequency."""
    f, gain = frequencies(rot)
    half = rot["dims"] // 2
    a = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * torch.tensor(f, dtype=torch.float64)[None, :]
    c, s = (gain * torch.cos(a)).to(x.dtype)[:, None, :], (gain * torch.sin(a)).to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def softmax_with_sink(s, sink):
    """exp(s_j) / (sum_j exp(s_j) + exp(sink)) over the last axis."""
    top = torch.maximum(s.amax(-1, keepdim=True), sink.view(1, 1))
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def attention(m, tw, p, h, storage):
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = linear(h, tw[p + ".q"], storage).view(T, H, d)
    k = linear(h, tw[p + ".k"], storage).view(T, G, d)
    v = linear(h, tw[p + ".v"], storage).view(T, G, dv)
    q, k = _rt(rotate(q, m["rot"]), storage), _rt(rotate(k, m["rot"]), storage)
    pos = torch.arange(T)
    later = pos[None, :] > pos[:, None]
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * m["scale"]
        s = m["softcap"] * torch.tanh(s / m["softcap"])
        out[:, hd] = softmax_with_sink(s.masked_fill(later, float("-inf")), tw[p + ".sink"][hd]) @ v[:, g]
    gate = torch.sigmoid(linear_wide(h, tw[p + ".g"], storage))
    out = _rt(out, storage) * gate[:, :, None]
    return linear(out.reshape(T, H * dv), tw[p + ".o"], storage)


# ---------------------------------------------------------------- feed-forward


def bounded_gate(g, u, limit):
    """g' sigmoid(1.702 g') (u' + 1) with g' = min(g, limit), u' = u within [-limit, limit]."""
    g, u = g.clamp(max=limit), u.clamp(-limit, limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def gated(tw, p, h, limit, storage):
    b = [tw.get("%s.%s.b" % (p, x)) for x in ("gate", "up", "down")]
    a = bounded_gate(linear(h, tw[p + ".gate"], storage, b[0]), linear(h, tw[p + ".up"], storage, b[1]), limit)
    return linear(_rt(a, storage), tw[p + ".down"], storage, b[2])


def choose_experts(logits, correction, top, scale):
    """logits [T, E] -> (the ``top`` experts with the largest softmax score + correction, their scores over the
    chosen ones' sum, times ``scale``)."""
    s = torch.softmax(logits, -1)
    chosen = torch.topk(s + correction, top, -1).indices
    w = torch.gather(s, 1, chosen)
    return chosen, w / (w.sum(-1, keepdim=True) + 1e-20) * scale


def moe(mlp, tw, p, h, storage):
    r = mlp["router"]
    chosen, weight = choose_experts(linear_wide(h, tw[p + ".router"], storage), tw[p + ".correction"], r["top"], r["scale"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        x = h[t:t + 1]
        for k, e in enumerate(chosen[t].tolist()):
            y = gated(tw, "%s.e%d" % (p, e), x, mlp["expert"]["limit"], storage) if e < r["experts"] else _rt(x, storage)
            out[t] = out[t] + weight[t, k] * y[0]
    if mlp.get("shared") is not None:
        own = torch.sigmoid(linear_wide(h, tw[p + ".shared.sg"], storage))
        out = out + own * gated(tw, p + ".shared", h, mlp["shared"]["limit"], storage)
    return _rt(out, storage)


# ---------------------------------------------------------------- the model


def layer_order(cfg):
    n = len(cfg["layers"])
    loop = cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    a, b = loop["start"], loop["stop"]
    return list(range(a)) + list(range(a, b)) * loop["times"] + list(range(b, n))


def forward(cfg, tw, tokens, dtype=torch.float64, storage=None, want_layers=False):
    """Logits [T, vocab] of one whole sequence (and the sum of the streams after every layer run)."""
    tw = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tw.items()}
    eps, c = cfg["norm"]["eps"], cfg["residual_mult"]
    X = tw["embed"][torch.tensor(tokens, dtype=torch.long)][None].repeat(cfg["streams"], 1, 1)
    after = []
    for i in layer_order(cfg):
        layer, p = cfg["layers"][i], "l%d" % i

        def sublayer(X, number, f):
            hc = "%s.hc%d" % (p, number)
            h = _rt(rms(read_streams(X, tw[hc + ".in"]), eps) * tw["%s.norm%d" % (p, number)], storage)
            return write_streams(X, tw[hc + ".mix"], tw[hc + ".out"], f(h), c)

        if layer["type"] == "mamba2":
            X = sublayer(X, 1, lambda h: mamba2(layer["mixer"], tw, p + ".mix", h, eps, storage))
        elif layer["type"] == "attention":
            X = sublayer(X, 1, lambda h: attention(layer["mixer"], tw, p + ".mix", h, storage))
        else:
            raise ValueError(layer["type"])
        mlp = layer.get("mlp")
        if mlp is not None and mlp["kind"] == "dense":
            X = sublayer(X, 2, lambda h: gated(tw, p + ".mlp", h, mlp["limit"], storage))
        elif mlp is not None:
            X = sublayer(X, 2, lambda h: moe(mlp, tw, p + ".mlp", h, storage))
        after.append(X.sum(0))
    x = rms(X.sum(0), eps) * tw["final.norm"]
    z = linear_wide(x, tw["embed"], storage)
    logits = cfg["logit_softcap"] * torch.tanh(z / cfg["logit_softcap"])
    return (logits, torch.stack(after)) if want_layers else logits
