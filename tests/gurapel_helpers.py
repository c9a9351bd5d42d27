"""Small Gurapel configurations and random weights by checkpoint name, made without the package's help, for the tests
that compare the engine with the plain implementation (plain_gurapel.py)."""
import json
import math
import os

import torch
from safetensors.torch import save_file

import plain_gurapel as P
from takosun_helpers import rel_err, replay, row_errs, within  # noqa: F401  (shared measures, re-exported)


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def pair(heads, kv_heads, dim, vdim, window, width, blocks, conv, scale=None, softcap=20.0, mlp=None):
    return {"type": "parallel", "mlp": mlp, "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5,
                 "softcap": softcap, "mask": {"size": window}},
        "right": {"width": width, "blocks": blocks, "conv": conv}}}


def delta(heads, kv_heads, dim, vdim, conv, mlp=None):
    return {"type": "delta", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                                   "conv": conv}}


def model(vocab, width, layers, eps=1e-5, scale=1.0, positions=512):
    return {"architecture": "Gurapel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "max_positions": positions, "layers": layers}


# Sizes differ between the configurations and inside each: one to six heads with one to five heads of keys, values wider
# and narrower than keys, sizes that are multiples of nothing, windows of 1 to 200 positions that are no multiples of a
# page, weak and strong caps, one block of channels and as many blocks as channels, filters of one to five taps, one to
# all of the experts, layers without a feed-forward, a model without the delta rule and one without attention.
CONFIGS = {
    "A": model(61, 48, [
        pair(4, 2, 12, 20, 11, 24, 3, 3, scale=0.3, softcap=5.0, mlp=moe(6, 2, 16)),
        delta(3, 1, 8, 12, 3, mlp=moe(4, 1, 12)),
        pair(2, 1, 16, 8, 40, 40, 1, 1),
    ], scale=0.7),
    "B": model(77, 64, [      # pages and the linear recurrence; windows of three sizes
        pair(1, 1, 24, 24, 1, 12, 12, 2, mlp=moe(3, 3, 20)),
        pair(6, 3, 4, 8, 19, 64, 2, 5, softcap=50.0),
        pair(5, 5, 7, 5, 7, 20, 4, 4, scale=0.5, softcap=2.0, mlp=moe(5, 2, 9)),
    ], eps=1e-6, scale=2.0),
    "C": model(40, 32, [      # state only: no pages at all
        delta(2, 2, 12, 12, 4, mlp=moe(8, 3, 16)),
        delta(1, 1, 20, 6, 5),
    ], scale=0.25, positions=300),
    "D": model(53, 40, [
        delta(4, 2, 8, 8, 1, mlp=moe(2, 1, 8)),
        pair(2, 2, 20, 16, 13, 30, 5, 2, mlp=moe(7, 4, 10)),
    ]),
    # sizes at which the matrix-core forms of the kernels run (GPU tests)
    "M": model(300, 256, [
        pair(4, 2, 64, 64, 50, 192, 3, 4, scale=0.125, softcap=30.0, mlp=moe(8, 2, 128)),
        delta(4, 2, 64, 128, 4, mlp=moe(6, 3, 64)),
        pair(16, 1, 128, 96, 90, 256, 2, 3, softcap=15.0, mlp=moe(8, 8, 64)),
        pair(3, 3, 80, 112, 200, 96, 3, 2, mlp=moe(4, 1, 256)),
    ]),
}


def make_weights(cfg, seed, spread=1.0, decisive=False):
    """Matrices N(0, 1 / inputs) (the weights of the queries' norm ``spread`` times larger, so that attention is peaked
    for spread > 1); norm weights of the layers around 0 (they act as 1 + w), the others around 1; distance biases and
    decays that differ from head to head and channel to channel; routers wide enough that the logits differ.

    ``decisive``: no choice of experts is a close call, so that rounding cannot flip one (a flipped choice moves a row,
    and every later row, by far more than rounding; bfloat16 runs are compared under such weights, float32 runs under
    the random routers). The last E entries of the stream (E: the most experts of a layer) hold a code of the token
    id, distinct levels in an order that turns with the id; no sublayer and no position vector writes to them; expert
    e's router row reads entry e with a large factor beside small random entries."""
    g = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]
    w = {}

    def mat(name, rows, cols, s=1.0):
        w[name] = torch.randn((rows, cols), generator=g) * (s / math.sqrt(cols))

    def around(name, n, centre=1.0, dev=0.2):
        w[name] = centre + dev * torch.randn((n,), generator=g)

    def between(name, n, lo, hi):
        w[name] = lo + (hi - lo) * torch.rand((n,), generator=g)

    w["embed"] = torch.randn((V, W), generator=g) / cfg["embedding"]["scale"]
    w["pos"] = torch.randn((cfg["max_positions"], W), generator=g) * 0.4
    for i, lay in enumerate(cfg["layers"]):
        p, m, q = "l%d" % i, lay["mixer"], "l%d.mix" % i
        around(p + ".norm1", W, 0.0)
        if lay["type"] == "parallel":
            a, b = m["left"], m["right"]
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            left, right = q + ".left", q + ".right"
            mat(left + ".q", H * d, W), mat(left + ".k", G * d, W), mat(left + ".v", G * dv, W)
            around(left + ".q.norm", d, spread), around(left + ".k.norm", d)
            between(left + ".r1", H, 0.1, 1.5), between(left + ".r2", H, 0.05, 0.8)
            mat(left + ".o", W, H * dv)
            C, n = b["width"], b["blocks"]
            c = C // n
            for x in ("y", "x"):
                mat("%s.%s" % (right, x), C, W)
                around("%s.%s.b" % (right, x), C, 0.0)
            w[right + ".conv"] = torch.randn((C, b["conv"]), generator=g) * 0.6
            around(right + ".conv.b", C, 0.0)
            for x, centre in (("ra", -1.0), ("ri", 0.3)):
                w["%s.%s" % (right, x)] = torch.randn((n, c, c), generator=g) / math.sqrt(c)
                w["%s.%s.b" % (right, x)] = centre + torch.randn((n, c), generator=g)
            around(right + ".lam", C, -2.0, 1.3)
            mat(right + ".o", W, C)
            around(left + ".out", W), around(right + ".out", W)
        else:
            H, G, d, dv, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            mat(q + ".q", G * d, W, 1.5), mat(q + ".k", G * d, W, 1.5), mat(q + ".v", H * dv, W, 1.5)
            for x, n in (("q", G * d), ("k", G * d), ("v", H * dv)):
                w["%s.%s.conv" % (q, x)] = torch.randn((n, taps), generator=g) * 0.6
            mat(q + ".b", H, W), mat(q + ".a", H, W)
            w[q + ".dt_bias"] = torch.randn((H,), generator=g)
            between(q + ".A_log", H, -3.0, 0.5)
            mat(q + ".g", H * dv, W, 1.5)
            around(q + ".norm", dv)
            mat(q + ".o", W, H * dv)
        mlp = lay["mlp"]
        if mlp is None:
            continue
        around(p + ".norm2", W, 0.0)
        F = mlp["expert"]["ff"]
        mat(p + ".mlp.router", mlp["router"]["experts"], W, 2.0)
        for e in range(mlp["router"]["experts"]):
            x = "%s.mlp.e%d" % (p, e)
            mat(x + ".gate", F, W, 1.5), mat(x + ".up", F, W), mat(x + ".down", W, F)
    around("final.norm", W, 0.0)
    mat("head", V, W)
    most = max([lay["mlp"]["router"]["experts"] for lay in cfg["layers"] if lay["mlp"] is not None], default=0)
    if decisive and most:
        code = list(range(W - most, W))
        levels = torch.linspace(-1.5, 1.5, most) if most > 1 else torch.zeros(1)
        for t in range(V):
            w["embed"][t, code] = torch.roll(levels, t % most) / cfg["embedding"]["scale"]
        w["pos"][:, code] = 0.0
        for name in list(w):
            if name.endswith(".o") or name.endswith(".down"):
                w[name][code, :] = 0.0
            elif name.endswith(".router"):
                w[name] *= 0.1
                for e in range(w[name].shape[0]):
                    w[name][e, code[e]] += 10.0
    return rounded(w)


def rounded(w):
    """The values a bfloat16 checkpoint holds, so that every run sees the same numbers."""
    return {k: v.to(torch.bfloat16).to(torch.float32) for k, v in w.items()}


def write_model(folder, cfg, weights):
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in weights.items()}, os.path.join(folder, "model.safetensors"))
    return folder


def make_model(tmp_path, which, seed=0, spread=1.0, weights=None, decisive=False):
    cfg = CONFIGS[which] if isinstance(which, str) else which
    weights = weights if weights is not None else make_weights(cfg, seed, spread, decisive)
    tag = which if isinstance(which, str) else "custom"
    folder = write_model(os.path.join(str(tmp_path), "gurapel_%s_%d_%g_%d" % (tag, seed, spread, decisive)), cfg, weights)
    return folder, cfg, weights


def plain_logits(cfg, weights, tokens, dtype=torch.float64, storage=None):
    return P.forward(cfg, weights, tokens, dtype=dtype, storage=storage).to(torch.float32)


def greedy(cfg, weights, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(plain_logits(cfg, weights, toks)[-1].argmax()))
    return toks[len(prompt):]


def bfloat16_limits(cfg, weights, tokens, ref, draws=3):
    """What rounding to bfloat16 may cost at every position: three times what it costs the plain implementation when
    it rounds what an engine may keep in 16 bits, the largest of ``draws`` draws of the rounding errors, but no less
    than three times the median of the first draw over the positions."""
    e = row_errs(plain_logits(cfg, weights, tokens, dtype=torch.float32, storage=torch.bfloat16), ref)
    worst = torch.maximum(e, e.median())
    for i in range(1, draws):
        gen = torch.Generator().manual_seed(1000 + i)
        worst = torch.maximum(worst, row_errs(plain_logits(cfg, weights, tokens, dtype=torch.float32,
                                                           storage=(torch.bfloat16, gen)), ref))
    return 3.0 * worst


def single_layer(which, index, vocab=47):
    """The configuration of one layer of ``which`` alone (a mechanism on its own)."""
    cfg = json.loads(json.dumps(CONFIGS[which]))
    cfg.update(vocab=vocab, layers=[cfg["layers"][index]])
    return cfg


def far_token_through_the_recurrence(n):
    """One layer whose linear recurrence holds one far token (its attention branch gives nothing): an entry of the stream
    that only token 0 sets drives every channel's input and its gate wide open; the decays are close to 1. Returns the
    configuration, the weights and two sequences that differ in their first token (0 or not)."""
    cfg = single_layer("D", 1)
    w = make_weights(cfg, 6)
    p = "l0.mix.right"
    w["l0.mix.left.o"][:] = 0.0
    w["embed"][:, 0], w["pos"][:, 0] = 0.0, 0.0
    w["embed"][0, 0] = 8.0
    w[p + ".x"][:, 0] = 6.0
    w[p + ".lam"][:], w[p + ".ra.b"][:], w[p + ".ra"][:] = -6.0, -5.0, 0.0
    w["l0.mlp.router"][:, 0] = 0.0
    return cfg, rounded(w), *_two_sequences(cfg, n)


def far_token_through_the_memory(n):
    """One layer of the delta rule whose memory holds one far token: the stream has an entry that only token 0 sets and
    one that every token sets alike; beta reads them, so that token 0 writes with all its weight and the others hardly
    at all; the decays are close to 1."""
    cfg = single_layer("C", 1)
    w = make_weights(cfg, 6)
    s = cfg["embedding"]["scale"]
    w["l0.mix.A_log"][:] = -6.0
    w["pos"][:, :2] = 0.0
    w["embed"][:, 0], w["embed"][:, 1] = 0.0, 2.0 / s
    w["embed"][0, 0] = 4.0 / s
    w["l0.mix.b"][:] = 0.0
    w["l0.mix.b"][:, 1], w["l0.mix.b"][:, 0] = -6.0, 20.0
    return cfg, rounded(w), *_two_sequences(cfg, n)


def _two_sequences(cfg, n):
    g = torch.Generator().manual_seed(13)
    rest = (1 + torch.randint(0, cfg["vocab"] - 1, (n - 1,), generator=g)).tolist()
    return [0] + rest, [1] + rest


def window_edge(which, index, n, spread=4.0):
    """One layer of attention (its recurrence gives nothing) with peaked scores, and three sequences of ``n`` tokens: the
    base, one that differs in the last token that the last position still sees, and one that differs in the token just
    before it. The differing token is the one that moves the plain implementation's last logits most."""
    cfg = single_layer(which, index)
    cfg["layers"][0]["mlp"] = None
    w = make_weights(cfg, 5, spread)
    w["l0.mix.right.o"][:] = 0.0
    w["l0.mix.left.r1"][:] = 0.05             # (a distance takes little off, so that the far key can stand out)
    w = rounded(w)
    size = cfg["layers"][0]["mixer"]["left"]["mask"]["size"]
    g = torch.Generator().manual_seed(12)
    base = torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()
    at_in, at_out = n - size, n - size - 1
    ref = plain_logits(cfg, w, base)

    def with_token(at, v):
        return base[:at] + [v] + base[at + 1:]

    v = max((x for x in range(cfg["vocab"]) if x != base[at_in]),
            key=lambda x: float((plain_logits(cfg, w, with_token(at_in, x))[-1] - ref[-1]).abs().max()))
    seqs = {"base": base, "inside": with_token(at_in, v),
            "outside": with_token(at_out, v if v != base[at_out] else (v + 1) % cfg["vocab"])}
    return cfg, w, seqs, {k: plain_logits(cfg, w, t) for k, t in seqs.items()}
