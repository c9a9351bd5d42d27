"""Small Zunilorn configurations and random weights by checkpoint name, made without the package's help, for the tests
that compare the engine with the plain implementation (plain_zunilorn.py)."""
import json
import math
import os

import torch
from safetensors.torch import save_file

import plain_zunilorn as P
from takosun_helpers import rel_err, replay, row_errs, within  # noqa: F401  (shared measures, re-exported)


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(experts, identity, top, ff, limit, scale=1.0, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit},
           "router": {"experts": experts, "identity": identity, "top": top, "scale": scale}}
    if shared is not None:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def attention(heads, kv_heads, dim, vdim, rot=None, base=1e4, scaling=None, scale=None, softcap=20.0, mlp=None):
    r = {"base": base, "dims": rot or dim}
    if scaling is not None:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                                       "scale": scale or dim ** -0.5, "softcap": softcap, "rot": r}}


def mamba(heads, vdim, state, groups, conv, norm_groups, mlp=None):
    return {"type": "mamba2", "mlp": mlp, "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                                                    "conv": conv, "norm_groups": norm_groups}}


def model(vocab, width, layers, streams=2, mult=1.0, cap=10.0, loop=None, eps=1e-5):
    out = {"architecture": "Zunilorn", "vocab": vocab, "width": width, "streams": streams, "residual_mult": mult,
           "norm": {"eps": eps}, "logit_softcap": cap, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


# Sizes differ between the configurations and inside each: one to five streams, loops at the start, in the middle and none,
# values wider and narrower than keys, rotations over a part of a head, weak and strong scalings, states that are multiples
# of nothing, one group of B and C and as many as heads, one norm part and several, filters of one to five taps, no, one and
# several experts that return their input, limits that differ between experts, shared expert and dense layers, layers
# without a feed-forward, a model without attention and one without recurrence.
CONFIGS = {
    "A": model(61, 48, [
        attention(4, 2, 12, 20, rot=8, scaling=(4.0, 64, 8.0, 1.0), scale=0.3, softcap=5.0,
                  mlp=moe(5, 2, 3, 16, 0.8, 1.7, (12, 1.3))),
        mamba(6, 10, 7, 3, 3, 2, mlp=dense(20, 0.9)),
        attention(2, 1, 16, 8, base=300.0, softcap=30.0),
    ], streams=3, mult=0.6, cap=7.0, loop=(0, 2, 2)),
    "B": model(77, 64, [
        mamba(4, 8, 16, 4, 2, 1, mlp=moe(6, 1, 2, 20, 2.0, 0.7)),
        attention(6, 3, 8, 12, rot=4, scaling=(1.5, 20, 2.0, 0.5), mlp=dense(24, 1.5)),
        mamba(5, 12, 33, 1, 5, 5),
        attention(5, 5, 6, 5, scale=0.5, softcap=2.0, mlp=moe(3, 0, 1, 10, 1.0, 2.0, (8, 0.6))),
    ], streams=2, mult=0.3, loop=(1, 4, 3), eps=1e-6),
    "C": model(40, 32, [      # state only: no pages at all
        mamba(2, 12, 12, 1, 4, 3, mlp=moe(2, 3, 2, 16, 1.1, 1.0, (9, 2.0))),
        mamba(3, 4, 20, 3, 1, 1, mlp=dense(11, 1.2)),
    ], streams=1, mult=0.5),
    "D": model(53, 40, [
        attention(3, 1, 20, 16, rot=12, scaling=(8.0, 40, 4.0, 1.0), mlp=moe(4, 4, 8, 12, 1.4, 3.0)),
        attention(2, 2, 8, 24, softcap=4.0, mlp=dense(16, 0.5)),
    ], streams=5, mult=1.2, cap=3.0, loop=(1, 2, 2)),
    # sizes at which the matrix-core forms of the kernels run (GPU tests)
    "M": model(300, 256, [
        mamba(8, 64, 128, 2, 4, 4, mlp=moe(6, 2, 2, 64, 1.5, 1.5, (96, 1.2))),
        attention(4, 2, 64, 80, rot=32, scaling=(2.0, 100, 16.0, 1.0), softcap=30.0, mlp=dense(128, 1.1)),
        mamba(6, 48, 64, 3, 3, 2, mlp=dense(64, 0.7)),
        attention(16, 1, 128, 96, base=1e5, softcap=15.0, mlp=moe(8, 3, 5, 128, 0.9, 2.2, (32, 3.0))),
    ], streams=4, mult=0.75, loop=(0, 3, 2)),
}


def make_weights(cfg, seed, spread=1.0, decisive=False):
    """Matrices N(0, 1 / inputs) (the queries' ``spread`` times larger, so that attention is peaked for spread > 1); norm
    weights around 1; sinks, decays, steps and biases that differ from head to head; streams that are read, mixed and
    written unevenly; corrections as wide as the scores differ.

    ``decisive``: no choice of experts is a close call, so that rounding cannot flip one (a flipped choice moves a row,
    and every later row, by far more than rounding; bfloat16 runs are compared under such weights, float32 runs under
    the random routers). The last entries of the stream hold a code of the token id, distinct levels in an order that
    turns with the id; no sublayer writes to them and the streams are read and mixed with positive numbers, so that they
    keep their order; expert e's router row reads entry e with a large factor beside small random entries; the corrections
    are zero but for one expert that is always chosen and one that never is."""
    g = torch.Generator().manual_seed(seed)
    W, V, n = cfg["width"], cfg["vocab"], cfg["streams"]
    w = {}

    def mat(name, rows, cols, s=1.0):
        w[name] = torch.randn((rows, cols), generator=g) * (s / math.sqrt(cols))

    def around(name, k, centre=1.0, dev=0.2):
        w[name] = centre + dev * torch.randn((k,), generator=g)

    def between(name, k, lo, hi):
        w[name] = lo + (hi - lo) * torch.rand((k,), generator=g)

    def gated(name, F, biased):
        mat(name + ".gate", F, W, 1.5), mat(name + ".up", F, W, 1.2), mat(name + ".down", W, F)
        if biased:
            around(name + ".gate.b", F, 0.0), around(name + ".up.b", F, 0.0), around(name + ".down.b", W, 0.0)

    w["embed"] = torch.randn((V, W), generator=g) * (2.5 / math.sqrt(W))      # (logits within a few times the caps)
    for i, lay in enumerate(cfg["layers"]):
        p, m, q = "l%d" % i, lay["mixer"], "l%d.mix" % i
        mlp = lay["mlp"]
        for k in (1, 2) if mlp is not None else (1,):
            around("%s.norm%d" % (p, k), W)
            hc = "%s.hc%d" % (p, k)
            if decisive:
                between(hc + ".in", n, 0.3 / n, 1.5 / n)
                w[hc + ".mix"] = (0.3 + torch.rand((n, n), generator=g)) / (0.8 * n)
            else:
                around(hc + ".in", n, 1.0 / n, 0.5)
                w[hc + ".mix"] = 0.8 * torch.eye(n) + torch.randn((n, n), generator=g) * (0.3 / math.sqrt(n))
            around(hc + ".out", n, 1.0, 0.6)
        if lay["type"] == "attention":
            H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            mat(q + ".q", H * d, W, 1.4 * spread), mat(q + ".k", G * d, W, 1.4), mat(q + ".v", G * dv, W)
            between(q + ".sink", H, -2.0, 3.0)
            mat(q + ".g", H, W, 1.5), mat(q + ".o", W, H * dv)
        else:
            H, dv, N, G, taps = m["heads"], m["vdim"], m["state"], m["groups"], m["conv"]
            C = H * dv + 2 * G * N
            mat(q + ".in", H * dv + C + H, W, 1.3)
            w[q + ".conv"] = torch.randn((C, taps), generator=g) * 0.6
            around(q + ".conv.b", C, 0.1)
            around(q + ".dt_bias", H, -1.0, 1.0), between(q + ".A_log", H, -3.0, 1.0), around(q + ".D", H, 0.7, 0.5)
            around(q + ".norm", H * dv), mat(q + ".o", W, H * dv)
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            gated(p + ".mlp", mlp["ff"], True)
            continue
        r = mlp["router"]
        E = r["experts"] + r["identity"]
        mat(p + ".mlp.router", E, W, 2.0)
        around(p + ".mlp.correction", E, 0.0, 0.15)
        for e in range(r["experts"]):
            gated("%s.mlp.e%d" % (p, e), mlp["expert"]["ff"], False)
        if mlp.get("shared") is not None:
            gated(p + ".mlp.shared", mlp["shared"]["ff"], False)
            mat(p + ".mlp.shared.sg", 1, W, 2.0)
    around("final.norm", W)
    w["final.norm"] *= torch.randint(0, 2, (W,), generator=g) * 2.0 - 1.0     # (else the shared table repeats the last token)
    routers = [lay["mlp"]["router"] for lay in cfg["layers"] if lay["mlp"] is not None and lay["mlp"]["kind"] == "moe"]
    most = max([r["experts"] + r["identity"] for r in routers], default=0)
    if decisive and most:
        code = list(range(W - most, W))
        levels = torch.linspace(-0.8, 0.8, most) if most > 1 else torch.zeros(1)
        for t in range(V):
            w["embed"][t, code] = torch.roll(levels, t % most)
        for name in list(w):
            if name.endswith(".o") or name.endswith(".down"):
                w[name][code, :] = 0.0
            elif name.endswith(".down.b"):
                w[name][code] = 0.0
            elif name.endswith(".router"):
                w[name] *= 0.1
                for e in range(w[name].shape[0]):
                    w[name][e, code[e]] += 6.0
            elif name.endswith(".correction"):
                E = w[name].shape[0]
                w[name][:] = 0.0
                w[name][E // 2] = 3.0
                if w[name[:-len("correction")] + "router"].shape[0] > cfg["layers"][int(name[1:name.index(".")])]["mlp"]["router"]["top"]:
                    w[name][0 if E // 2 != 0 else E - 1] = -3.0
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
    folder = write_model(os.path.join(str(tmp_path), "zunilorn_%s_%d_%g_%d" % (tag, seed, spread, decisive)), cfg, weights)
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
    """The configuration of one layer of ``which`` alone, run once (a mechanism on its own)."""
    cfg = json.loads(json.dumps(CONFIGS[which]))
    cfg.pop("loop", None)
    cfg.update(vocab=vocab, layers=[cfg["layers"][index]])
    return cfg


def _two_sequences(cfg, n):
    """``n`` tokens that differ in their first: 0, which occurs nowhere else, or 1."""
    g = torch.Generator().manual_seed(13)
    rest = (1 + torch.randint(0, cfg["vocab"] - 1, (n - 1,), generator=g)).tolist()
    return [0] + rest, [1] + rest


def far_token_through_the_state(n):
    """One layer of the recurrence whose state holds one far token: the stream has an entry that only token 0 sets and one
    that every token sets alike; the step sizes read them, so that token 0 writes with a step of about one and the others
    hardly at all, and the decays are close to 1. Returns the configuration, the weights and two sequences that differ in
    their first token (0 or not)."""
    cfg = single_layer("C", 0)
    cfg["layers"][0]["mlp"] = None
    m = cfg["layers"][0]["mixer"]
    w = make_weights(cfg, 6)
    p = "l0.mix"
    H = m["heads"]
    w["embed"][:, 0], w["embed"][:, 1] = 0.0, 2.0
    w["embed"][0, 0] = 6.0
    w[p + ".in"][-H:] = 0.0
    w[p + ".in"][-H:, 0], w[p + ".in"][-H:, 1] = 3.0, -3.0
    w[p + ".A_log"][:], w[p + ".D"][:] = -3.0, 0.0
    return cfg, rounded(w), *_two_sequences(cfg, n)


def far_key(n, which="A", index=0):
    """One layer of attention in which one far key stands out: an entry of the stream that only token 0 sets and one that
    every token sets alike; every query reads the second into an entry of its head that is not rotated, the key of token 0
    reads the first into it, so that its score is near the cap at every distance."""
    cfg = single_layer(which, index)
    cfg["layers"][0]["mlp"] = None
    m = cfg["layers"][0]["mixer"]
    m["softcap"] = 12.0
    w = make_weights(cfg, 6)
    p, d, rot = "l0.mix", m["dim"], m["rot"]["dims"]
    assert rot < d
    w["embed"][:, 0], w["embed"][:, 1] = 0.0, 3.0
    w["embed"][0, 0] = 8.0
    for name, heads, entry in ((".q", m["heads"], 1), (".k", m["kv_heads"], 0)):
        w[p + name] *= 0.3
        for h in range(heads):
            w[p + name][h * d + rot] = 0.0
            w[p + name][h * d + rot, entry] = 5.0
    return cfg, rounded(w), *_two_sequences(cfg, n)
