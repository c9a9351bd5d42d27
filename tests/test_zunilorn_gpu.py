"""Zunilorn on the GPU: the new kernels alone against the plain implementation's function of the same mechanism, every
kind of layer alone and the whole model through the engine's step function in float32 and bfloat16 under the ways of
cutting a request into steps, far tokens and sinks made to decide the logits, pages and state slots used again, long
decoding from graphs, configurations drawn at random, and generation through the entry point."""
import os
import random
import subprocess
from types import SimpleNamespace

import pytest
import torch

import plain_zunilorn as P
from helpers import (random_tokens, replay_in_process, replay_with_program, trace_bulk_then_single, trace_mixed,
                     trace_portions, trace_whole)
from zunilorn_helpers import (attention, bfloat16_limits, dense, far_key, far_token_through_the_state, greedy, make_model,
                              make_weights, mamba, model, moe, plain_logits, rel_err, replay, row_errs, single_layer,
                              within)

pytestmark = pytest.mark.gpu

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

DTYPES = [torch.float32, torch.bfloat16]
TOL_F32 = 3e-5


def ops():
    from lmsf_amd.ops import get_ops
    return get_ops()


def close(got, ref, dtype, scale=1.0):
    tol = 2e-5 if dtype == torch.float32 else 1.2e-2
    err = float((got.double().cpu() - ref.double().cpu()).abs().max())
    assert err <= tol * max(scale, float(ref.double().abs().max())), (err, float(ref.double().abs().max()))


def check(got, ref, dtype, what, model_, yardstick=0.0):
    """float32: three times what float32 rounding costs the plain implementation itself, where that is more than
    TOL_F32 (``yardstick``: that cost as the caller has measured it on other requests of the same model); bfloat16: per
    position three times what rounding costs the plain implementation when it rounds what an engine may keep in 16
    bits."""
    cfg, w, toks = model_
    if dtype == "float32":
        tol = max(TOL_F32, 3 * max(yardstick, rel_err(plain_logits(cfg, w, toks, dtype=torch.float32), ref)))
        assert rel_err(got, ref) < tol, (what, rel_err(got, ref), tol)
    else:
        ok, worst = within(got, ref, bfloat16_limits(cfg, w, toks, ref))
        assert ok, (what, worst)


def batch_of(lens, slots, first_pos=None, dev="cuda"):
    """What the kernels read of a step: segments of ``lens`` tokens in state slots ``slots``."""
    starts = [0]
    for n in lens:
        starts.append(starts[-1] + n)
    first_pos = first_pos or [0] * len(lens)
    pos = [p0 + i for p0, n in zip(first_pos, lens) for i in range(n)]
    seg = [s for s, n in enumerate(lens) for _ in range(n)]
    i32 = dict(dtype=torch.int32, device=dev)
    return SimpleNamespace(n_segments=len(lens), seg_starts=torch.tensor(starts, **i32), state_slots=torch.tensor(slots, **i32),
                           seg_of_token=torch.tensor(seg, **i32), positions=torch.tensor(pos, **i32), n_tokens=len(pos),
                           host_seg_lens=list(lens), host_seg_starts=starts[:-1], host_seg_first_pos=list(first_pos),
                           max_context=max(pos) + 1, all_single=all(n == 1 for n in lens), replayed=False, aux={})


# ---------------------------------------------------------------- kernels alone


def state_space_case(dtype, H, G, N, dv, lens, seed=0, dt_scale=1.0):
    """Inputs of a step, and what the plain recurrence gives from states that an earlier step left."""
    g = torch.Generator().manual_seed(H * 1000 + N + dv + seed)
    slots = [2, 0, 3][:len(lens)]
    T, C = sum(lens), H * dv + 2 * G * N
    u = torch.randn((T, C + 8), generator=g).to(dtype)
    dt = (torch.randn((T, H + 3), generator=g) - 1.0) * dt_scale
    bias, a_log, D = torch.randn(H, generator=g), torch.rand(H, generator=g) * 4 - 3, torch.randn(H, generator=g)
    state0 = torch.randn((5, H * N * dv + 4), generator=g)
    v = u.double()
    x = v[:, :H * dv].reshape(T, H, dv)
    B, C_ = (v[:, at:at + G * N].reshape(T, G, N) for at in (H * dv, H * dv + G * N))
    step = torch.nn.functional.softplus(dt[:, :H].double() + bias.double())
    rate = torch.exp(a_log)
    want, after, at = [], state0.clone().double(), 0
    for n, slot in zip(lens, slots):
        part = slice(at, at + n)
        own = P.state_space(x[part], B[part], C_[part], step[part], a_log.double(), D.double())
        # what the earlier state adds to an output: C . (the decays so far) S_0; the state after is linear in S_0 too
        S = state0[slot, :H * N * dv].double().reshape(H, dv, N)
        decay = torch.exp(torch.cumsum(-torch.exp(a_log.double()) * step[part], 0))              # [n, H]
        Ch = C_[part].repeat_interleave(H // G, 1)
        want.append(own + torch.einsum("hen,thn->the", S, Ch * decay[:, :, None]))
        Bh = B[part].repeat_interleave(H // G, 1)
        for t in range(n):
            keep = torch.exp(-torch.exp(a_log.double()) * step[at + t])
            S = keep[:, None, None] * S + x[at + t][:, :, None] * (step[at + t][:, None] * Bh[t])[:, None, :]
        after[slot, :H * N * dv] = S.reshape(-1)
        at += n
    args = (u.cuda(), 0, H * dv, H * dv + G * N, dt.cuda(), bias.cuda(), rate.cuda(), D.cuda())
    return args, state0, slots, torch.cat(want).reshape(T, H * dv), after


@pytest.mark.parametrize("dtype,form", [(torch.float32, "tokens"), (torch.bfloat16, "tokens"), (torch.bfloat16, "chunks")])
@pytest.mark.parametrize("H,G,N,dv,lens", [(4, 2, 128, 64, [63, 65, 130]), (6, 3, 32, 48, [64, 1, 200]), (2, 1, 7, 10, [5, 1, 70]),
                                            (3, 3, 33, 20, [66, 2, 1]), (2, 2, 256, 16, [129, 64]), (1, 1, 64, 128, [300, 17]),
                                            (5, 1, 100, 36, [1, 1, 1]), (2, 1, 16, 200, [90]), (8, 8, 4, 8, [1, 128, 3])])
def test_the_recurrence_from_states_an_earlier_step_left(dtype, form, H, G, N, dv, lens):
    """Segments in scattered slots, shorter than a chunk, a chunk long, one token more and many chunks, single tokens
    beside them and alone; states and values that the vectors and the matrix cores' tiles do and do not divide. What the
    products keep in float32 is float32 in both types."""
    o = ops()
    args, state0, slots, want, after = state_space_case(dtype, H, G, N, dv, lens)
    state = state0.cuda()
    got = o.state_space(*args, state, batch_of(lens, slots), H, G, N, dv, form=form)
    assert float((got.double().cpu() - want).abs().max()) <= 2e-5 * max(1.0, float(want.abs().max()))
    n = H * N * dv
    assert float((state.cpu()[:, :n].double() - after[:, :n]).abs().max()) <= 2e-5 * max(1.0, float(after.abs().max()))
    assert torch.equal(state.cpu()[:, n:], state0[:, n:])
    assert torch.equal(state.cpu()[1], state0[1]) and torch.equal(state.cpu()[4], state0[4])


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_recurrence_with_states_beyond_a_wave_and_with_strong_decays(dtype):
    o = ops()
    for H, G, N, dv, lens, scale in ((2, 1, 400, 12, [30, 1], 1.0), (1, 1, 1000, 5, [9], 1.0), (4, 2, 64, 32, [200, 90], 40.0)):
        args, state0, slots, want, after = state_space_case(dtype, H, G, N, dv, lens, dt_scale=scale)
        state = state0.cuda()
        got = o.state_space(*args, state, batch_of(lens, slots), H, G, N, dv)
        assert torch.isfinite(got).all()
        assert float((got.double().cpu() - want).abs().max()) <= 2e-5 * max(1.0, float(want.abs().max())), (N, dv)
        n = H * N * dv
        assert float((state.cpu()[:, :n].double() - after[:, :n]).abs().max()) <= 2e-5 * max(1.0, float(after.abs().max()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,inner,parts", [(1, 60, 2), (5, 4096, 8), (600, 384, 3), (3, 75, 5), (2, 12288, 1), (40, 30, 30)])
def test_the_gate_and_the_norm_in_parts(dtype, T, inner, parts):
    g = torch.Generator().manual_seed(inner)
    y, z = torch.randn((T, inner), generator=g) * 2, torch.randn((T, inner + 12), generator=g).to(dtype)
    w = 1 + 0.3 * torch.randn(inner, generator=g)
    want = P.gated_group_norm(y.double(), z[:, :inner].double(), w.double(), parts, 1e-5)
    close(ops().gated_group_norm(y.cuda(), z.cuda()[:, :inner], w.cuda(), parts, 1e-5), want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,n,W", [(1, 1, 48), (3, 2, 2048), (520, 4, 96), (5, 3, 50), (2, 8, 4100), (600, 5, 4096), (4, 11, 64),
                                   (2, 32, 10), (7, 6, 16384), (3, 7, 260)])
def test_the_streams_are_mixed_read_and_normed_in_one_launch(dtype, T, n, W):
    """With and without an update, with the weighted sum or the plain one, at all rows and at some (which leaves the
    streams as they were)."""
    from lmsf_amd.ops.handles import StreamUpdate
    o = ops()
    g = torch.Generator().manual_seed(n * 100 + W)
    X = torch.randn((T, n, W), generator=g)
    y = torch.randn((T, W + 8), generator=g).to(dtype)
    M, b, a = (torch.randn(s, generator=g) for s in ((n, n), (n,), (n,)))
    w = 1 + 0.3 * torch.randn(W, generator=g)
    rows = torch.tensor([T - 1, 0, T // 2]).int()
    Xd = X.double().transpose(0, 1)
    new = P.write_streams(Xd, M.double(), b.double(), y[:, :W].double(), 1.0)
    yc, dev = y.cuda()[:, :W], dict(mix=M.cuda(), add=b.cuda())
    for update in (True, False):
        S = new if update else Xd
        up = StreamUpdate(yc, **dev) if update else None
        for read in (a, None):
            u = P.read_streams(S, a.double() if read is not None else torch.ones(n).double())
            want = P.rms(u, 1e-5) * w.double()
            for r in (None, rows):
                Xc = X.cuda()
                got = o.mix_streams(Xc, update=up, read=a.cuda() if read is not None else None, weight=w.cuda(), eps=1e-5,
                                    out_dtype=dtype, rows=r.cuda() if r is not None else None)
                assert got.dtype == dtype
                close(got, want if r is None else want[r.long()], dtype)
                if update and r is None:
                    close(Xc, new.transpose(0, 1), torch.float32)
                else:
                    assert torch.equal(Xc.cpu(), X)
    Xc = X.cuda()
    assert o.mix_streams(Xc, update=StreamUpdate(yc, **dev)) is None
    close(Xc, new.transpose(0, 1), torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,W", [(1, 40), (4, 2052), (3, 33)])
def test_every_stream_begins_as_the_tokens_row(dtype, n, W):
    g = torch.Generator().manual_seed(3)
    table = torch.randn((31, W), generator=g).to(dtype)
    ids = torch.tensor([0, 30, 7, 7, 19]).int()
    X = ops().stream_embedding(ids.cuda(), table.cuda(), n, 0.5)
    assert X.shape == (5, n, W) and X.dtype == torch.float32
    assert torch.equal(X.cpu(), (table[ids.long()].float() * 0.5)[:, None].repeat(1, n, 1))


@pytest.mark.parametrize("dtype,exact", [(torch.float32, True), (torch.bfloat16, True), (torch.bfloat16, False)])
@pytest.mark.parametrize("H,G,D,window", [(4, 2, 64, 0), (3, 1, 192, 90), (16, 1, 128, 0), (2, 2, 16, 1), (5, 5, 96, 0),
                                          (20, 1, 256, 64), (2, 1, 320, 0)])
def test_a_sink_stands_in_the_denominator(dtype, exact, H, G, D, window):
    """All attention kernels under a cap, requests of one and of many tokens, contexts of one and of several splits; sinks
    far below, among and far above the scores."""
    from torch_ops import TorchOps
    o = ops()
    g = torch.Generator().manual_seed(5)
    ps = 16
    lens, first = [70, 1, 1, 130, 1], [0, 700, 3, 20, 0]
    pages = 60
    kp = (torch.randn((pages, G, ps, D), generator=g) * 1.5).to(dtype)
    vp = torch.randn((pages, G, D, ps), generator=g).to(dtype)
    N = sum(lens)
    q = (torch.randn((N, H * D), generator=g) * 1.5).to(dtype)
    tables = torch.stack([torch.randperm(pages, generator=g)[:48] for _ in lens]).int()
    for shift in (0.0, -60.0, 9.0, 60.0):
        sink = torch.randn(H, generator=g) * 2 + shift
        b = batch_of(lens, [0, 1, 2, 3, 4], first, dev="cpu")
        want = TorchOps().paged_attention(q.float(), kp.float(), vp.float(), tables, b.seg_of_token, b.positions, H, G, D,
                                          D ** -0.5, window, softcap=6.0, sink=sink)
        bc = batch_of(lens, [0, 1, 2, 3, 4], first)
        for batch in (bc, None):
            for kernel in ((None, "generic") if shift == 0.0 else (None,)):
                got = o.paged_attention(q.cuda(), kp.cuda(), vp.cuda(), tables.cuda(), bc.seg_of_token, bc.positions, H, G, D,
                                        D ** -0.5, window, batch=batch, softcap=6.0, sink=sink.cuda(), weights_f32=exact,
                                        kernel=kernel)
                close(got, want, dtype)
    plain = o.paged_attention(q.cuda(), kp.cuda(), vp.cuda(), tables.cuda(), bc.seg_of_token, bc.positions, H, G, D, D ** -0.5,
                              window, batch=bc, softcap=6.0)
    assert float((plain.float().cpu() - want).abs().max()) > 0.5      # (without it the values come through)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,rot,ps", [(4, 2, 16, 24, 16, 4), (1, 1, 64, 64, 32, 16), (6, 3, 8, 5, 6, 8),
                                             (2, 1, 96, 128, 96, 16), (16, 4, 128, 128, 128, 16), (3, 3, 200, 40, 112, 8),
                                             (2, 2, 40, 8, 24, 16)])
def test_queries_and_keys_are_turned_on_their_way_into_the_pages(dtype, H, G, d, dv, rot, ps):
    """Rotations whose partner entries are whole pieces of eight (the lanes' exchange) and others."""
    from torch_ops import TorchOps
    g = torch.Generator().manual_seed(d + dv)
    N, pages, D = 9, 5, (max(d, dv) + 15) // 16 * 16
    p = (torch.randn((N, (H + G) * d + G * dv + 8), generator=g) * 2).to(dtype)
    pos = torch.tensor([0, 1, 2, 3, 4, 17, 18, 39, 7]).int()
    slots = torch.tensor([0, 1, ps - 1, ps, 2 * ps + 1, 3 * ps, 4 * ps + ps - 1, -1, 2], dtype=torch.int32)
    f, gain = P.frequencies({"base": 500.0, "dims": rot, "scaling": {"factor": 3.0, "original": 30, "fast": 4.0, "slow": 1.0}})
    angle = torch.arange(40).double()[:, None] * torch.tensor(f).double()[None]
    table = (torch.cat([torch.cos(angle), torch.sin(angle)], 1) * gain).float()
    outs = []
    for op, dev, dt in ((TorchOps(), "cpu", torch.float32), (ops(), "cuda", dtype)):
        pc = p.to(dev).to(dt)
        kp = torch.full((pages, G, ps, D), 9.0, dtype=dt, device=dev)
        vp = torch.full((pages, G, D, ps), 9.0, dtype=dt, device=dev)
        qa = op.attn_prepare(pc[:, :H * d], pc[:, H * d:(H + G) * d], pc[:, (H + G) * d:], H, G, d, dv, D, pos.to(dev),
                             slots.to(dev), kp, vp, table=table.to(dev))
        outs.append((qa, kp, vp))
    for got, want in zip(outs[1], outs[0]):
        close(got, want, dtype, scale=9.0)
    whole = P.rotate(p[:1, :H * d].double().view(1, H, d).repeat(40, 1, 1), {
        "base": 500.0, "dims": rot, "scaling": {"factor": 3.0, "original": 30, "fast": 4.0, "slow": 1.0}})
    close(outs[1][0].view(N, H, D)[0, :, :d], whole[0], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,vdim,D", [(3, 20, 32), (2, 5, 16), (4, 64, 64)])
def test_one_gate_a_head(dtype, H, vdim, D):
    g = torch.Generator().manual_seed(4)
    a, gate = torch.randn((6, H * D), generator=g).to(dtype), torch.randn((6, H + 5), generator=g).to(dtype)
    want = a.double().view(6, H, D)[..., :vdim] * torch.sigmoid(gate[:, :H].double())[..., None]
    got = ops().attn_finish(a.cuda(), D, H, vdim, torch.arange(6).int().cuda(), gate=gate.cuda()[:, :H])
    close(got, want.reshape(6, H * vdim), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("M,K,I,biased", [(1, 64, 48, True), (2, 256, 40, False), (5, 128, 128, True), (16, 72, 24, True),
                                          (40, 192, 96, True), (130, 256, 64, False), (300, 320, 160, True), (3, 50, 7, True)])
def test_the_bounded_activation_at_every_number_of_rows(dtype, M, K, I, biased):
    g = torch.Generator().manual_seed(M + K)
    o = ops()
    x = torch.randn((M, K), generator=g).to(dtype)
    w = (torch.randn((2 * I, K), generator=g) * (2.0 / K ** 0.5)).to(dtype)
    bias = torch.randn(2 * I, generator=g).to(dtype) if biased else None
    z = x.double() @ w.double().T + (bias.double() if biased else 0.0)
    if dtype == torch.bfloat16:
        z = z.to(dtype).double()
    want = P.bounded_gate(z[:, :I], z[:, I:], 1.3)
    close(o.linear_gated(x.cuda(), w.cuda(), bias.cuda() if biased else None, "bounded", limit=1.3), want, dtype, scale=4.0)
    close(o.gated_act(z.to(dtype).cuda(), "bounded", 1.3), P.bounded_gate(z[:, :I].to(dtype).double(), z[:, I:].to(dtype).double(), 1.3),
          dtype)
    with pytest.raises(ValueError):
        o.linear_gated(x.cuda(), w.cuda(), None, "bounded")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,E,same,top,F,W", [(3, 4, 2, 3, 24, 48), (70, 8, 3, 3, 64, 128), (1, 3, 1, 4, 10, 36),
                                              (300, 6, 6, 2, 96, 64), (40, 5, 0, 5, 32, 96), (9, 70, 30, 6, 16, 32),
                                              (64, 2, 5, 7, 32, 64), (50, 6, 2, 2, 32, 42)])
def test_experts_that_return_their_input_beside_bounded_ones(dtype, N, E, same, top, F, W):
    """Router with corrections and a gate's column, experts streamed (few pairs, float32 at any number) and grouped on the
    matrix cores, a shared part behind the gate."""
    o = ops()
    g = torch.Generator().manual_seed(N + E)
    h = torch.randn((N, W), generator=g).to(dtype)
    gu = (torch.randn((E, 2 * F, W), generator=g) * (1.5 / W ** 0.5)).to(dtype)
    down = (torch.randn((E, W, F), generator=g) / F ** 0.5).to(dtype)
    base = torch.randn((N, W), generator=g).to(dtype)
    z = torch.randn((N, E + same + 3), generator=g) * 2
    corr = torch.randn(E + same, generator=g) * 0.2
    chosen, weight = P.choose_experts(z[:, :E + same].double(), corr.double(), top, 1.7)
    choice, got_w, gate = o.moe_route_groups(z.cuda(), E + same, top, renorm=True, correction=corr.cuda(), scale=1.7,
                                             extra=E + same)
    assert torch.equal(choice.cpu().long(), chosen)
    assert float((got_w.cpu().double() - weight).abs().max()) < 1e-6
    assert float((gate.cpu() - torch.sigmoid(z[:, E + same])).abs().max()) < 1e-6
    st = None if dtype == torch.float32 else dtype
    want = base.double() * gate.cpu().double()[:, None]
    for n in range(N):
        for j, e in enumerate(chosen[n].tolist()):
            x = h[n:n + 1].double()
            if e < E:
                x = P.gated({"x.gate": gu[e, :F].double(), "x.up": gu[e, F:].double(), "x.down": down[e].double()}, "x", x, 0.9, st)
            want[n] += weight[n, j] * x[0]
    got = o.table_moe(h.cuda(), gu.cuda(), down.cuda(), None, choice, 1.0, base=base.cuda(), base_scale=gate,
                      out_scale=got_w, limit=0.9, identity=same)
    close(got, want, dtype)


# ---------------------------------------------------------------- the engine against the plain implementation


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which,index", [("A", 0), ("A", 1), ("A", 2), ("B", 3), ("C", 1), ("M", 0), ("M", 1), ("M", 2), ("M", 3)])
def test_every_kind_of_layer_alone(tmp_path, which, index, dtype):
    from lmsf_amd.engine import StepEntry, load_engine_core
    folder, cfg, w = make_model(tmp_path, single_layer(which, index), 3, decisive=dtype == "bfloat16")
    toks = random_tokens(90, cfg["vocab"], 11)
    core = load_engine_core(folder, dtype=dtype, block_size=8, num_pages=16, max_model_len=128, max_num_seqs=2)
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", c)] for c in (37, 2, 30, 1, 1, 1, 18)])["a"]
    check(got, plain_logits(cfg, w, toks), dtype, (which, index), (cfg, w, toks))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "B", "C", "D", "M"])
def test_four_ways_of_cutting_give_the_plain_logits(tmp_path, which, dtype):
    from lmsf_amd.engine import load_engine_core
    folder, cfg, w = make_model(tmp_path, which, 1, decisive=dtype == "bfloat16")
    lens = [150, 1, 37, 260, 5, 64]
    reqs = {"r%d" % i: random_tokens(n, cfg["vocab"], 30 + i) for i, n in enumerate(lens)}
    refs = {rid: plain_logits(cfg, w, toks) for rid, toks in reqs.items()}
    worst32 = 0.0
    if dtype == "float32":
        worst32 = max(rel_err(plain_logits(cfg, w, toks, dtype=torch.float32), refs[rid]) for rid, toks in reqs.items())
    page = 16 if which == "M" else 8
    alone = -(-max(lens) // page) + 1
    for what, steps, pages in (("whole", trace_whole(reqs), alone),
                               ("bulk then single", trace_bulk_then_single(reqs, tail=20), alone),
                               ("portions", trace_portions(reqs, seed=3), alone),
                               ("mixed", trace_mixed(reqs, 512, seed=4), 512 // page)):
        core = load_engine_core(folder, dtype=dtype, block_size=page, num_pages=pages,
                                max_model_len=pages * page, max_num_seqs=4)
        got = replay_in_process(core.executor, steps)
        for rid in reqs:
            check(got[rid], refs[rid], dtype, (what, rid), (cfg, w, reqs[rid]), yardstick=worst32)
        mgr = core.storage.manager
        mgr.check_invariants()
        assert all(mgr.num_free_pages(g) == pages for g in range(len(mgr.groups))) and mgr.num_free_state_slots() == 4
        del core


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("make", [far_token_through_the_state, far_key])
def test_a_far_token_decides(tmp_path, make, dtype):
    """The first token of 400 through the state, or as the one key that stands out; prompts, portions and decoding, the
    slot and the pages used a second time."""
    from lmsf_amd.engine import StepEntry, load_engine_core
    cfg, w, a, b = make(400)
    folder, cfg, w = make_model(tmp_path, cfg, 6, weights=w)
    ra, rb = plain_logits(cfg, w, a), plain_logits(cfg, w, b)
    assert float((ra[-1] - rb[-1]).abs().max()) > 0.3 * float(ra.double().std())
    core = load_engine_core(folder, dtype=dtype, block_size=8, num_pages=51, max_model_len=408, max_num_seqs=1)
    for k, t, r in (("a", a, ra), ("b", b, rb)):
        got = replay(core.executor, StepEntry, {k: t}, [[(k, c)] for c in [330, 3, 50] + [1] * 17])[k]
        check(got, r, dtype, k, (cfg, w, t))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sinks_decide(tmp_path, dtype):
    from lmsf_amd.engine import StepEntry, load_engine_core
    cfg = single_layer("M", 1)
    w = make_weights(cfg, 3)
    w["l0.mix.sink"][:] = torch.tensor([-4.0, 2.0, 5.0, 9.0])
    without = dict(w, **{"l0.mix.sink": torch.full((4,), -1e4)})
    toks = random_tokens(90, cfg["vocab"], 3)
    ref = plain_logits(cfg, w, toks)
    off = row_errs(plain_logits(cfg, without, toks), ref)
    assert float(off.min()) > 0.0 and float((off / bfloat16_limits(cfg, w, toks, ref)).median()) > 3.0
    folder, cfg, w = make_model(tmp_path, cfg, 3, weights=w)
    core = load_engine_core(folder, dtype=dtype, block_size=8, num_pages=16, max_model_len=128, max_num_seqs=2)
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", c)] for c in (1, 37, 2, 30, 1, 1, 18)])["a"]
    check(got, ref, dtype, "sinks", (cfg, w, toks))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("W,streams,lay", [(50, 3, attention(3, 1, 24, 300, rot=10, mlp=moe(3, 1, 2, 14, 1.2))),
                                           (46, 9, attention(2, 2, 272, 33, mlp=dense(21, 0.7))),
                                           (54, 2, mamba(2, 7, 300, 1, 3, 7, mlp=moe(4, 2, 4, 6, 0.8, 1.0, (5, 1.0)))),
                                           (36, 4, mamba(3, 130, 9, 3, 6, 1)),
                                           (64, 12, attention(20, 1, 32, 48, mlp=moe(96, 4, 5, 8, 1.0, 2.0, (16, 1.5))))])
def test_sizes_that_the_fast_kernels_do_not_take(tmp_path, W, streams, lay, dtype):
    """Heads wider than the matrix cores' attention takes, widths that are multiples of two only, odd sizes of values and
    states, states wider than a workgroup's LDS or a wave, more streams than fit registers, many experts."""
    from lmsf_amd.engine import StepEntry, load_engine_core
    folder, cfg, w = make_model(tmp_path, model(59, W, [lay], streams=streams, mult=0.9), 8)
    toks = random_tokens(90, cfg["vocab"], 3)
    core = load_engine_core(folder, dtype=dtype, block_size=16, num_pages=8, max_model_len=128, max_num_seqs=2)
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", c)] for c in (41, 2, 30, 1, 1, 15)])["a"]
    ref = plain_logits(cfg, w, toks)
    if dtype == "float32":
        check(got, ref, dtype, W, (cfg, w, toks))
    else:
        # (a router's close call may flip an expert in a few rows)
        assert (row_errs(got, ref) <= bfloat16_limits(cfg, w, toks, ref)).double().mean() > 0.9


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_from_graphs_equals_eager(tmp_path, dtype):
    from lmsf_amd.engine import StepEntry, load_engine_core
    folder, cfg, w = make_model(tmp_path, "A", 7, decisive=dtype == "bfloat16")
    reqs = {"a": random_tokens(140, cfg["vocab"], 1), "b": random_tokens(111, cfg["vocab"], 2)}
    steps = [[("a", 20), ("b", 3)]] + [[("a", 1), ("b", 1)]] * 100 + [[("a", 1)]] * 20 + [[("b", 1)]] * 8
    outs = []
    for eager in (True, False):
        core = load_engine_core(folder, dtype=dtype, block_size=8, num_pages=40, max_model_len=160, max_num_seqs=2,
                                enforce_eager=eager)
        outs.append(replay(core.executor, StepEntry, reqs, steps))
    for k, t in reqs.items():
        assert torch.equal(outs[0][k], outs[1][k]), k
        check(outs[1][k], plain_logits(cfg, w, t), dtype, k, (cfg, w, t))


def draw_config(seed):
    rng = random.Random(seed)
    pick = rng.choice

    def mlp():
        if rng.random() < 0.2:
            return None
        if rng.random() < 0.3:
            return dense(pick([8, 20, 64, 100]), pick([0.5, 1.0, 3.0]))
        experts, same = pick([1, 2, 3, 5, 8, 12]), pick([0, 1, 2, 5])
        return moe(experts, same, pick([t for t in (1, 2, 3, 4) if t <= experts + same]), pick([8, 20, 64, 96]),
                   pick([0.6, 1.0, 2.5]), pick([0.5, 1.0, 2.5]), pick([None, (12, 1.0), (64, 0.7)]))

    layers = []
    for i in range(pick([2, 3, 4])):
        if rng.random() < 0.5:
            G, d = pick([1, 2, 3]), pick([8, 12, 20, 40, 64])
            layers.append(attention(G * pick([1, 2, 3]), G, d, pick([6, 9, 12, 24, 80]), rot=pick([d, d // 4 * 2]),
                                    base=pick([100.0, 1e4, 1e6]), scaling=pick([None, (2.0, 50, 8.0, 1.0), (16.0, 8, 2.0, 0.5)]),
                                    scale=pick([None, 0.2]), softcap=pick([3.0, 30.0]), mlp=mlp()))
        else:
            G, parts = pick([1, 2, 3]), pick([1, 2, 3])
            layers.append(mamba(G * parts * pick([1, 2]), pick([4, 10, 16, 33, 64]), pick([4, 9, 16, 32, 64, 128]), G,
                                pick([1, 2, 4, 5]), parts, mlp=mlp()))
    n = len(layers)
    start = pick(range(n))
    loop = pick([None, (start, pick(range(start + 1, n + 1)), 2)])
    cfg = model(pick([41, 97, 256, 331]), pick([40, 72, 100, 136, 256]), layers, streams=pick([1, 2, 3, 4, 6]),
                mult=pick([0.4, 0.7, 1.0]), cap=pick([5.0, 20.0]), loop=loop, eps=pick([1e-5, 1e-6]))
    return cfg, pick([4, 8, 16, 32]), [pick([1, 2, 5, 17, 40, 77, 130, 200, 300]) for _ in range(5)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [1, 2, 3, 4, 5, 6, 7, 8])
def test_a_configuration_drawn_at_random(tmp_path, seed, dtype):
    from lmsf_amd.engine import load_engine_core
    cfg, page, lens = draw_config(seed)
    folder, cfg, w = make_model(tmp_path, cfg, seed, decisive=dtype == "bfloat16")
    reqs = {"r%d" % i: random_tokens(n, cfg["vocab"], 50 + i) for i, n in enumerate(lens)}
    refs = {rid: plain_logits(cfg, w, toks) for rid, toks in reqs.items()}
    worst32 = 0.0
    if dtype == "float32":
        worst32 = max(rel_err(plain_logits(cfg, w, toks, dtype=torch.float32), refs[rid]) for rid, toks in reqs.items())
    alone = -(-max(lens) // page) + 1
    for what, steps, pages in (("whole", trace_whole(reqs), alone),
                               ("bulk then single", trace_bulk_then_single(reqs, tail=8), alone),
                               ("portions", trace_portions(reqs, seed=seed), alone),
                               ("mixed", trace_mixed(reqs, 512, seed=seed), 512 // page)):
        core = load_engine_core(folder, dtype=dtype, block_size=page, num_pages=pages, max_model_len=pages * page,
                                max_num_seqs=4)
        got = replay_in_process(core.executor, steps)
        for rid in reqs:
            assert torch.isfinite(got[rid]).all(), (what, rid, cfg)
            check(got[rid], refs[rid], dtype, (what, rid, cfg, page), (cfg, w, reqs[rid]), yardstick=worst32)
        core.storage.manager.check_invariants()
        assert core.storage.manager.num_free_state_slots() == 4
        del core


def test_greedy_generation_through_the_entry_point(tmp_path):
    from lmsf_amd.engine import LLM
    from lmsf_amd.sampling import SamplingParams
    folder, cfg, w = make_model(tmp_path, "A", 2)
    prompts = [random_tokens(n, cfg["vocab"], 40 + n) for n in (1, 9, 40)]
    llm = LLM(model=folder, dtype="float32", block_size=8, num_gpu_blocks_override=40, max_num_seqs=2,
              prefill_chunk_size=16, max_model_len=200)
    outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert list(o.outputs[0].token_ids) == greedy(cfg, w, p, 6)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_trace_runner_as_a_program(tmp_path, dtype):
    """bin/trace_run as a child process on a model folder: it picks the class by config.json, and a mixed schedule in a
    pool of 256 tokens with four state slots gives the plain logits."""
    folder, cfg, w = make_model(tmp_path, "A", 4, decisive=dtype == "bfloat16")
    lens = [90, 1, 37, 120, 5, 64]
    reqs = {"r%d" % i: random_tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate(lens)}
    steps = trace_mixed(reqs, 256, seed=5)
    got = replay_with_program(os.path.join(ROOT, "bin", "trace_run"), folder, dtype, steps, str(tmp_path / "out"), 256,
                              cfg["vocab"])
    for rid, toks in reqs.items():
        check(got[rid], plain_logits(cfg, w, toks), dtype, rid, (cfg, w, toks))


def test_the_command_line_generates(tmp_path):
    folder, cfg, w = make_model(tmp_path, "D", 3)
    prompt = random_tokens(11, cfg["vocab"], 9)
    proc = subprocess.run([os.path.join(ROOT, "bin", "lmsf_generate"), "--model", folder, "--dtype", "float32",
                           "--gpu-memory-utilization", "0.5", "--block-size", "8", "--max-model-len", "64",
                           "--prompt-ids", ",".join(map(str, prompt)), "--temperature", "0", "--presence-penalty", "0",
                           "--max-tokens", "8",
                           "--ignore-eos"], stdout=subprocess.PIPE, stderr=subprocess.PIPE, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-3000:]
    assert [int(t) for t in proc.stdout.strip().splitlines()[0].split()] == greedy(cfg, w, prompt, 8)
