"""Gurapel on the GPU: the new kernels alone against the plain implementation's function of the same mechanism, every
kind of layer alone and the whole model through the engine's step function in float32 and bfloat16 under the ways of
cutting a request into steps, keys at a window's edges and far away made to decide the logits, pages and state slots
used again, long decoding from graphs, configurations drawn at random, and generation through the entry point."""
import os
import random
import subprocess
from types import SimpleNamespace

import pytest
import torch

import plain_gurapel as P
from gurapel_helpers import (bfloat16_limits, delta, far_token_through_the_memory, far_token_through_the_recurrence, greedy,
                             make_model, model, moe, pair, plain_logits, rel_err, replay, single_layer, window_edge,
                             within)
from helpers import (random_tokens, replay_in_process, replay_with_program, trace_bulk_then_single, trace_mixed,
                     trace_portions, trace_whole)

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


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,blocks,lens", [(24, 3, [5, 1, 17]), (40, 1, [31, 32, 33]), (12, 12, [64, 65, 2]),
                                            (192, 3, [130, 1, 70]), (256, 2, [1, 1, 1]), (96, 3, [200, 3, 100]),
                                            (320, 5, [90] * 3), (20, 4, [1, 1, 1]), (512, 16, [600])])
def test_the_linear_recurrence_from_states_an_earlier_step_left(dtype, C, blocks, lens):
    """Segments in scattered slots, shorter than a chunk, a chunk long, one token more and many chunks, single tokens
    beside them and alone (the step's own kernel); blocks that the matrix cores take and blocks that they do not."""
    o = ops()
    g = torch.Generator().manual_seed(C + blocks)
    slots = [2, 0, 3][:len(lens)]
    N, c = sum(lens), C // blocks
    u = torch.randn((N, C), generator=g).to(dtype)
    y = (torch.randn((N, 2 * C), generator=g) * 1.5).to(dtype)
    wr, wi = [(torch.randn((blocks, c, c), generator=g) / c ** 0.5).to(dtype) for _ in range(2)]
    br, bi = torch.randn((C,), generator=g) * 2 - 1, torch.randn((C,), generator=g)
    lam = torch.randn((C,), generator=g) * 2 - 2
    rate = 8.0 * torch.nn.functional.softplus(lam)
    state0 = torch.randn((5, C + 3), generator=g)
    r_pre = P.block_linear(u.double(), wr.double(), br.double().view(blocks, c))
    i_pre = P.block_linear(u.double(), wi.double(), bi.double().view(blocks, c))
    log_a = -8.0 * torch.sigmoid(r_pre) * torch.nn.functional.softplus(lam.double())
    a, b = torch.exp(log_a), torch.sqrt(-torch.expm1(2 * log_a)) * torch.sigmoid(i_pre) * u.double()
    want, st = torch.empty((N, C), dtype=torch.float64), state0[:, :C].double().clone()
    at = 0
    for n, slot in zip(lens, slots):
        for t in range(at, at + n):
            st[slot] = a[t] * st[slot] + b[t]
            want[t] = st[slot]
        at += n
    # from a zero state that is the plain implementation's function
    zero = P.gated_linear_recurrence(u[:lens[0]].double(), r_pre[:lens[0]], i_pre[:lens[0]], lam.double())
    carried = state0[slots[0], :C].double() * torch.cumprod(a[:lens[0]], 0)
    assert (zero + carried - want[:lens[0]]).abs().max() < 1e-9
    state = state0.cuda()
    got = o.linear_recurrence(u.cuda(), wr.cuda(), br.cuda(), wi.cuda(), bi.cuda(), rate.cuda(), y.cuda()[:, :C], state,
                              batch_of(lens, slots))
    close(got, want * P.gelu_tanh(y[:, :C].double()), dtype)
    # (the bfloat16 gates' products add up in float32 too: the state keeps float32's digits in both types)
    assert float((state.cpu()[:, :C].double() - st).abs().max()) <= 2e-5 * max(1.0, float(st.abs().max()))
    assert torch.equal(state.cpu()[:, C:], state0[:, C:])
    assert torch.equal(state.cpu()[1], state0[1]) and torch.equal(state.cpu()[4], state0[4])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,lens", [(3, 1, 8, 20, [5, 1, 17]), (2, 2, 64, 96, [70, 2, 9]), (1, 1, 24, 8, [1, 1, 1]),
                                            (4, 2, 128, 40, [33, 64]), (6, 3, 33, 65, [9]), (2, 1, 200, 12, [18, 7])])
def test_the_delta_rule_with_one_decay_a_head(dtype, H, G, d, dv, lens):
    o = ops()
    g = torch.Generator().manual_seed(H * 100 + d)
    slots = [2, 0, 3][:len(lens)]
    N, rep = sum(lens), H // G
    qkv = (torch.randn((N, 2 * G * d + H * dv), generator=g) * 0.7).to(dtype)
    ba = torch.randn((N, 2 * H + 3), generator=g) * 2
    dt_bias, a_log = torch.randn((H,), generator=g), torch.rand((H,), generator=g) * 2 - 1.5
    pd = qkv.double()
    q = (P.unit(pd[:, :G * d].reshape(N, G, d)) * d ** -0.5).repeat_interleave(rep, 1)
    k = P.unit(pd[:, G * d:2 * G * d].reshape(N, G, d)).repeat_interleave(rep, 1)
    v = pd[:, 2 * G * d:].reshape(N, H, dv)
    beta = torch.sigmoid(ba[:, :H].double())
    decay = torch.exp(-torch.exp(a_log.double()) * torch.nn.functional.softplus(ba[:, H:2 * H].double() + dt_bias.double()))
    floats = o.gated_delta_state_floats(H, d, dv)
    state = torch.zeros((5, floats), device="cuda")
    got = o.gated_delta(qkv.cuda(), 0, G * d, 2 * G * d, ba.cuda()[:, H:2 * H], dt_bias.cuda(), a_log.cuda(), ba.cuda(), state,
                        batch_of(lens, slots), H, G, d, dv, d ** -0.5, 1e-6, per_head=True)
    at = 0
    for n in lens:
        part = slice(at, at + n)
        want = P.delta_rule(q[part], k[part], v[part], beta[part], decay[part]).reshape(n, -1)
        assert float((got[part].double().cpu() - want).abs().max()) <= 3e-5 * max(1.0, float(want.abs().max()))
        at += n
    assert float(state[1].abs().max()) == 0.0 and float(state[4].abs().max()) == 0.0


@pytest.mark.parametrize("dtype,exact", [(torch.float32, True), (torch.bfloat16, True), (torch.bfloat16, False)])
@pytest.mark.parametrize("H,G,D,window", [(4, 2, 64, 37), (3, 1, 192, 90), (16, 1, 128, 0), (2, 2, 16, 1), (5, 5, 96, 200),
                                          (20, 1, 256, 64)])
def test_a_distance_takes_its_part_off_the_scores(dtype, exact, H, G, D, window):
    """All three attention kernels (the general one in float32; the prefill and decode kernels of the matrix cores in
    bfloat16, with float32 and with rounded weights) under a cap, a window, and requests of one and of many tokens."""
    from torch_ops import TorchOps
    o = ops()
    g = torch.Generator().manual_seed(5)
    ps = 16
    lens, first = [70, 1, 1, 130], [0, 155, 3, 20]
    pages = 40
    kp = (torch.randn((pages, G, ps, D), generator=g) * 1.5).to(dtype)
    vp = torch.randn((pages, G, D, ps), generator=g).to(dtype)
    N = sum(lens)
    q = (torch.randn((N, H * D), generator=g) * 1.5).to(dtype)
    tables = torch.stack([torch.randperm(pages, generator=g)[:10] for _ in lens]).int()
    bias = torch.stack([torch.rand((H,), generator=g) * 2, torch.rand((H,), generator=g)])
    b = batch_of(lens, [0, 1, 2, 3], first, dev="cpu")
    args = (tables, b.seg_of_token, b.positions, H, G, D, D ** -0.5, window)
    want = TorchOps().paged_attention(q.float(), kp.float(), vp.float(), *args, softcap=6.0, distance_bias=bias)
    bc = batch_of(lens, [0, 1, 2, 3], first)
    for batch in (bc, None):
        got = o.paged_attention(q.cuda(), kp.cuda(), vp.cuda(), tables.cuda(), bc.seg_of_token, bc.positions, H, G, D,
                                D ** -0.5, window, batch=batch, softcap=6.0, distance_bias=bias.cuda(), weights_f32=exact)
        close(got, want, dtype)
    if window != 1:
        plain = TorchOps().paged_attention(q.float(), kp.float(), vp.float(), *args, softcap=6.0)
        assert float((plain - want).abs().max()) > 0.05


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_far_key_against_the_distance(dtype):
    """One key among 300 stands out (its score is at the cap); with a small r1 it keeps nearly all the weight at every
    distance, with a large one it loses it, as r1 ln(1 + r2 n) says: prompts and single tokens."""
    from torch_ops import TorchOps
    o = ops()
    g = torch.Generator().manual_seed(8)
    H, G, D, ps, n = 2, 1, 64, 8, 300
    pages = n // ps + 1
    kp, vp = torch.randn((pages, G, ps, D), generator=g) * 0.1, torch.randn((pages, G, D, ps), generator=g)
    far = torch.randn((D,), generator=g)
    kp[0, 0, 3] = far * 4.0
    q = (far * 4.0).repeat(n, H)
    bias = torch.tensor([[0.05, 6.0], [0.5, 0.5]])
    table = torch.arange(pages).int()[None]
    seg, pos = torch.zeros(n).int(), torch.arange(n).int()
    kp, vp, q = kp.to(dtype), vp.to(dtype), q.to(dtype)
    want = TorchOps().paged_attention(q.float(), kp.float(), vp.float(), table, seg, pos, H, G, D, 0.125, softcap=12.0,
                                      distance_bias=bias)
    value = vp[0, 0, :, 3].float()
    assert float((want[n - 1, :D] - value).abs().max()) < 0.05 and float((want[n - 1, D:] - value).abs().max()) > 0.3
    got = o.paged_attention(q.cuda(), kp.cuda(), vp.cuda(), table.cuda(), seg.cuda(), pos.cuda(), H, G, D, 0.125,
                            softcap=12.0, distance_bias=bias.cuda(), weights_f32=True)
    close(got, want, dtype)
    last = o.paged_attention(q[n - 1:].contiguous().cuda(), kp.cuda(), vp.cuda(), table.cuda(), seg[:1].cuda(),
                             pos[n - 1:].contiguous().cuda(), H, G, D, 0.125, softcap=12.0, distance_bias=bias.cuda(),
                             weights_f32=True)
    close(last, want[n - 1:], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rot", [0, 6])
@pytest.mark.parametrize("H,G,d,dv,ps", [(4, 2, 12, 20, 4), (1, 1, 64, 64, 16), (6, 3, 7, 5, 8), (2, 1, 96, 128, 16)])
def test_every_head_of_queries_and_keys_normed_with_a_weight(dtype, rot, H, G, d, dv, ps):
    from torch_ops import TorchOps
    o = ops()
    g = torch.Generator().manual_seed(d + dv)
    N, pages, D = 9, 5, (max(d, dv) + 15) // 16 * 16
    p = (torch.randn((N, (H + G) * d + G * dv), generator=g) * 2).to(dtype)
    wq, wk = 1 + 0.3 * torch.randn((d,), generator=g), 1 + 0.3 * torch.randn((d,), generator=g)
    pos = torch.tensor([0, 1, 2, 3, 4, 17, 18, 39, 7]).int()
    slots = torch.tensor([0, 1, ps - 1, ps, 2 * ps + 1, 3 * ps, 4 * ps + ps - 1, -1, 2], dtype=torch.int32)
    table = torch.randn((40, rot), generator=g) if rot else None
    outs = []
    for op, dev, dt in ((TorchOps(), "cpu", torch.float32), (o, "cuda", dtype)):
        pc = p.to(dev).to(dt)
        kp = torch.full((pages, G, ps, D), 9.0, dtype=dt, device=dev)
        vp = torch.full((pages, G, D, ps), 9.0, dtype=dt, device=dev)
        qa = op.attn_prepare(pc[:, :H * d], pc[:, H * d:(H + G) * d], pc[:, (H + G) * d:], H, G, d, dv, D, pos.to(dev),
                             slots.to(dev), kp, vp, table=table.to(dev) if rot else None, unit_norm_eps=1e-5,
                             q_weight=wq.to(dev), k_weight=wk.to(dev))
        outs.append((qa, kp, vp))
    for got, want in zip(outs[1], outs[0]):
        close(got, want, dtype, scale=9.0)
    q = P.rms(p[:, :H * d].double().view(N, H, d), 1e-5) * wq.double()
    if not rot:
        close(outs[1][0].view(N, H, D)[..., :d], q, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,W", [(1, 48), (3, 50), (7, 2048), (600, 96), (530, 4100), (5, 4100), (2, 12288), (1, 12290), (513, 2048)])
def test_a_sublayers_output_and_a_pairs_join_the_stream(dtype, N, W):
    """stream += norm(v), v a mixer's output or the mean of a pair's, each normed: widths that a workgroup holds in
    registers and widths that go the other way, one row and many, rows at a stride."""
    from lmsf_amd.ops.handles import NormedPair
    o = ops()
    g = torch.Generator().manual_seed(W)
    a, b = [(torch.randn((N, W + 8), generator=g) * s).to(dtype) for s in (3.0, 0.1)]
    wa, wb, wn = [1 + 0.3 * torch.randn((W,), generator=g) for _ in range(3)]
    x0 = torch.randn((N, W), generator=g) * 2
    va, vb = a[:, :W].double(), b[:, :W].double()
    mean = 0.5 * (P.rms(va, 1e-5) * wa.double() + P.rms(vb, 1e-5) * wb.double())
    ac, bc = a.cuda()[:, :W], b.cuda()[:, :W]
    for v, branch in ((va, ac), (mean, NormedPair(ac, bc, wa.cuda(), wb.cuda(), 1e-5, 0.5))):
        want = x0.double() + P.rms(v, 1e-6) * wn.double()
        for want_out in (True, False):
            x = x0.cuda()
            out = o.norm_add(branch, wn.cuda(), 1e-6, x, want_out=want_out)
            # (a pair that goes the other way is rounded to the run's type in between)
            close(x, want, dtype if W % 4 else torch.float32)
            if want_out:
                assert torch.equal(out, x.to(dtype))
            else:
                assert out is None


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,taps,act", [(24, 2, None), (130, 3, "silu"), (514, 4, None), (600, 5, "silu"), (33, 4, "silu"),
                                        (40, 6, None)])
def test_the_short_convolution_across_segments_of_every_length(dtype, C, taps, act):
    """Segments shorter than the filter, single tokens between longer ones, borders inside and on the edges of the tiles
    of tokens that a thread walks, states that an earlier step left."""
    o = ops()
    g = torch.Generator().manual_seed(C)
    lens = [1, 2, 1, 3, 40, 1, 17, 16, 5, 9]
    slots = [7, 0, 3, 11, 2, 9, 4, 1, 8, 5]
    N = sum(lens)
    u = torch.randn((N, C + 6), generator=g).to(dtype)
    w = (torch.randn((C, taps), generator=g) * 0.6).to(dtype)
    bias = torch.randn((C,), generator=g).to(dtype)
    state0 = torch.randn((12, C * (taps - 1) + 3), generator=g)
    want, after, at = [], state0.clone(), 0
    for n, slot in zip(lens, slots):
        old = state0[slot, :C * (taps - 1)].reshape(C, taps - 1).t().double()
        seq = torch.cat([old, u[at:at + n, :C].double()], 0)
        y = P.short_conv(seq, w.double(), bias.double())[taps - 1:]
        want.append(P.silu(y) if act else y)
        after[slot, :C * (taps - 1)] = seq[-(taps - 1):].t().reshape(-1).float()
        at += n
    state = state0.cuda()
    got = o.short_conv(u.cuda()[:, :C], w.cuda(), bias.cuda(), state, batch_of(lens, slots), act)
    close(got, torch.cat(want), dtype)
    assert torch.equal(state.cpu(), after)


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_embedding_adds_the_positions_vector(dtype):
    g = torch.Generator().manual_seed(2)
    V, W, n = 29, 44, 50
    table, places = torch.randn((V, W), generator=g).to(dtype), torch.randn((n, W), generator=g).to(dtype)
    ids, pos = torch.tensor([0, 28, 5, 5, 9]).int(), torch.tensor([0, 1, 7, 49, 49]).int()
    x, rounded = ops().position_embedding(ids.cuda(), pos.cuda(), table.cuda(), places.cuda(), 0.3)
    want = table[ids.long()].double() * 0.3 + places[pos.long()].double()
    assert x.dtype == torch.float32 and rounded.dtype == dtype
    assert float((x.double().cpu() - want).abs().max()) < 1e-6
    assert torch.equal(rounded, x.to(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,E,top,F,W", [(3, 4, 2, 24, 48), (70, 8, 3, 64, 128), (1, 3, 1, 10, 36), (300, 6, 2, 96, 64),
                                         (40, 5, 5, 32, 96), (9, 70, 6, 16, 32)])
def test_gated_experts_weighted_by_the_softmax_over_the_chosen(dtype, N, E, top, F, W):
    """Router and experts, streamed (few pairs, float32 at any number) and grouped on the matrix cores."""
    o = ops()
    g = torch.Generator().manual_seed(N + E)
    h = torch.randn((N, W), generator=g).to(dtype)
    gu = (torch.randn((E, 2 * F, W), generator=g) * (1.5 / W ** 0.5)).to(dtype)
    down = (torch.randn((E, W, F), generator=g) / F ** 0.5).to(dtype)
    z = torch.randn((N, E + 3), generator=g) * 2
    chosen, weight = P.choose_experts(z[:, :E].double(), top)
    choice, got_w = o.moe_route_groups(z.cuda(), E, top, renorm=True)
    assert torch.equal(choice.cpu().long(), chosen)
    assert float((got_w.cpu().double() - weight).abs().max()) < 1e-6
    st = None if dtype == torch.float32 else dtype
    want = torch.zeros((N, W), dtype=torch.float64)
    for n in range(N):
        for j, e in enumerate(chosen[n].tolist()):
            tw = {"x.gate": gu[e, :F].double(), "x.up": gu[e, F:].double(), "x.down": down[e].double()}
            want[n] += weight[n, j] * P.expert(tw, "x", h[n:n + 1].double(), st)[0]
    got = o.table_moe(h.cuda(), gu.cuda(), down.cuda(), None, choice, 1.0, out_scale=got_w)
    close(got, want, dtype)


# ---------------------------------------------------------------- the engine against the plain implementation


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which,index", [("A", 0), ("A", 1), ("A", 2), ("B", 2), ("M", 0), ("M", 1), ("M", 2)])
def test_every_kind_of_layer_alone(tmp_path, which, index, dtype):
    from lmsf_amd.engine import StepEntry, load_engine_core
    folder, cfg, w = make_model(tmp_path, single_layer(which, index), 3, decisive=dtype == "bfloat16")
    toks = random_tokens(90, cfg["vocab"], 11)
    core = load_engine_core(folder, dtype=dtype, block_size=8, num_pages=16, max_model_len=128, max_num_seqs=2)
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", c)] for c in (37, 2, 30, 1, 1, 1, 18)])["a"]
    check(got, plain_logits(cfg, w, toks), dtype, (which, index), (cfg, w, toks))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("W,lay", [(50, pair(3, 1, 24, 300, 21, 30, 2, 3, mlp=moe(3, 2, 14))),
                                   (46, pair(2, 2, 272, 33, 40, 28, 7, 2)), (54, delta(2, 1, 250, 7, 3, mlp=moe(4, 4, 6))),
                                   (64, pair(20, 1, 32, 48, 77, 64, 1, 4, mlp=moe(96, 5, 8)))])
def test_sizes_that_the_fast_kernels_do_not_take(tmp_path, W, lay, dtype):
    """Heads wider than the matrix cores' attention takes, widths that are multiples of two only, more query heads a key
    head than a workgroup's block, many experts."""
    from lmsf_amd.engine import StepEntry, load_engine_core
    folder, cfg, w = make_model(tmp_path, model(59, W, [lay], positions=200), 8)
    toks = random_tokens(90, cfg["vocab"], 3)
    core = load_engine_core(folder, dtype=dtype, block_size=16, num_pages=8, max_model_len=128, max_num_seqs=2)
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", c)] for c in (41, 2, 30, 1, 1, 15)])["a"]
    ref = plain_logits(cfg, w, toks)
    if dtype == "float32":
        check(got, ref, dtype, W, (cfg, w, toks))
    else:
        # (a router's close call may flip an expert in a few rows)
        from gurapel_helpers import row_errs
        assert (row_errs(got, ref) <= bfloat16_limits(cfg, w, toks, ref)).double().mean() > 0.9


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "B", "C", "D", "M"])
def test_four_ways_of_cutting_give_the_plain_logits(tmp_path, which, dtype):
    from lmsf_amd.engine import load_engine_core
    folder, cfg, w = make_model(tmp_path, which, 1, decisive=dtype == "bfloat16")
    lens = [150, 1, 37, 260, 5, 64]
    reqs = {"r%d" % i: random_tokens(n, cfg["vocab"], 30 + i) for i, n in enumerate(lens)}
    refs = {rid: plain_logits(cfg, w, toks) for rid, toks in reqs.items()}
    page = 16 if which == "M" else 8
    alone = -(-max(lens) // page) + 1
    for what, steps, pages in (("whole", trace_whole(reqs), alone),
                               ("bulk then single", trace_bulk_then_single(reqs, tail=20), alone),
                               ("portions", trace_portions(reqs, seed=3), alone),
                               ("mixed", trace_mixed(reqs, 512, seed=4), 512 // page)):
        core = load_engine_core(folder, dtype=dtype, block_size=page, num_pages=pages,
                                max_model_len=min(pages * page, cfg["max_positions"]), max_num_seqs=4)
        got = replay_in_process(core.executor, steps)
        for rid in reqs:
            check(got[rid], refs[rid], dtype, (what, rid), (cfg, w, reqs[rid]))
        mgr = core.storage.manager
        mgr.check_invariants()
        assert all(mgr.num_free_pages(g) == pages for g in range(len(mgr.groups))) and mgr.num_free_state_slots() == 4
        del core


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which,index,n", [("A", 0, 60), ("M", 0, 130), ("M", 2, 200)])
def test_keys_at_a_windows_edges_decide_or_do_not(tmp_path, which, index, n, dtype):
    """Peaked attention with a window: changing the token at its first place moves the plain implementation's last
    logits, changing the one before it moves nothing; the engine agrees on each sequence, in prompts and decoding."""
    from lmsf_amd.engine import StepEntry, load_engine_core
    cfg, w, seqs, ref = window_edge(which, index, n)
    folder, cfg, w = make_model(tmp_path, cfg, 5, weights=w)
    inside, base = ref["inside"][-1].double(), ref["base"][-1].double()
    assert float((inside - base).abs().max()) > 0.1 * float(ref["base"].double().std())
    assert float((ref["outside"][-1] - ref["base"][-1]).abs().max()) == 0.0
    for cuts in ([n], [n - 15] + [1] * 15, [n - 23, 2, 21]):
        core = load_engine_core(folder, dtype=dtype, block_size=4, num_pages=n // 4 + 2, max_model_len=n + 4, max_num_seqs=2)
        for k, t in seqs.items():
            got = replay(core.executor, StepEntry, {k: t}, [[(k, c)] for c in cuts])[k]
            check(got, ref[k], dtype, (k, cuts), (cfg, w, t))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("make", [far_token_through_the_memory, far_token_through_the_recurrence])
def test_a_far_token_decides_through_the_state(tmp_path, make, dtype):
    from lmsf_amd.engine import StepEntry, load_engine_core
    cfg, w, a, b = make(200)
    folder, cfg, w = make_model(tmp_path, cfg, 6, weights=w)
    ra, rb = plain_logits(cfg, w, a), plain_logits(cfg, w, b)
    assert float((ra[-1] - rb[-1]).abs().max()) > 0.3 * float(ra.double().std())
    core = load_engine_core(folder, dtype=dtype, block_size=8, num_pages=26, max_model_len=208, max_num_seqs=1)
    for k, t, r in (("a", a, ra), ("b", b, rb)):
        got = replay(core.executor, StepEntry, {k: t}, [[(k, c)] for c in [130, 3, 50] + [1] * 17])[k]
        if dtype == "float32":
            check(got, r, dtype, k, (cfg, w, t))
        else:
            # (the first token's part of the last logits, far above what rounding costs; experts may be a close call)
            near, far = (float((got[-1].double().cpu() - x[-1].double()).pow(2).mean()) for x in ((ra, rb) if k == "a" else (rb, ra)))
            assert near < 0.1 * far, (k, near, far)


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
        if rng.random() < 0.25:
            return None
        experts = pick([1, 2, 3, 5, 8, 12])
        return moe(experts, pick([t for t in (1, 2, 3, 4) if t <= experts]), pick([8, 20, 64, 100]))

    layers = []
    for i in range(pick([2, 3, 4, 5])):
        G = pick([1, 2, 3])
        if rng.random() < 0.6:
            blocks = pick([1, 2, 3, 5])
            layers.append(pair(G * pick([1, 2, 3]), G, pick([8, 12, 15, 20, 40, 64]), pick([6, 8, 12, 24, 80]),
                               pick([1, 5, 16, 37, 64, 130, 500]), blocks * pick([8, 20, 32, 64]), blocks, pick([1, 2, 4, 5]),
                               scale=pick([None, 0.2]), softcap=pick([4.0, 30.0]), mlp=mlp()))
        else:
            layers.append(delta(G * pick([1, 2]), G, pick([8, 12, 20, 24, 64, 72]), pick([4, 8, 20, 33, 64, 100]),
                                pick([1, 2, 4, 5]), mlp=mlp()))
    cfg = model(pick([41, 97, 256, 331]), pick([40, 72, 100, 136, 256]), layers, eps=pick([1e-5, 1e-6]),
                scale=pick([0.5, 1.0, 3.0]), positions=1024)
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
                           "--prompt-ids", ",".join(map(str, prompt)), "--temperature", "0", "--max-tokens", "8",
                           "--ignore-eos"], stdout=subprocess.PIPE, stderr=subprocess.PIPE, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-3000:]
    assert [int(t) for t in proc.stdout.strip().splitlines()[0].split()] == greedy(cfg, w, prompt, 8)
