"""Zunilorn through the engine's host side (configuration, weights by name, pages, state slots, the loop, batching,
scheduler, sampling) on the CPU, with torch stand-ins for the kernels, against the plain implementation. The kernels
themselves are tested on the GPU (test_zunilorn_gpu.py)."""
import copy
import math

import pytest
import torch

import plain_zunilorn as P
from helpers import random_tokens
from torch_ops import TorchOps
from zunilorn_helpers import (CONFIGS, far_key, far_token_through_the_state, greedy, make_model, make_weights, plain_logits,
                              rel_err, replay, single_layer, write_model)

from lmsf_amd.config import ConfigError, resolve_architecture
from lmsf_amd.engine import EngineArgs, LLMEngine, StepEntry, load_engine_core
from lmsf_amd.parts.rotary import yarn_frequencies
from lmsf_amd.sampling import SamplingParams
from lmsf_amd.weights.loader import WeightsError

TOL = 3e-5
SMALL = ("A", "B", "C", "D")


def build(tmp_path, which, pages=24, block=8, seed=0, **kw):
    folder, cfg, w = make_model(tmp_path, which, seed, spread=kw.pop("spread", 1.0), weights=kw.pop("weights", None))
    core = load_engine_core(folder, dtype="float32", block_size=block, num_pages=pages, max_model_len=pages * block,
                            device="cpu", ops=TorchOps(), max_num_seqs=kw.pop("slots", 4), **kw)
    return core, cfg, w


def agrees(got, cfg, w, toks, ref=None):
    """float32: within TOL of the plain implementation in float64, or within three times what float32 rounding costs
    the plain implementation itself where that is more."""
    ref = plain_logits(cfg, w, toks) if ref is None else ref
    tol = max(TOL, 3 * rel_err(plain_logits(cfg, w, toks, dtype=torch.float32), ref))
    return rel_err(got, ref) < tol


def test_the_architecture_is_found_by_its_name():
    assert resolve_architecture({"architecture": "Zunilorn"}).name == "Zunilorn"


# ---------------------------------------------------------------- the plain implementation's own mechanisms


def test_plain_streams_by_hand():
    X = torch.tensor([[[1.0, 2.0]], [[10.0, 20.0]]])                      # two streams, one token, two entries
    assert P.read_streams(X, torch.tensor([0.5, -1.0])).tolist() == [[-9.5, -19.0]]
    M = torch.tensor([[1.0, 2.0], [0.5, 0.0]])                            # from row to column
    got = P.write_streams(X, M, torch.tensor([1.0, 3.0]), torch.tensor([[4.0, 8.0]]), 0.5)
    assert got.tolist() == [[[1.0 + 5.0 + 2.0, 2.0 + 10.0 + 4.0]], [[2.0 + 6.0, 4.0 + 12.0]]]


def test_plain_state_space_by_hand():
    x = torch.tensor([[[2.0]], [[-1.0]]])
    B, C = torch.tensor([[[1.0, 3.0]], [[0.5, 0.0]]]), torch.tensor([[[1.0, 1.0]], [[2.0, -1.0]]])
    dt, A_log, D = torch.tensor([[0.5], [2.0]]), torch.tensor([0.3]), torch.tensor([0.25])
    S = [0.5 * 1.0 * 2.0, 0.5 * 3.0 * 2.0]
    y0 = S[0] + S[1] + 0.25 * 2.0
    keep = math.exp(-math.exp(0.3) * 2.0)
    S = [keep * S[0] + 2.0 * 0.5 * -1.0, keep * S[1]]
    y1 = 2.0 * S[0] - S[1] - 0.25
    got = P.state_space(x, B, C, dt, A_log, D).flatten().tolist()
    assert abs(got[0] - y0) < 1e-5 and abs(got[1] - y1) < 1e-5
    # heads share the B and C of their group
    g = torch.Generator().manual_seed(1)
    x, B, C = (torch.randn(s, generator=g) for s in ((5, 4, 3), (5, 2, 6), (5, 2, 6)))
    dt, A, D = torch.rand((5, 4), generator=g), torch.randn(4, generator=g), torch.randn(4, generator=g)
    whole = P.state_space(x, B, C, dt, A, D)
    for h, grp in ((0, 0), (1, 0), (2, 1), (3, 1)):
        one = P.state_space(x[:, h:h + 1], B[:, grp:grp + 1], C[:, grp:grp + 1], dt[:, h:h + 1], A[h:h + 1], D[h:h + 1])
        assert (one[:, 0] - whole[:, h]).abs().max() < 1e-6


def test_plain_gate_comes_before_the_norm():
    y, z = torch.tensor([[1.0, 2.0, 3.0, 4.0]]), torch.tensor([[0.5, -1.0, 2.0, 0.0]])
    a = [v * s / (1.0 + math.exp(-s)) for v, s in zip(y[0].tolist(), z[0].tolist())]
    want = []
    for part in (a[:2], a[2:]):
        r = math.sqrt(sum(v * v for v in part) / 2 + 1e-3)
        want += [v / r for v in part]
    got = P.gated_group_norm(y, z, torch.tensor([1.0, 1.0, 1.0, 1.0]), 2, 1e-3)[0].tolist()
    assert max(abs(x - v) for x, v in zip(got, want)) < 1e-6


def test_plain_sink_takes_its_share():
    s = torch.tensor([[0.0, 1.0], [float("-inf"), 2.0]], dtype=torch.float64)
    w = P.softmax_with_sink(s, torch.tensor(0.5, dtype=torch.float64))
    total = 1.0 + math.e + math.exp(0.5)
    assert abs(float(w[0, 0]) - 1.0 / total) < 1e-12 and abs(float(w[0, 1]) - math.e / total) < 1e-12
    assert float(w[1, 0]) == 0.0 and abs(float(w[1, 1]) - math.exp(2.0) / (math.exp(2.0) + math.exp(0.5))) < 1e-12
    nothing_left = P.softmax_with_sink(s, torch.tensor(500.0, dtype=torch.float64))
    assert float(nothing_left.sum()) < 1e-100


def test_plain_frequencies_are_those_of_the_rotation_part():
    for rot in ({"base": 250.0, "dims": 12, "scaling": {"factor": 8.0, "original": 40, "fast": 4.0, "slow": 1.0}},
                {"base": 1e4, "dims": 64, "scaling": {"factor": 2.5, "original": 4096, "fast": 32.0, "slow": 1.0}}):
        f, gain = P.frequencies(rot)
        sc = rot["scaling"]
        mine = yarn_frequencies(rot["dims"], rot["base"], {
            "factor": sc["factor"], "original_max_position_embeddings": sc["original"], "beta_fast": sc["fast"],
            "beta_slow": sc["slow"]})
        assert max(abs(a - b) for a, b in zip(f, mine.tolist())) < 1e-12
        assert abs(gain - (0.1 * math.log(sc["factor"]) + 1.0)) < 1e-12
        # the fastest pair keeps its frequency, the slowest is divided
        assert f[0] == 1.0 and f[-1] < rot["base"] ** (2.0 / rot["dims"] - 1.0)
    assert P.frequencies({"base": 9.0, "dims": 4}) == ([1.0, 9.0 ** -0.5], 1.0)


def test_plain_router_corrects_the_choice_and_not_the_weights():
    z = torch.tensor([[0.0, 3.0, 1.0, 2.0]])
    s = torch.softmax(z, -1)[0]
    chosen, weight = P.choose_experts(z, torch.tensor([5.0, 0.0, 0.0, -5.0]), 2, 2.5)
    assert chosen.tolist() == [[0, 1]]
    assert abs(float(weight[0, 0]) - 2.5 * float(s[0] / (s[0] + s[1]))) < 1e-6 and abs(float(weight.sum()) - 2.5) < 1e-5


def test_plain_activation_bounds_both_operands():
    g, u = torch.tensor([9.0, -9.0, 0.5]), torch.tensor([-7.0, 7.0, 0.25])
    sg = lambda x: 1.0 / (1.0 + math.exp(-1.702 * x))                                       # noqa: E731
    want = [2.0 * sg(2.0) * (-2.0 + 1.0), -9.0 * sg(-9.0) * 3.0, 0.5 * sg(0.5) * 1.25]
    assert max(abs(a - b) for a, b in zip(P.bounded_gate(g, u, 2.0).tolist(), want)) < 1e-6


# ---------------------------------------------------------------- the engine against the plain implementation


@pytest.mark.parametrize("which", SMALL)
def test_whole_prompt(tmp_path, which):
    core, cfg, w = build(tmp_path, which)
    toks = random_tokens(45, cfg["vocab"], 1)
    out = core.executor.step([StepEntry("a", toks, list(range(len(toks))))])
    assert agrees(out, cfg, w, toks)


@pytest.mark.parametrize("which,index", [("A", 0), ("A", 1), ("A", 2), ("B", 0), ("B", 2), ("B", 3), ("C", 0), ("C", 1), ("D", 0)])
def test_every_kind_of_layer_alone(tmp_path, which, index):
    core, cfg, w = build(tmp_path, single_layer(which, index))
    toks = random_tokens(30, cfg["vocab"], 11)
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", c)] for c in (7, 2, 12, 1, 1, 1, 6)])["a"]
    assert agrees(got, cfg, w, toks)


@pytest.mark.parametrize("which", SMALL)
def test_portions_down_to_two_tokens_then_one_by_one(tmp_path, which):
    core, cfg, w = build(tmp_path, which)
    toks = random_tokens(61, cfg["vocab"], 2)
    cuts = [3, 2, 8, 7, 2, 16, 9] + [1] * 14          # portions that end inside and on the edges of pages
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", c)] for c in cuts])["a"]
    assert agrees(got, cfg, w, toks)
    core.storage.manager.check_invariants()


@pytest.mark.parametrize("which", SMALL)
def test_token_by_token_from_the_first(tmp_path, which):
    core, cfg, w = build(tmp_path, which)
    toks = random_tokens(24, cfg["vocab"], 3)
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", 1)] for _ in toks])["a"]
    assert agrees(got, cfg, w, toks)


@pytest.mark.parametrize("which", SMALL)
def test_unequal_requests_together_with_pages_and_slots_used_again(tmp_path, which):
    core, cfg, w = build(tmp_path, which, pages=20, slots=3)     # 160 tokens of room, three state slots
    V = cfg["vocab"]
    reqs = {"a": random_tokens(70, V, 4), "b": random_tokens(1, V, 5), "c": random_tokens(33, V, 6),
            "d": random_tokens(90, V, 7), "e": random_tokens(5, V, 8)}
    steps = [[("a", 30), ("b", 1), ("c", 2)], [("a", 1), ("c", 17), ("e", 2)], [("c", 14), ("a", 38)], [("a", 1), ("e", 3)],
             [("d", 50)], [("d", 39)], [("d", 1)]]
    got = replay(core.executor, StepEntry, reqs, steps)
    for k, t in reqs.items():
        assert agrees(got[k], cfg, w, t), k
    mgr = core.storage.manager
    mgr.check_invariants()
    assert all(mgr.num_free_pages(g) == 20 for g in range(len(mgr.groups))) and mgr.num_free_state_slots() == 3


def test_every_pass_of_the_loop_has_a_cache_and_a_state_of_its_own(tmp_path):
    core, cfg, w = build(tmp_path, "B")
    order = [0, 1, 2, 3, 1, 2, 3, 1, 2, 3]
    assert P.layer_order(cfg) == order and [e.layer for e in core.model.schedule] == order
    pages = [b.k_pages.data_ptr() for b in core.model.bindings if b.k_pages is not None]
    states = [b.state.data_ptr() for b in core.model.bindings if b.state is not None]
    assert len(set(pages)) == 6 and len(set(states)) == 4
    # and the layers of one pass are the layers of the other: one set of weights
    assert len(core.model.blocks) == 4


@pytest.mark.parametrize("make", [far_token_through_the_state, far_key])
def test_a_far_token_reaches_the_last(tmp_path, make):
    """The first token of 150 moves the last logits, through the state or as the one key that stands out; the engine
    carries it through portions, single tokens and a slot that another request has used before."""
    cfg, w, a, b = make(150)
    folder, cfg, w = make_model(tmp_path, cfg, 6, weights=w)
    ra, rb = plain_logits(cfg, w, a), plain_logits(cfg, w, b)
    assert float((ra[-1] - rb[-1]).abs().max()) > 0.3 * float(ra.double().std())
    core = load_engine_core(folder, dtype="float32", block_size=8, num_pages=20, max_model_len=160, device="cpu",
                            ops=TorchOps(), max_num_seqs=1)
    for k, t, ref in (("a", a, ra), ("b", b, rb)):
        got = replay(core.executor, StepEntry, {k: t}, [[(k, c)] for c in [64, 3, 70] + [1] * 13])[k]
        assert agrees(got, cfg, w, t, ref), k


def test_the_sinks_decide_and_the_engine_has_them(tmp_path):
    cfg = single_layer("A", 0)
    w = make_weights(cfg, 3)
    w["l0.mix.sink"][:] = torch.tensor([-4.0, 2.0, 4.0, 8.0])
    without = dict(w, **{"l0.mix.sink": torch.full((4,), -1e4)})
    toks = random_tokens(40, cfg["vocab"], 3)
    ref = plain_logits(cfg, w, toks)
    assert rel_err(plain_logits(cfg, without, toks), ref) > 0.05
    core, cfg, w = build(tmp_path, cfg, weights=w)
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", c)] for c in (1, 20, 2, 1, 1, 15)])["a"]
    assert agrees(got, cfg, w, toks, ref)


def test_greedy_generation_through_the_engine_and_its_scheduler(tmp_path):
    folder, cfg, w = make_model(tmp_path, "A", 2)
    prompts = [random_tokens(n, cfg["vocab"], 20 + n) for n in (9, 23, 2)]
    want = [greedy(cfg, w, p, 6) for p in prompts]
    engine = LLMEngine(EngineArgs(model=folder, dtype="float32", block_size=8, num_gpu_blocks_override=16, max_num_seqs=2,
                                  max_model_len=120, prefill_chunk_size=8, max_num_batched_tokens=12, device="cpu"),
                       ops=TorchOps())
    for i, p in enumerate(prompts):
        engine.add_request(i, p, SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True))
    done = {}
    while engine.has_unfinished_requests():
        for out in engine.step():
            if out.finished:
                done[int(out.request_id)] = list(out.outputs[0].token_ids)
    assert [done[i] for i in range(3)] == want


# ---------------------------------------------------------------- configuration and weights


def test_a_configuration_survives_being_written():
    for name in ("A", "B", "C"):
        cls = resolve_architecture(CONFIGS[name]).config_class
        one = cls.from_dict(CONFIGS[name])
        assert cls.from_dict(one.to_dict()) == one


def test_configuration_faults_name_their_key():
    def parse(cfg):
        return resolve_architecture(cfg).config_class.from_dict(cfg)

    for path, value, word in ((("layers", 0, "mixer", "kv_heads"), 3, "kv_heads"),
                              (("layers", 0, "mixer", "softcap"), -1.0, "softcap"),
                              (("layers", 0, "mixer", "rot", "dims"), 7, "dims"),
                              (("layers", 0, "mixer", "rot", "dims"), 14, "dims"),
                              (("layers", 0, "mixer", "rot", "scaling"), {"factor": 2.0}, "original"),
                              (("layers", 0, "mlp", "router", "top"), 9, "router"),
                              (("layers", 0, "mlp", "router", "identity"), -1, "identity"),
                              (("layers", 0, "mlp", "expert", "limit"), 0, "limit"),
                              (("layers", 0, "mlp", "shared"), {"ff": 3}, "limit"),
                              (("layers", 0, "mlp", "kind"), "sparse", "kind"),
                              (("layers", 1, "mixer", "groups"), 4, "groups"),
                              (("layers", 1, "mixer", "norm_groups"), 7, "norm_groups"),
                              (("layers", 1, "mixer", "conv"), 0, "conv"),
                              (("layers", 1, "mixer", "state"), 2000, "state"),
                              (("layers", 1, "mlp", "limit"), "1", "limit"),
                              (("layers", 1, "type"), "mamba1", "type"),
                              (("loop", "stop"), 4, "loop"),
                              (("loop", "times"), 0, "times"),
                              (("streams",), 0, "streams"),
                              (("streams",), 99, "streams"),
                              (("logit_softcap",), -2.0, "logit_softcap")):
        cfg = copy.deepcopy(CONFIGS["A"])
        at = cfg
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ConfigError, match=word):
            parse(cfg)


def test_weight_faults_are_listed_by_name(tmp_path):
    cfg = CONFIGS["A"]
    w = make_weights(cfg, 0)
    del w["l0.mix.sink"], w["l1.hc2.mix"], w["l0.mlp.correction"]
    w["l1.mix.in"] = w["l1.mix.in"][:-1]
    w["l0.mlp.e5.gate"] = w["l0.mlp.e4.gate"]            # (an expert that returns its input has no tensors)
    folder = write_model(str(tmp_path / "broken"), cfg, w)
    with pytest.raises(WeightsError) as e:
        load_engine_core(folder, dtype="float32", block_size=8, num_pages=4, device="cpu", ops=TorchOps())
    assert {"l0.mix.sink", "l1.hc2.mix", "l0.mlp.correction"} <= set(e.value.missing)
    assert any(n == "l1.mix.in" for n, _, _ in e.value.wrong_shape)
    assert "l0.mlp.e5.gate" in str(e.value)


def test_a_layer_without_a_feed_forward_may_carry_the_tensors_of_one(tmp_path):
    cfg = single_layer("A", 2)
    w = make_weights(cfg, 0)
    w.update({"l0.norm2": torch.ones(48), "l0.hc2.in": torch.ones(3), "l0.hc2.out": torch.ones(3), "l0.hc2.mix": torch.eye(3)})
    core, cfg, w = build(tmp_path, cfg, weights=w)
    toks = random_tokens(12, cfg["vocab"], 1)
    assert agrees(core.executor.step([StepEntry("a", toks, list(range(12)))]), cfg, w, toks)
