"""Gurapel through the engine's host side (configuration, weights by name, pages with windows, state slots, batching,
scheduler, sampling) on the CPU, with torch stand-ins for the kernels, against the plain implementation. The kernels
themselves are tested on the GPU (test_gurapel_gpu.py)."""
import copy
import json
import math
import os

import pytest
import torch

import plain_gurapel as P
from gurapel_helpers import (CONFIGS, far_token_through_the_memory, far_token_through_the_recurrence, greedy, make_model,
                             make_weights, plain_logits, rel_err, replay, single_layer, window_edge, write_model)
from helpers import random_tokens
from torch_ops import TorchOps

from lmsf_amd.config import ConfigError, load_model_config, resolve_architecture
from lmsf_amd.engine import EngineArgs, LLMEngine, StepEntry, load_engine_core
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
    assert resolve_architecture({"architecture": "Gurapel"}).name == "Gurapel"


# ---------------------------------------------------------------- the plain implementation's own mechanisms


def test_plain_distance_bias():
    off = P.distance_bias(torch.tensor([0.5, 2.0]), torch.tensor([0.1, 3.0]), torch.tensor([[0, 4]]))
    assert off.shape == (2, 1, 2) and float(off[:, 0, 0].abs().max()) == 0.0
    assert abs(float(off[0, 0, 1]) - 0.5 * math.log(1.4)) < 1e-6 and abs(float(off[1, 0, 1]) - 2.0 * math.log(13.0)) < 1e-6


def test_plain_linear_recurrence_by_hand():
    """Two tokens of one channel; with log a = 0 nothing is let in, with a = 0 only the input stays."""
    u, r, i = torch.tensor([[2.0], [-1.0]]), torch.tensor([[0.3], [-0.7]]), torch.tensor([[0.1], [1.2]])
    lam = torch.tensor([-0.4])
    sig = lambda z: 1.0 / (1.0 + math.exp(-z))                                              # noqa: E731
    sp = math.log1p(math.exp(-0.4))
    S, want = 0.0, []
    for t in range(2):
        a = math.exp(-8.0 * sig(float(r[t, 0])) * sp)
        S = a * S + math.sqrt(1.0 - a * a) * sig(float(i[t, 0])) * float(u[t, 0])
        want.append(S)
    got = P.gated_linear_recurrence(u.double(), r.double(), i.double(), lam.double())
    assert max(abs(float(got[t, 0]) - want[t]) for t in range(2)) < 1e-6
    closed = P.gated_linear_recurrence(u, torch.full_like(r, -200.0), i, lam)
    assert float(closed.abs().max()) == 0.0
    open_ = P.gated_linear_recurrence(u, torch.full_like(r, 50.0), i, torch.tensor([40.0]))
    assert float((open_ - torch.sigmoid(i) * u).abs().max()) < 1e-6


def test_plain_blocks_have_matrices_of_their_own():
    u = torch.tensor([[1.0, 2.0, 3.0, 4.0]])
    w = torch.tensor([[[1.0, 0.0], [1.0, 1.0]], [[0.0, 2.0], [0.0, 0.0]]])
    got = P.block_linear(u, w, torch.tensor([[0.0, 10.0], [0.5, 0.0]]))
    assert got.tolist() == [[1.0, 13.0, 8.5, 0.0]]


def test_plain_delta_rule_writes_what_it_reads_back():
    g0 = torch.Generator().manual_seed(3)
    k = torch.nn.functional.normalize(torch.randn((2, 1, 5), generator=g0, dtype=torch.float64), dim=-1)
    v = torch.randn((2, 1, 3), generator=g0, dtype=torch.float64)
    ones = torch.ones((2, 1), dtype=torch.float64)
    assert (P.delta_rule(k, k, v, ones, ones) - v).abs().max() < 1e-12
    g, beta = torch.rand((2, 1), generator=g0, dtype=torch.float64), torch.rand((2, 1), generator=g0, dtype=torch.float64)
    q = torch.randn((2, 1, 5), generator=g0, dtype=torch.float64)
    o = P.delta_rule(q, k, v, beta, g)
    S1 = beta[0, 0] * torch.outer(k[0, 0], v[0, 0])
    Sd = g[1, 0] * S1
    S2 = Sd + torch.outer(k[1, 0], beta[1, 0] * (v[1, 0] - Sd.T @ k[1, 0]))
    assert (o[0, 0] - S1.T @ q[0, 0]).abs().max() < 1e-12 and (o[1, 0] - S2.T @ q[1, 0]).abs().max() < 1e-12


def test_plain_router_weighs_the_chosen_alone():
    chosen, weight = P.choose_experts(torch.tensor([[0.0, 3.0, 1.0, 2.0]]), 2)
    assert chosen.tolist() == [[1, 3]]
    assert abs(float(weight[0, 0]) - 1.0 / (1.0 + math.exp(-1.0))) < 1e-6 and abs(float(weight.sum()) - 1.0) < 1e-6


# ---------------------------------------------------------------- the engine against the plain implementation


@pytest.mark.parametrize("which", SMALL)
def test_whole_prompt(tmp_path, which):
    core, cfg, w = build(tmp_path, which)
    toks = random_tokens(45, cfg["vocab"], 1)
    out = core.executor.step([StepEntry("a", toks, list(range(len(toks))))])
    assert agrees(out, cfg, w, toks)


@pytest.mark.parametrize("which,index", [("A", 0), ("A", 1), ("A", 2), ("B", 0), ("B", 2), ("C", 1)])
def test_every_kind_of_layer_alone(tmp_path, which, index):
    core, cfg, w = build(tmp_path, single_layer(which, index))
    toks = random_tokens(30, cfg["vocab"], 11)
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", c)] for c in (7, 2, 12, 1, 1, 1, 6)])["a"]
    assert agrees(got, cfg, w, toks)


@pytest.mark.parametrize("which", SMALL)
def test_portions_down_to_two_tokens_then_one_by_one(tmp_path, which):
    core, cfg, w = build(tmp_path, which)
    toks = random_tokens(61, cfg["vocab"], 2)
    cuts = [3, 2, 8, 7, 2, 16, 9] + [1] * 14          # portions that end inside and on the edges of pages and windows
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


def test_a_window_gives_its_pages_back(tmp_path):
    core, cfg, w = build(tmp_path, "B", pages=30, block=4)
    assert sorted(g.spec.window for g in core.storage.groups) == [1, 7, 19]
    toks = random_tokens(100, cfg["vocab"], 9)
    got = replay(core.executor, StepEntry, {"a": toks}, [[("a", 50)]] + [[("a", 1)]] * 50)
    assert agrees(got["a"], cfg, w, toks)
    assert all(core.storage.manager.num_free_pages(g) == 30 for g in range(3))


def test_keys_just_inside_and_just_outside_a_window_decide_or_do_not(tmp_path):
    """Changing the token at the window's first place moves the last logits, changing the one before it moves nothing;
    the engine agrees with the plain implementation on all three sequences, in a prompt and decoding."""
    cfg, w, seqs, ref = window_edge("A", 0, 40)
    folder, cfg, w = make_model(tmp_path, cfg, 5, weights=w)
    assert float((ref["inside"][-1] - ref["base"][-1]).abs().max()) > 0.1 * float(ref["base"].double().std())
    assert float((ref["outside"][-1] - ref["base"][-1]).abs().max()) == 0.0
    for cuts in ([40], [30] + [1] * 10, [27, 2, 11]):
        core = load_engine_core(folder, dtype="float32", block_size=4, num_pages=12, max_model_len=48, device="cpu",
                                ops=TorchOps(), max_num_seqs=2)
        for k, t in seqs.items():
            got = replay(core.executor, StepEntry, {k: t}, [[(k, c)] for c in cuts])[k]
            assert agrees(got, cfg, w, t, ref[k]), (k, cuts)


@pytest.mark.parametrize("make", [far_token_through_the_memory, far_token_through_the_recurrence])
def test_a_far_token_reaches_the_last_through_the_state(tmp_path, make):
    """The state keeps the first token of 150: it moves the last logits, and the engine carries it through portions,
    single tokens and a slot that another request has used before."""
    cfg, w, a, b = make(150)
    folder, cfg, w = make_model(tmp_path, cfg, 6, weights=w)
    ra, rb = plain_logits(cfg, w, a), plain_logits(cfg, w, b)
    assert float((ra[-1] - rb[-1]).abs().max()) > 0.3 * float(ra.double().std())
    core = load_engine_core(folder, dtype="float32", block_size=8, num_pages=20, max_model_len=160, device="cpu",
                            ops=TorchOps(), max_num_seqs=1)
    for k, t, ref in (("a", a, ra), ("b", b, rb)):
        got = replay(core.executor, StepEntry, {k: t}, [[(k, c)] for c in [64, 3, 70] + [1] * 13])[k]
        assert agrees(got, cfg, w, t, ref), k


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


def test_a_request_is_no_longer_than_there_are_position_vectors(tmp_path):
    folder, cfg, w = make_model(tmp_path, "C", 0)
    arch, parsed = load_model_config(folder)
    assert arch.name == "Gurapel" and parsed.max_position_embeddings == 300
    with pytest.raises(ValueError, match="300"):
        load_engine_core(folder, dtype="float32", block_size=8, num_pages=64, max_model_len=301, device="cpu", ops=TorchOps())


def test_the_number_of_position_vectors_comes_from_the_tensor_where_the_configuration_lacks_it(tmp_path):
    folder, cfg, w = make_model(tmp_path, "D", 0)
    path = os.path.join(folder, "config.json")
    d = json.load(open(path))
    del d["max_positions"]
    with open(path, "w") as f:
        json.dump(d, f)
    assert load_model_config(folder)[1].position_rows == cfg["max_positions"]


def test_a_configuration_survives_being_written(tmp_path):
    cls = resolve_architecture(CONFIGS["A"]).config_class
    one = cls.from_dict(CONFIGS["A"])
    assert cls.from_dict(one.to_dict()) == one


def test_configuration_faults_name_their_key():
    def parse(cfg):
        return resolve_architecture(cfg).config_class.from_dict(cfg)

    for path, value, word in ((("layers", 0, "mixer", "left", "kv_heads"), 3, "kv_heads"),
                              (("layers", 0, "mixer", "left", "softcap"), -1.0, "softcap"),
                              (("layers", 0, "mixer", "right", "blocks"), 5, "blocks"),
                              (("layers", 0, "mlp", "router", "top"), 9, "router"),
                              (("layers", 0, "mlp", "kind"), "dense", "kind"),
                              (("layers", 1, "mixer", "conv"), 0, "conv"),
                              (("layers", 1, "type"), "attention", "type"),
                              (("embedding", "scale"), "1", "scale"),
                              (("max_positions",), 0, "max_positions")):
        cfg = copy.deepcopy(CONFIGS["A"])
        at = cfg
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        with pytest.raises(ConfigError, match=word):
            parse(cfg)
    cfg = copy.deepcopy(CONFIGS["A"])
    del cfg["layers"][0]["mixer"]["left"]["mask"]
    with pytest.raises(ConfigError, match="mask"):
        parse(cfg)


def test_weight_faults_are_listed_by_name(tmp_path):
    cfg = CONFIGS["A"]
    w = make_weights(cfg, 0)
    del w["l0.mix.left.r2"], w["pos"]
    w["l0.mix.right.ra"] = w["l0.mix.right.ra"][:1]
    folder = write_model(str(tmp_path / "broken"), cfg, w)
    with pytest.raises(WeightsError) as e:
        load_engine_core(folder, dtype="float32", block_size=8, num_pages=4, device="cpu", ops=TorchOps())
    assert "l0.mix.left.r2" in e.value.missing and "pos" in e.value.missing
    assert any(n == "l0.mix.right.ra" for n, _, _ in e.value.wrong_shape)
