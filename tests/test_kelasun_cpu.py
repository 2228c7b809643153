"""Kelasun through the framework's step function, cache manager and parts on the CPU with the emulated kernels, against the plain
implementation: what differs here is a fault of the host logic (tables, columns of fused products, permuted rows, results left for the
next pass), not of a kernel. Also the plain implementation's own mechanisms against direct statements of what they must do."""
import copy
import math
import os

import pytest
import torch

import plain_kelasun as P
import traces as TR
from emulated_kernels import EmulatedKernels
from kelasun_configs import KEL
from levanter_amd.cache import PagedKv
from levanter_amd.config import ConfigError, InferenceEngineConfig, KelasunConfig, LmConfig
from levanter_amd.engine import ModelRunner, StepEntry
from levanter_amd.engine.loading import load_model, make_cache
from levanter_amd.parts import BuildEnv
from levanter_amd.parts.position import rotary_frequencies
from levanter_amd.weights import WeightsError, write_random_model


def build(name, tmp, dtype=torch.float32, change=None):
    raw, seed = KEL[name]
    raw = copy.deepcopy(raw)
    W = P.random_weights(raw, seed)
    if change is not None:
        change(raw, W)
    d = P.write_folder(raw, W, os.path.join(str(tmp), name), torch.float32)
    env = BuildEnv(dtype, torch.device("cpu"), EmulatedKernels())
    config, model = load_model(d, env)
    return raw, W, model, env, config


LENGTHS = {"A": [50, 35, 70, 37], "B": [60, 45, 33], "C": [40, 12, 50], "D": [33, 50, 41]}


@pytest.fixture(scope="module", params=list(KEL))
def setup(request, tmp_path_factory):
    raw, W, model, env, _ = build(request.param, tmp_path_factory.mktemp("kel"))
    reqs = TR.random_requests(raw["vocab"], LENGTHS[request.param], 5)
    plain = {rid: P.plain_logits(W, raw, t) for rid, t in reqs.items()}
    return raw, W, model, env, reqs, plain


def replay(model, env, steps, max_tokens, ps=16, max_seqs=4):
    cfg = InferenceEngineConfig(max_pages=max(1, max_tokens // ps), max_seqs=max_seqs, page_size=ps, max_pages_per_seq=16, compute_dtype="float32")
    cache = make_cache(model, cfg)
    runner = ModelRunner(model, cache, env)
    live, out = {}, {}
    for s in steps:
        entries = []
        for e in s["entries"]:
            if e["id"] not in live:
                live[e["id"]] = cache.open(e["id"])
            entries.append(StepEntry(live[e["id"]], e["tokens"], e["want"]))
        logits = runner.step(entries)
        cache.check_invariants()
        if logits.shape[0]:
            out[s["step"]] = logits
        for rid in s["end"]:
            cache.close(live.pop(rid))
    cache.check_invariants()
    assert all(g.pool.n_free == g.pool.n_pages for g in cache.groups)
    return out, cache


@pytest.mark.parametrize("mode", ["whole", "singles", "portions", "mixed"])
def test_every_way_of_cutting_gives_the_plain_logits(setup, mode):
    raw, W, model, env, reqs, plain = setup
    steps = {"whole": TR.trace_whole, "singles": lambda r: TR.trace_prefill_then_singles(r, n_single=20), "portions": TR.trace_portions,
             "mixed": lambda r: TR.trace_mixed(r, seed=4)}[mode](reqs)
    TR.number(steps)
    got, _ = replay(model, env, steps, TR.peak_tokens(steps))
    want = TR.expected_rows(steps, lambda rid: plain[rid[1:]])
    assert set(got) == set(want)
    for k in want:
        torch.testing.assert_close(got[k].double(), want[k], rtol=2e-4, atol=2e-4)


def test_the_registry_finds_the_architecture(tmp_path):
    raw, W, model, env, config = build("A", tmp_path)
    assert isinstance(config, KelasunConfig) and config.model_type_name == "kelasun"
    assert LmConfig.from_dict(config.to_hf_config()) == config
    assert [b.kind for b in model.blocks] == ["post_norm"] * 4 and model.graph_safe
    assert [(e.layer, e.cache, e.writes_cache) for e in model.plan] == [(i, i, True) for i in range(4)]
    reqs = dict(model.cache_requirements())
    # the latent layers keep the latent and the rotated key part, whatever their heads
    assert reqs == {0: PagedKv(2, 16, None, value_dim=8), 1: PagedKv(1, 32, None, value_dim=24), 2: PagedKv(3, 8, None, value_dim=24), 3: PagedKv(1, 48, None, value_dim=32)}
    spec = config.model_spec()
    assert set(spec.all_tensors()) == set(W) and all(tuple(W[n].shape) == t.shape for n, t in spec.all_tensors().items())
    # a folder with drawn weights has the tensors of the description and loads
    write_random_model(config, 3, str(tmp_path / "drawn"), torch.float32)
    load_model(str(tmp_path / "drawn"), env)
    # defaults: key/value heads and value size of the heads and keys, no factor on the stream and the logits
    c = copy.deepcopy(raw)
    for key in ("postln_alpha", "logit_scale"):
        c.pop(key)
    for key in ("kv_heads", "vdim", "q_temp"):
        c["layers"][0]["mixer"].pop(key)
    cfg = LmConfig.from_dict(c)
    assert (cfg.postln_alpha, cfg.logit_scale) == (1.0, 1.0) and cfg.layers[0]["mixer"]["kv_heads"] == 4 and cfg.layers[0]["mixer"]["vdim"] == 16
    assert "kv_heads" not in c["layers"][0]["mixer"]  # the caller's object stays as it is


@pytest.mark.parametrize("name", ["A", "D"])
def test_the_residual_stream_after_every_layer(name, tmp_path, monkeypatch):
    import levanter_amd.parts.gated_block as G

    raw, W, model, env, _ = build(name, tmp_path)
    toks = TR.random_requests(raw["vocab"], [29], 3)["r0"]
    _, want = P.forward(toks, W, raw)
    got = []
    orig = G.PostNormBlock.forward

    def fwd(self, x, ctx, unit, wc):
        orig(self, x, ctx, unit, wc)
        assert ctx.pending is not None  # the last sublayer's sum and norm wait for the pass that reads the stream next
        ctx.settle()
        got.append(x.clone())

    monkeypatch.setattr(G.PostNormBlock, "forward", fwd)
    cache = make_cache(model, InferenceEngineConfig(max_pages=8, max_seqs=2, page_size=16, max_pages_per_seq=8, compute_dtype="float32"))
    ModelRunner(model, cache, env).step([StepEntry(cache.open("a"), toks, [])])
    assert len(got) == len(want) == len(raw["layers"])
    for g, w in zip(got, want):
        torch.testing.assert_close(g.double(), w, rtol=2e-4, atol=2e-4)


def test_pages_and_a_slot_that_are_used_again(tmp_path):
    raw, W, model, env, _ = build("A", tmp_path)
    reqs = TR.random_requests(raw["vocab"], [40, 23, 39], 2)
    steps = TR.number(TR.trace_prefill_then_singles(reqs, n_single=5))
    got, _ = replay(model, env, steps, 64, max_seqs=1)
    plain = {rid: P.plain_logits(W, raw, t) for rid, t in reqs.items()}
    want = TR.expected_rows(steps, lambda rid: plain[rid[1:]])
    for k in want:
        torch.testing.assert_close(got[k].double(), want[k], rtol=2e-4, atol=2e-4)


CHANGES = {
    "no sink": lambda raw, W: W["l0.mix.sink"].fill_(-60.0),
    "no temperature": lambda raw, W: raw["layers"][0]["mixer"].pop("q_temp"),
    "another temperature's stretch": lambda raw, W: raw["layers"][0]["mixer"]["q_temp"].update(every=17),
    "no stretched frequencies": lambda raw, W: raw["layers"][1]["mixer"]["rot"].pop("scaling"),
    "another rotation base": lambda raw, W: raw["layers"][1]["mixer"]["rot"].update(base=101.0),
    "another stream factor": lambda raw, W: raw.update(postln_alpha=1.4),
    "another logit scale": lambda raw, W: raw.update(logit_scale=0.51),
    "another score scale": lambda raw, W: raw["layers"][3]["mixer"].update(scale=0.19),
    "no head gate": lambda raw, W: W["l2.mix.g"].zero_(),
    "no element gate": lambda raw, W: W["l3.mix.g"].zero_(),
    "no shared expert": lambda raw, W: W["l0.mlp.shared.down"].zero_(),
    "fewer experts a token": lambda raw, W: raw["layers"][1]["mlp"]["router"].update(top=2),
}


@pytest.mark.parametrize("what", list(CHANGES))
def test_every_mechanism_shows_in_the_logits(what):
    """The plain implementation itself: a model without one mechanism, or with another constant, has other logits by far more than any
    tolerance of these tests, so a model that ignored it would not pass."""
    raw, seed = KEL["A"]
    raw, W = copy.deepcopy(raw), P.random_weights(raw, seed)
    toks = TR.random_requests(raw["vocab"], [40], 9)["r0"]
    want = P.plain_logits(W, raw, toks)
    CHANGES[what](raw, W)
    assert float((P.plain_logits(W, raw, toks)[20:] - want[20:]).abs().max()) > 5e-3


def test_bad_configurations_and_checkpoints_are_refused(tmp_path):
    raw, _ = KEL["A"]

    def broken(change):
        c = copy.deepcopy(raw)
        change(c)
        return c

    cases = [
        lambda c: c["layers"][0].update(type="mamba"),
        lambda c: c["layers"][0].pop("mixer"),
        lambda c: c["layers"][0]["mixer"].update(kv_heads=3),
        lambda c: c["layers"][0]["mixer"].pop("scale"),
        lambda c: c["layers"][0]["mixer"].pop("heads"),
        lambda c: c["layers"][0]["mixer"]["q_temp"].update(every=0),
        lambda c: c["layers"][0]["mixer"]["q_temp"].pop("coef"),
        lambda c: c["layers"][1]["mixer"].pop("q_rank"),
        lambda c: c["layers"][1]["mixer"].update(kv_rank=0),
        lambda c: c["layers"][1]["mixer"]["rot"].update(dims=7),
        lambda c: c["layers"][1]["mixer"]["rot"].update(dims=10),
        lambda c: c["layers"][1]["mixer"]["rot"].pop("base"),
        lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("slow"),
        lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].update(factor=0),
        lambda c: c["layers"][0]["mlp"].update(kind="dense"),
        lambda c: c["layers"][0]["mlp"]["router"].update(top=9),
        lambda c: c["layers"][0]["mlp"].pop("router"),
        lambda c: c["layers"][0]["mlp"]["expert"].pop("ff"),
        lambda c: c["layers"][0]["mlp"]["shared"].update(ff=-1),
        lambda c: c.update(postln_alpha="2"),
        lambda c: c.update(layers=[]),
        lambda c: c.pop("norm"),
        lambda c: c.pop("width"),
    ]
    for i, change in enumerate(cases):
        with pytest.raises(ConfigError):
            LmConfig.from_dict(broken(change))
            pytest.fail(f"case {i} was accepted")
    # a checkpoint that lacks a tensor, has one too many and one of the wrong shape; the second norm of a layer without a feed-forward is no fault
    W = P.random_weights(raw, 1)
    del W["l0.mix.sink"]
    W["l2.norm2"] = torch.zeros(64, dtype=torch.float64)
    W["l1.mlp.shared.up"] = torch.zeros(8, 64, dtype=torch.float64)
    W["l3.mix.dkv"] = torch.zeros(3, 64, dtype=torch.float64)
    d = P.write_folder(raw, W, str(tmp_path / "bad"), torch.float32)
    env = BuildEnv(torch.float32, torch.device("cpu"), EmulatedKernels())
    with pytest.raises(WeightsError) as e:
        load_model(d, env)
    assert e.value.missing == ["l0.mix.sink"] and e.value.unexpected == ["l1.mlp.shared.up"] and len(e.value.wrong_shape) == 1


# ---- the plain implementation's mechanisms against direct statements ------------------------------------------------------
def test_the_norm_behind_a_sum_by_hand():
    x, y = torch.tensor([[1.0, 2.0, 3.0, 6.0]], dtype=torch.float64), torch.tensor([[0.0, 0.0, 2.0, -4.0]], dtype=torch.float64)
    w = torch.tensor([1.0, 1.0, 2.0, 10.0], dtype=torch.float64)
    # 2 x + y = 2, 4, 8, 8: mean 5.5, deviations -3.5, -1.5, 2.5, 2.5, mean square (12.25 + 2.25 + 12.5) / 4 = 6.75
    r = 1 / math.sqrt(6.75 + 0.25)
    torch.testing.assert_close(P.norm_after_sum(x, y, 2.0, w, 0.25), torch.tensor([[-3.5 * r, -1.5 * r, 5.0 * r, 25.0 * r]], dtype=torch.float64))


def test_rotation_of_neighbours_and_stretched_frequencies_by_hand():
    v = torch.zeros(1, 1, 8, dtype=torch.float64)
    v[0, 0, 2], v[0, 0, 7] = 1.0, 2.0  # dimension 2 is paired with dimension 3; dimensions 6 and 7 never turn
    f = P.stretched_frequencies(6, 100.0, None)
    out = P.rotate_pairs(v, torch.tensor([3]), f, 1.25)
    a = 3 * 100.0 ** (-2 / 6)
    want = torch.zeros(8, dtype=torch.float64)
    want[2], want[3], want[7] = 1.25 * math.cos(a), 1.25 * math.sin(a), 2.0
    torch.testing.assert_close(out[0, 0], want)
    # a base of e^4 over 8 dimensions: pair i turns e^-i radians a position. One turn over 2 pi e^2 positions is pair 2's rate, a turn more
    # than e times that is below pair 1: pairs 0 and 1 keep their rate, pair 2 is halfway, pair 3 turns four times slower
    sc = {"factor": 4.0, "original": 2 * math.pi * math.exp(2), "fast": math.exp(0.9), "slow": math.exp(-0.5)}
    got = P.stretched_frequencies(8, math.exp(4), sc)  # index(fast) = 1.1 -> lo 1, index(slow) = 2.5 -> hi 3
    want = [1.0, math.exp(-1), math.exp(-2) * (0.5 + 0.5 / 4), math.exp(-3) / 4]
    torch.testing.assert_close(torch.tensor(got), torch.tensor(want))
    torch.testing.assert_close(torch.tensor(rotary_frequencies(8, math.exp(4), sc)), torch.tensor(want))
    assert abs(P.rotation_magnitude(sc) - (1 + 0.1 * math.log(4))) < 1e-15 and P.rotation_magnitude(None) == 1.0


def test_the_queries_temperature_by_hand():
    t = P.temperature(torch.tensor([0, 2, 3, 6, 7, 31]), {"coef": 0.5, "every": 4})
    want = [1.0, 1.0, 1 + 0.5 * math.log(2), 1 + 0.5 * math.log(2), 1 + 0.5 * math.log(3), 1 + 0.5 * math.log(9)]
    torch.testing.assert_close(t, torch.tensor(want, dtype=torch.float64))
    assert P.temperature(torch.tensor([5, 9]), None).tolist() == [1.0, 1.0]


def test_a_sinks_share_and_the_distance_term():
    """Equal scores of s: a query at position i gives the key at distance d the share 2^-d / (sum + exp(sink - s)) under a slope of ln 2."""
    q = k = torch.ones(3, 1, 1, dtype=torch.float64)
    o = P.sink_attention(q, k, torch.eye(3, dtype=torch.float64).view(3, 1, 3), 2.0, [math.log(2.0)], torch.tensor([2.0 + math.log(3.0)], dtype=torch.float64))
    torch.testing.assert_close(o[:, 0], torch.tensor([[1 / 4, 0, 0], [0.5 / 4.5, 1 / 4.5, 0], [0.25 / 4.75, 0.5 / 4.75, 1 / 4.75]], dtype=torch.float64))
    far = P.sink_attention(q, k, torch.ones(3, 1, 1, dtype=torch.float64), 1.0, [0.0], torch.tensor([700.0], dtype=torch.float64))
    assert float(far.max()) < 1e-200 and torch.isfinite(far).all()
    assert P.distance_slopes(4) == [0.25, 0.0625, 2.0 ** -6, 2.0 ** -8] and P.distance_slopes(16)[0] == 2.0 ** -0.5


def test_the_routers_weights_are_a_softmax_over_the_chosen_alone():
    z = torch.tensor([[3.0, -1.0, 3.0 + math.log(2.0), 0.0], [900.0, 0.0, 0.0, 899.0]], dtype=torch.float64)
    chosen, w = P.route(z, 2)
    assert chosen.tolist() == [[2, 0], [0, 3]]
    torch.testing.assert_close(w, torch.tensor([[2 / 3, 1 / 3], [1 / (1 + math.exp(-1)), 1 / (1 + math.e)]], dtype=torch.float64))
    assert P.squared_relu(torch.tensor([-3.0, 0.0, 3.0])).tolist() == [0.0, 0.0, 9.0]
