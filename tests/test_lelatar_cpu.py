"""Lelatar through the framework's step function, cache manager and parts on the CPU with the emulated kernels, against the plain
implementation: what differs here is a fault of the host logic (tables, state slots, the loop's passes and their cache units, columns of
fused products), not of a kernel. Also the plain implementation's own mechanisms against direct statements of what they must do."""
import copy
import math
import os

import pytest
import torch

import plain_lelatar as P
import traces as TR
from emulated_kernels import EmulatedKernels
from lelatar_configs import LEL
from levanter_amd.cache import PagedKv, SlotState
from levanter_amd.config import ConfigError, InferenceEngineConfig, LelatarConfig, LmConfig
from levanter_amd.engine import ModelRunner, StepEntry
from levanter_amd.engine.loading import load_model, make_cache
from levanter_amd.parts import BuildEnv
from levanter_amd.parts.position import rotary_frequencies
from levanter_amd.weights import WeightsError, write_random_model


def build(name, tmp, dtype=torch.float32):
    raw, seed = LEL[name]
    W = P.random_weights(raw, seed)
    d = P.write_folder(raw, W, os.path.join(str(tmp), name), torch.float32)
    env = BuildEnv(dtype, torch.device("cpu"), EmulatedKernels())
    config, model = load_model(d, env)
    return raw, W, model, env, config


def close(got: torch.Tensor, want: torch.Tensor) -> None:
    """Equal to 2e-4, but for one element in a hundred ten times that: a recurrence whose head norm divides a sum that nearly cancels (a
    request's first tokens, a single written value) multiplies the 32-bit sum's last bits."""
    torch.testing.assert_close(got, want, rtol=2e-3, atol=2e-3)
    bad = ((got - want).abs() > 2e-4 + 2e-4 * want.abs()).double().mean()
    assert float(bad) <= 0.01, f"{float(bad):.3%} of the elements differ by more than 2e-4"


LENGTHS = {"A": [50, 35, 70, 37], "B": [60, 45, 33], "C": [40, 12, 50], "D": [33, 50, 21]}


@pytest.fixture(scope="module", params=list(LEL))
def setup(request, tmp_path_factory):
    raw, W, model, env, _ = build(request.param, tmp_path_factory.mktemp("lel"))
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
        close(got[k].double(), want[k])


def test_the_registry_finds_the_architecture_and_every_pass_of_the_loop_has_a_cache_unit(tmp_path):
    raw, W, model, env, config = build("A", tmp_path)
    assert isinstance(config, LelatarConfig) and config.model_type_name == "lelatar"
    assert LmConfig.from_dict(config.to_hf_config()) == config
    assert [b.kind for b in model.blocks] == ["pre_norm"] * 4
    # layers 1 and 2 run twice; the loop's entry stands before the first layer of each pass
    assert [(e.layer, e.cache, e.writes_cache, e.enters) for e in model.plan] == [
        (0, 0, True, None), (1, 1, True, (0, 0)), (2, 2, True, None), (1, 3, True, (0, 1)), (2, 4, True, None), (3, 5, True, None)]
    reqs = dict(model.cache_requirements())
    conv = 2 * 2 * 16 + 4 * 8  # channels of q, k and v
    assert reqs[0].paged() == PagedKv(2, 16, None, value_dim=8) and reqs[0].slot_state() == SlotState((4 * conv + 4 * 16 * 8,), "float32")
    assert reqs[1] == reqs[3] == SlotState((3 * (4 * 16 + 2 * 2 * 12) + 4 * 12 * 16,), "float32")
    assert reqs[2].paged() == reqs[4].paged() == PagedKv(1, 24, None)
    assert reqs[5] == SlotState((4 * (6 * 8 + 2 * 3 * 16) + 6 * 16 * 8,), "float32")
    spec = config.model_spec()
    assert set(spec.all_tensors()) == set(W) and all(tuple(W[n].shape) == t.shape for n, t in spec.all_tensors().items())
    # every layer's part of the second table is a stretch of its rows
    for i, b in enumerate(model.blocks):
        torch.testing.assert_close(b.token_input.table.double(), W["side.embed"][:, 8 * i:8 * i + 8])
    # a model without a loop and a second table has neither parts nor tensors of them
    raw_b, W_b, model_b, _, config_b = build("B", tmp_path)
    assert model_b.stream_entries == [] and all(b.token_input is None for b in model_b.blocks) and all(e.enters is None for e in model_b.plan)
    assert "loop" not in config_b.to_hf_config() and set(config_b.model_spec().all_tensors()) == set(W_b)
    # a folder with drawn weights has the tensors of the description and loads
    d = write_random_model(config, 3, str(tmp_path / "drawn"), torch.float32) or str(tmp_path / "drawn")
    load_model(str(tmp_path / "drawn"), env)


@pytest.mark.parametrize("name", ["A", "C"])
def test_the_residual_stream_after_every_layer(name, tmp_path, monkeypatch):
    import levanter_amd.parts.block as B

    raw, W, model, env, _ = build(name, tmp_path)
    toks = TR.random_requests(raw["vocab"], [29], 3)["r0"]
    _, want = P.forward(toks, W, raw)
    got = []
    orig = B.PreNormBlock.forward

    def fwd(self, x, ctx, unit, wc):
        orig(self, x, ctx, unit, wc)
        assert ctx.pending is not None  # the token input's write waits for the pass that reads the stream next
        ctx.settle()
        got.append(x.clone())

    monkeypatch.setattr(B.PreNormBlock, "forward", fwd)
    cache = make_cache(model, InferenceEngineConfig(max_pages=8, max_seqs=2, page_size=16, max_pages_per_seq=8, compute_dtype="float32"))
    ModelRunner(model, cache, env).step([StepEntry(cache.open("a"), toks, [])])
    assert len(got) == len(want) == 6
    for g, w in zip(got, want):
        close(g.double(), w)


def test_a_slot_that_is_used_again_starts_from_zero_state(tmp_path):
    """Two requests one after the other in an engine of one slot: the second finds the first one's states, inputs and pages."""
    raw, W, model, env, _ = build("A", tmp_path)
    reqs = TR.random_requests(raw["vocab"], [40, 23], 2)
    steps = TR.number(TR.trace_prefill_then_singles(reqs, n_single=5))
    got, _ = replay(model, env, steps, 64, max_seqs=1)
    plain = {rid: P.plain_logits(W, raw, t) for rid, t in reqs.items()}
    want = TR.expected_rows(steps, lambda rid: plain[rid[1:]])
    for k in want:
        close(got[k].double(), want[k])


def test_bad_configurations_and_checkpoints_are_refused(tmp_path):
    raw, _ = LEL["A"]

    def broken(change):
        c = copy.deepcopy(raw)
        change(c)
        return c

    cases = [
        lambda c: c["layers"][0].update(type="attention"),
        lambda c: c["layers"][0]["mixer"].pop("right"),
        lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3),
        lambda c: c["layers"][0]["mixer"]["right"].update(kv_heads=3),
        lambda c: c["layers"][0]["mixer"]["right"].pop("conv"),
        lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=7),
        lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=18),
        lambda c: c["layers"][0]["mixer"]["left"]["rot"].pop("base"),
        lambda c: c["layers"][0]["mixer"]["left"].pop("scale"),
        lambda c: c["layers"][1]["mixer"].update(groups=3),
        lambda c: c["layers"][1]["mixer"].update(norm_groups=5),
        lambda c: c["layers"][1]["mixer"].update(conv=0),
        lambda c: c["layers"][1]["mixer"].pop("state"),
        lambda c: c["layers"][0]["mlp"].update(kind="moe"),
        lambda c: c["loop"].update(stop=5),
        lambda c: c["loop"].update(start=3),
        lambda c: c["loop"].update(start=-1),
        lambda c: c["loop"].update(times=0),
        lambda c: c["token_side"].update(dim=0),
        lambda c: c.pop("norm"),
        lambda c: c.pop("width"),
    ]
    for i, change in enumerate(cases):
        with pytest.raises(ConfigError):
            LmConfig.from_dict(broken(change))
            pytest.fail(f"case {i} was accepted")
    # a checkpoint that lacks a tensor, has one too many and one of the wrong shape
    W = P.random_weights(raw, 1)
    del W["l0.mix.right.dt_bias"]
    W["l1.mlp.gate"] = torch.zeros(8, 64, dtype=torch.float64)
    W["loop.step"] = torch.zeros(3, 64, dtype=torch.float64)
    d = P.write_folder(raw, W, str(tmp_path / "bad"), torch.float32)
    env = BuildEnv(torch.float32, torch.device("cpu"), EmulatedKernels())
    with pytest.raises(WeightsError) as e:
        load_model(d, env)
    assert e.value.missing == ["l0.mix.right.dt_bias"] and e.value.unexpected == ["l1.mlp.gate"] and len(e.value.wrong_shape) == 1
    # heads larger than the kernels take are refused when the model is built
    big = P.make_config(vocab=20, width=16, loop=None, side=None, layers=[P.mamba_layer(heads=1, vdim=8, state=300, groups=1, norm_groups=1)])
    d = P.write_folder(big, P.random_weights(big, 1), str(tmp_path / "big"), torch.float32)
    with pytest.raises(ValueError, match="at most 256"):
        load_model(d, env)


# ---- the plain implementation's mechanisms against direct statements ------------------------------------------------------
def test_the_convolution_by_hand():
    x = torch.tensor([[1.0, 10.0], [2.0, 20.0], [4.0, 40.0]], dtype=torch.float64)
    taps = torch.tensor([[100.0, 10.0, 1.0], [0.0, 0.5, 2.0]], dtype=torch.float64)  # the last column is the current token's
    out = P.causal_conv(x, taps, torch.tensor([0.0, 1.0], dtype=torch.float64))
    assert out.tolist() == [[1.0, 21.0], [2.0 + 10.0, 40.0 + 5.0 + 1.0], [4.0 + 20.0 + 100.0, 80.0 + 10.0 + 1.0]]
    assert P.causal_conv(x, taps[:, 2:]).tolist() == [[1.0, 20.0], [2.0, 40.0], [4.0, 80.0]]


def test_rotation_of_halves_by_hand():
    v = torch.zeros(1, 1, 8, dtype=torch.float64)
    v[0, 0, 1], v[0, 0, 7] = 1.0, 2.0  # dimension 1 is paired with dimension 4 of 6; dimensions 6 and 7 never turn
    out = P.rotate_half(v, torch.tensor([3]), 6, 100.0)
    a = 3 * 100.0 ** (-2 / 6)
    want = torch.zeros(8, dtype=torch.float64)
    want[1], want[4], want[7] = math.cos(a), math.sin(a), 2.0
    torch.testing.assert_close(out[0, 0], want)
    q, k = torch.randn(2, 1, 1, 8, dtype=torch.float64)  # scores depend on the distance alone
    s = [float((P.rotate_half(q, torch.tensor([p + 5]), 8, 50.0) * P.rotate_half(k, torch.tensor([p]), 8, 50.0)).sum()) for p in (0, 7, 300)]
    assert abs(s[0] - s[1]) < 1e-9 and abs(s[0] - s[2]) < 1e-9
    torch.testing.assert_close(torch.tensor(rotary_frequencies(6, 100.0), dtype=torch.float64), torch.tensor([100.0 ** (-2 * i / 6) for i in range(3)], dtype=torch.float64))


def test_a_sinks_share():
    """Equal scores of s: a query at position i gives every key 1 / (i + 1 + exp(sink - s))."""
    q = k = torch.ones(3, 1, 1, dtype=torch.float64)
    o = P.sink_attention(q, k, torch.eye(3, dtype=torch.float64).view(3, 1, 3), 2.0, torch.tensor([2.0 + math.log(3.0)], dtype=torch.float64))
    torch.testing.assert_close(o[:, 0], torch.tensor([[1 / 4, 0, 0], [1 / 5, 1 / 5, 0], [1 / 6] * 3], dtype=torch.float64))
    far = P.sink_attention(q, k, torch.ones(3, 1, 1, dtype=torch.float64), 1.0, torch.tensor([700.0], dtype=torch.float64))
    assert float(far.max()) < 1e-200 and torch.isfinite(far).all()


def test_two_steps_of_the_state_space_recurrence_written_out():
    """One head with two state rows and one value; a carried state equals one run; heads read their own group."""
    x, B, C = (torch.tensor(v, dtype=torch.float64) for v in ([[[3.0]], [[2.0]]], [[[1.0, 2.0]], [[0.5, -1.0]]], [[[1.0, 1.0]], [[2.0, 1.0]]]))
    dt, A, D = torch.tensor([[0.5], [0.25]], dtype=torch.float64), torch.tensor([2.0], dtype=torch.float64), torch.tensor([0.1], dtype=torch.float64)
    y, S = P.ssd_scan(x, B, C, dt, A, D)
    S1 = [0.5 * 1.0 * 3.0, 0.5 * 2.0 * 3.0]
    S2 = [math.exp(-0.5) * S1[0] + 0.25 * 0.5 * 2.0, math.exp(-0.5) * S1[1] - 0.25 * 2.0]
    torch.testing.assert_close(S[0, :, 0], torch.tensor(S2, dtype=torch.float64))
    torch.testing.assert_close(y[:, 0, 0], torch.tensor([S1[0] + S1[1] + 0.3, 2 * S2[0] + S2[1] + 0.2], dtype=torch.float64))
    g = torch.Generator().manual_seed(0)
    x, B, C = torch.randn(5, 4, 3, generator=g).double(), torch.randn(5, 2, 6, generator=g).double(), torch.randn(5, 2, 6, generator=g).double()
    dt, A, D = torch.rand(5, 4, generator=g).double(), torch.rand(4, generator=g).double(), torch.rand(4, generator=g).double()
    y, S = P.ssd_scan(x, B, C, dt, A, D)
    y1, S1 = P.ssd_scan(x[:2], B[:2], C[:2], dt[:2], A, D)
    y2, S2 = P.ssd_scan(x[2:], B[2:], C[2:], dt[2:], A, D, S1)
    torch.testing.assert_close(torch.cat([y1, y2]), y)
    torch.testing.assert_close(S2, S)
    y3, _ = P.ssd_scan(x[:, 3:], B[:, 1:], C[:, 1:], dt[:, 3:], A[3:], D[3:])  # the last of four heads reads the second of two groups
    torch.testing.assert_close(y3[:, 0], y[:, 3])


def test_two_steps_of_the_delta_rule_written_out():
    """A second write along the same unit key with a write rate of one replaces what the first wrote; the read-out sees it."""
    k = torch.tensor([[[1.0, 0.0]], [[1.0, 0.0]]], dtype=torch.float64)
    q = torch.tensor([[[2.0, 5.0]], [[2.0, 5.0]]], dtype=torch.float64)
    v = torch.tensor([[[3.0]], [[7.0]]], dtype=torch.float64)
    one = torch.ones(2, 1, dtype=torch.float64)
    o, S = P.delta_scan(q, k, v, one, one)
    assert o[:, 0, 0].tolist() == [6.0, 14.0] and S[0, :, 0].tolist() == [7.0, 0.0]
    o, S = P.delta_scan(q, k, v, one * 0.5, one * 0.25)  # S1 = 0.75; then 0.375 + 0.25 (7 - 0.375)
    assert o[:, 0, 0].tolist() == [1.5, 2 * (0.375 + 0.25 * 6.625)] and abs(float(S[0, 0, 0]) - 2.03125) < 1e-12
    torch.testing.assert_close(P.unit(torch.tensor([[3.0, 4.0]], dtype=torch.float64)), torch.tensor([[0.6, 0.8]], dtype=torch.float64), rtol=1e-6, atol=0)


def test_where_the_loops_passes_begin():
    cfg = {"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}
    assert P.layer_order(cfg) == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (3, None)]
    assert P.layer_order({"layers": [0] * 2, "loop": {"start": 0, "stop": 2, "times": 1}}) == [(0, 0), (1, None)]
    assert P.layer_order({"layers": [0] * 2}) == [(0, None), (1, None)]
    x, x0 = torch.tensor([[1.0, 2.0]], dtype=torch.float64), torch.tensor([[10.0, 20.0]], dtype=torch.float64)
    W = {"loop.in": torch.tensor([[1.0, 0, 0, 1.0], [0, 1.0, 1.0, 0]], dtype=torch.float64), "loop.step": torch.tensor([[0.0, 0], [100.0, 200.0]], dtype=torch.float64)}
    assert P.loop_entry(x, x0, W, 1).tolist() == [[1 + 20 + 100.0, 2 + 10 + 200.0]]
