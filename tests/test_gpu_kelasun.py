"""Kelasun on the GPU: every kernel it brought or extended against the plain function of its mechanism, its two mixers as parts, whole
models through ``bin/trace_run`` in every cutting, generation through the engine and the command line."""
import copy
import math
import os

import pytest
import torch

import plain_kelasun as P
import traces as TR
from helpers import make_meta, random_block_tables
from kelasun_configs import KEL

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


def K():
    from levanter_amd.kernels import get_kernels

    return get_kernels()


def tol(dtype, f32=2e-5, bf16=2e-2):
    return dict(rtol=f32, atol=f32) if dtype == torch.float32 else dict(rtol=bf16, atol=bf16)


def bfn(x):
    """Numbers that bfloat16 holds exactly, as float64."""
    return x.to(torch.bfloat16).double()


def dev(x, dtype=torch.float32):
    return x.to(dtype).to(DEV)


def ints(x):
    return torch.tensor(x, dtype=torch.int32, device=DEV)


# ---- the norm behind a sum -------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,D,top", [(7, 64, 2), (33, 30, 1), (3, 257, 5), (2, 1000, 4), (1, 8, 3), (5, 4096, 2), (4, 1, 1), (3, 9001, 2), (2, 16384, 3), (65, 2048, 4)])
def test_the_norm_behind_a_sum(dtype, T, D, top):
    from levanter_amd.kernels.library import PendingExperts

    kern = K()
    g = torch.Generator().manual_seed(D + top)
    x0, y = torch.randn(T, D, generator=g) * 2 + 0.5, torch.randn(T, D, generator=g) * 3
    w, b, w2, b2 = (m + 0.3 * torch.randn(D, generator=g) for m in (1.0, 0.0, 1.0, 0.0))
    eo, wt = torch.randn(T * top, D, generator=g), torch.rand(T, top, generator=g)
    pos = torch.randperm(T * top, generator=g).to(torch.int32)
    experts = PendingExperts(dev(eo), pos.to(DEV), dev(wt), False)
    eps, alpha = 1e-3, 1.7
    summed = (wt.double()[:, :, None] * eo.double()[pos.long()].view(T, top, D)).sum(1)
    x64, y64, w64, b64 = x0.double(), y.double(), w.double(), b.double()
    cases = [
        (dict(y=dev(y), write_norm=(dev(w), None, eps, False)), P.norm_after_sum(x64, y64, alpha, w64, eps)),
        (dict(y=dev(y), experts=experts, write_norm=(dev(w), dev(b), eps, False)), P.norm_after_sum(x64, y64 + summed, alpha, w64, eps) + b64),
        (dict(experts=experts, write_norm=(dev(w), None, eps, True)), P.rms_norm(alpha * x64 + summed, w64, eps)),
        (dict(write_norm=(dev(w), dev(b), eps, True)), P.rms_norm(alpha * x64, w64, eps) + b64),
    ]
    limit = 2e-5 if D > 1 else 2e-4
    for args, want in cases:
        x, h = dev(x0), torch.full((T, D), float("nan"), dtype=dtype, device=DEV)
        pending = kern.sum_norm_step(x, alpha=alpha, defer=True, **args)
        assert torch.equal(x.cpu(), x0)  # nothing has run
        kern.sum_norm_step(x, pending=pending, h_out=h)
        torch.testing.assert_close(x.cpu().double(), want, rtol=limit, atol=limit)
        assert torch.equal(h, x.to(dtype))
        again = dev(x0)
        kern.finish(kern.sum_norm_step(again, alpha=alpha, defer=True, **args))  # the write by itself leaves the same bits
        assert torch.equal(again, x)
        # chosen rows, one of them twice, through the second norm (what stands ahead of the head): nothing is stored
        rows = ints([T - 1, 0, T - 1])
        again = dev(x0)
        out = torch.full((3, D), float("nan"), dtype=dtype, device=DEV)
        kern.norm(again, dev(w2), dev(b2), 1e-5, out, rows=rows, pending=kern.sum_norm_step(again, alpha=alpha, defer=True, **args))
        want2 = P.layer_norm(want, w2.double(), 1e-5) + b2.double()
        if D > 1:  # (a layer norm of one number is the bias)
            torch.testing.assert_close(out.cpu().double(), want2[rows.cpu().long()], **tol(dtype, f32=1e-4))
        assert torch.equal(again.cpu(), x0)
    # the read alone: as it is, and normed
    x, h = dev(x0), torch.empty(T, D, dtype=dtype, device=DEV)
    kern.sum_norm_step(x, h_out=h)
    assert torch.equal(h, x.to(dtype)) and torch.equal(x.cpu(), x0)
    kern.sum_norm_step(x, norm=(dev(w2), None, 1e-5, True), h_out=h)
    torch.testing.assert_close(h.cpu().double(), P.rms_norm(x64, w2.double(), 1e-5), **tol(dtype))


@pytest.mark.parametrize("M,N,Kd,bias", [(3, 512, 4096, True), (16, 512, 4096, False), (40, 264, 1024, True)])
def test_the_norm_behind_a_sum_adds_up_a_product_that_has_left_its_ranges(M, N, Kd, bias):
    kern = K()
    g = torch.Generator().manual_seed(N)
    a, w = dev(torch.randn(M, Kd, generator=g), torch.bfloat16), dev(torch.randn(N, Kd, generator=g) / math.sqrt(Kd), torch.bfloat16)
    lin_bias = dev(torch.randn(N, generator=g)) if bias else None
    x0, nw = torch.randn(M, N, generator=g), dev(1 + 0.1 * torch.randn(N, generator=g))
    outs = []
    for fold in (True, False):
        x, y, h = dev(x0), torch.full((M, N), float("nan"), device=DEV), torch.empty(M, N, dtype=torch.bfloat16, device=DEV)
        product = kern.linear(a, w, lin_bias, y, may_leave_pending=True)
        if product is None:
            pytest.skip("this shape's product does not split its sum")
        if not fold:
            kern.finish(product)
        args = dict(product=product) if fold else dict(y=y)
        kern.sum_norm_step(x, pending=kern.sum_norm_step(x, alpha=0.5, write_norm=(nw, None, 1e-5, False), defer=True, **args), h_out=h)
        outs.append((x.cpu(), h.cpu()))
    torch.testing.assert_close(outs[0][0], outs[1][0], rtol=2e-6, atol=2e-6)
    want = P.norm_after_sum(x0.double(), a.cpu().double() @ w.cpu().double().T + (lin_bias.cpu().double() if bias else 0), 0.5, nw.cpu().double(), 1e-5)
    torch.testing.assert_close(outs[0][0].double(), want, rtol=2e-5, atol=2e-5)


def test_large_means_do_not_cost_the_digits_of_the_deviations():
    """A row whose numbers share a mean a thousand times their spread: the deviations are taken before they are squared."""
    g = torch.Generator().manual_seed(1)
    x0 = (torch.randn(4, 512, generator=g) + 1000.0).float()
    x, w = dev(x0), torch.ones(512, device=DEV)
    K().sum_norm_step(x, pending=K().sum_norm_step(x, alpha=1.0, write_norm=(w, None, 1e-5, False), defer=True))
    torch.testing.assert_close(x.cpu().double(), P.layer_norm(x0.double(), torch.ones(512, dtype=torch.float64), 1e-5), rtol=1e-3, atol=1e-3)


# ---- row kernels of the two attentions -------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,hd,true,vd,pairs,temp", [(4, 2, 16, 16, 8, 0, (0.7, 5)), (3, 1, 32, 20, 32, 0, (0.3, 64)), (2, 2, 16, 16, 16, 8, (0.5, 1)), (6, 3, 8, 8, 16, 0, (-0.2, 256)),
                                                        (16, 4, 128, 128, 64, 0, (0.4, 2048)), (2, 1, 16, 12, 8, 3, (0.9, 3.5))])
def test_norm_over_the_projection_with_a_temperature_of_the_position(dtype, H, G, hd, true, vd, pairs, temp):
    """Queries just below, at and above the positions where the temperature steps; keys have none; the write into pages in the same kernel
    leaves the same bits; neighbours may turn in the same kernel."""
    g = torch.Generator().manual_seed(hd + vd + H)
    every = temp[1]
    pos = sorted({0, 1, 2, 15, 16, 4000, *(int(math.ceil(n * every)) + d for n in (1, 2, 7) for d in (-2, -1, 0) if n * every + d >= 0)})
    T, ps, eps = len(pos), 16, 1e-5
    q, k = (bfn(torch.randn(T, n, hd, generator=g) * 2) for n in (H, G))
    for t in (q, k):
        t[:, :, true:] = 0.0
    wq, wk = 1.5 + torch.randn(H, hd, generator=g).double() * 0.3, 1.5 + torch.randn(G, hd, generator=g).double() * 0.3
    v = torch.randn(T, G * vd, generator=g).to(dtype).to(DEV)
    dest = ints([int(d) for d in torch.randperm(8 * ps, generator=g)[:T]])
    freqs = [300.0 ** (-i / max(pairs, 1)) for i in range(pairs)]
    p64 = torch.tensor(pos)

    def plain(x, w, heads, factor):
        y = P.rms_norm(x[:, :, :true].reshape(T, -1), w[:, :true].reshape(-1), eps) * factor[:, None]
        return P.rotate_pairs(y.view(T, heads, true), p64, freqs)

    factor = P.temperature(p64, {"coef": temp[0], "every": every})
    assert len(set(factor.tolist())) >= 3
    args = dict(q_norm_dim=H * true, k_norm_dim=G * true, positions=ints(pos), temperature=temp, **({"freqs": dev(torch.tensor(freqs))} if pairs else {}))
    q1, k1 = dev(q.reshape(T, -1), dtype), dev(k.reshape(T, -1), dtype)
    K().projection_norm_rotate(q1, k1, H, G, hd, eps, dev(wq.reshape(-1)), dev(wk.reshape(-1)), **args)
    t = tol(dtype, f32=2e-3 if pairs else 2e-5)  # angles are 32-bit: at position 4,000 known to 4000 * 2^-24
    torch.testing.assert_close(q1.cpu().double().view(T, H, hd)[:, :, :true], plain(q, wq, H, factor), **t)
    torch.testing.assert_close(k1.cpu().double().view(T, G, hd)[:, :, :true], plain(k, wk, G, torch.ones(T, dtype=torch.float64)), **t)
    kp1, vp1 = torch.zeros(8, G * hd * ps, dtype=dtype, device=DEV), torch.zeros(8, G * vd * ps, dtype=dtype, device=DEV)
    kp2, vp2 = torch.zeros_like(kp1), torch.zeros_like(vp1)
    K().kv_write(k1, v, kp1, vp1, dest, G, hd, ps, value_dim=vd)
    q2, k2 = dev(q.reshape(T, -1), dtype), dev(k.reshape(T, -1), dtype)
    K().projection_norm_rotate(q2, k2, H, G, hd, eps, dev(wq.reshape(-1)), dev(wk.reshape(-1)), v=v, value_dim=vd, k_pages=kp2, v_pages=vp2, dest=dest, page_size=ps, **args)
    assert torch.equal(q1, q2) and torch.equal(kp1, kp2) and torch.equal(vp1, vp2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R,true_R,DR,dims,H,dk", [(32, 20, 16, 4, 3, 12), (16, 16, 16, 16, 1, 8), (64, 64, 48, 32, 5, 40), (224, 224, 32, 32, 16, 64)])
def test_a_rotation_that_grows_is_the_same_bits_alone_and_in_the_kernel_that_writes_the_latent(dtype, R, true_R, DR, dims, H, dk):
    g = torch.Generator().manual_seed(R + DR)
    T, ps, n_pages, mag = 7, 16, 12, 1.2079
    KD, qh = R + DR, dk + DR
    kv0, q0 = torch.randn(T, KD + 16, generator=g), torch.randn(T, H * qh, generator=g)
    kv0[:, 8 + true_R:8 + R] = 0
    w = torch.cat([1 + 0.2 * torch.randn(true_R, generator=g), torch.zeros(R - true_R)]).to(DEV)
    f = torch.tensor(P.stretched_frequencies(dims, 77.0, {"factor": 8.0, "original": 300, "fast": 9.0, "slow": 0.7}), dtype=torch.float32, device=DEV)
    positions, dest = ints([0, 5, 130, 4000, 17, 1, 64]), ints([3 * ps + 1, 0, 11 * ps + 15, -1, 5 * ps + 7, 5 * ps + 8, 2 * ps])
    outs = []
    for fused in (True, False):
        kv, q = dev(kv0, dtype)[:, 8:8 + KD], dev(q0, dtype)
        kp, vp = torch.zeros(n_pages, KD * ps, dtype=dtype, device=DEV), torch.zeros(n_pages, R * ps, dtype=dtype, device=DEV)
        if fused:
            K().latent_rope_write(kv, R, w, 1e-5, true_R, q, H, qh, dk, f, positions, kp, vp, dest, ps, magnitude=mag)
        else:
            K().rotary_half(q, H, qh, dk, f, positions, magnitude=mag)
            K().rotary_half(kv, 1, KD, R, f, positions, magnitude=mag)
            K().head_prepare(kv[:, :R], 1, R, 1e-5, norm_dim=true_R, norm_weight=w)
            K().kv_write(kv, kv[:, :R], kp, vp, dest, 1, KD, ps, value_dim=R)
        outs.append((kv.clone(), q, kp, vp))
    for a, b in zip(*outs):
        assert torch.equal(a, b)
    # halves side by side are neighbours in another order
    n = dims // 2
    order = [*range(0, dims, 2), *range(1, dims, 2), *range(dims, DR)]
    back = [order.index(i) for i in range(DR)]
    src = q0.to(dtype).double().view(T, H, qh)[:, :, dk:][..., back]
    want = P.rotate_pairs(src, positions.cpu(), [float(x) for x in f.cpu()], mag)
    torch.testing.assert_close(outs[0][1].cpu().double().view(T, H, qh)[:, :, dk:][..., back], want, **tol(dtype, f32=2e-3))
    assert n == len(f)


@pytest.mark.parametrize("dtype,mfma", [(torch.float32, True), (torch.bfloat16, True), (torch.bfloat16, False)])
@pytest.mark.parametrize("T,B,n_in,n_out", [(1, 3, 24, 8), (5, 4, 64, 48), (33, 2, 20, 10), (200, 3, 128, 64), (130, 1, 8, 24)])
def test_products_per_head_with_a_gate_per_element(dtype, mfma, T, B, n_in, n_out, monkeypatch):
    monkeypatch.setattr(K(), "use_mfma", mfma)
    g = torch.Generator().manual_seed(T + n_in)
    a, w = bfn(torch.randn(T, B * n_in, generator=g)), bfn(torch.randn(B, n_out, n_in, generator=g) / math.sqrt(n_in))
    wide = bfn(torch.randn(T, B * n_out + 16, generator=g) * 2)
    gate = wide[:, 8:8 + B * n_out]
    want = torch.cat([a[:, b * n_in:(b + 1) * n_in] @ w[b].T for b in range(B)], 1) * torch.sigmoid(gate)
    for a_dtype in {dtype, torch.float32}:
        out = torch.full((T, B * n_out), float("nan"), dtype=dtype, device=DEV)
        K().block_linear(dev(a, a_dtype), dev(w, dtype), None, out, gate=dev(wide, dtype)[:, 8:8 + B * n_out])
        torch.testing.assert_close(out.cpu().double(), want, **tol(dtype))


# ---- experts -----------------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("T,E,top", [(37, 8, 2), (5, 18, 4), (64, 12, 1), (3, 6, 6), (200, 64, 8), (9, 1, 1), (11, 300, 32)])
def test_the_router_that_weights_by_a_softmax_over_the_chosen(T, E, top):
    g = torch.Generator().manual_seed(E * top)
    z = torch.randn(T, E + 3, generator=g) * 3
    z[0] *= 100.0  # logits of several hundred: a softmax over all of them would leave the others nothing
    z[1, :E] = 0.25  # equal logits: the lower index first, equal weights
    chosen, weights = torch.empty(T, top, dtype=torch.int32, device=DEV), torch.empty(T, top, device=DEV)
    K().moe_route(dev(z)[:, :E], None, chosen, weights, scoring="softmax_chosen")
    want_c, want_w = P.route(z[:, :E].double(), top)
    want_c[1] = torch.arange(top)
    assert torch.equal(chosen.cpu().long(), want_c)
    torch.testing.assert_close(weights.cpu().double(), want_w, rtol=2e-5, atol=1e-6)


@pytest.mark.parametrize("T,E,G,keep,top,scoring,extra", [(1, 8, 1, 1, 2, "softmax_chosen", True), (16, 32, 1, 1, 4, "softmax_chosen", True), (7, 18, 3, 2, 4, "sigmoid", False),
                                                           (13, 256, 64, 5, 8, "softmax", False), (5, 12, 6, 6, 12, "sigmoid", True), (17, 8, 1, 1, 2, "softmax_chosen", True),
                                                           (9, 300, 1, 1, 3, "softmax", True), (200, 1024, 1, 1, 32, "softmax_chosen", True), (3, 1, 1, 1, 1, "softmax_chosen", True)])
def test_routing_and_sorting_in_one_kernel(T, E, G, keep, top, scoring, extra):
    """The choices and weights of the routing kernel, bit for bit, with one choice more if asked for; every pair has one place, experts lie
    in rising order, and the tiles cover them (also beyond the sizes of the one kernel, where two run)."""
    kern = K()
    g = torch.Generator().manual_seed(E + T)
    z, corr = dev(torch.randn(T, E, generator=g) * 2), dev(torch.randn(E, generator=g) * 0.1)
    n, cols = E + int(extra), top + int(extra)
    Pn = T * cols
    rows = kern.moe_tile_rows(Pn, n)
    want_c, want_w = torch.empty(T, top, dtype=torch.int32, device=DEV), torch.empty(T, top, device=DEV)
    kw = dict(n_groups=G, keep=keep, group_top=2, scoring=scoring, renormalize=scoring == "sigmoid")
    kern.moe_route(z, corr, want_c, want_w, **kw)
    chosen, weights = torch.full((T, cols), -1, dtype=torch.int32, device=DEV), torch.full((T, cols), -1.0, device=DEV)
    tables = torch.full((2 * Pn + 3 * kern.moe_max_tiles(Pn, n, rows) + 1,), -7, dtype=torch.int32, device=DEV)
    sorted_pairs, pos_of, meta, tiles = tables[:Pn], tables[Pn:2 * Pn], tables[2 * Pn:2 * Pn + 1], tables[2 * Pn + 1:]
    n_real = n if extra else max(1, E - 2)
    kern.moe_route_sort(z, corr, chosen, weights, sorted_pairs, pos_of, tiles, meta, extra=extra, tile_rows=rows, n_real=n_real, **kw)
    assert torch.equal(chosen[:, :top], want_c) and torch.equal(weights[:, :top], want_w)
    if extra:
        assert bool((chosen[:, top] == E).all()) and bool((weights[:, top] == 1.0).all())
    sp, po, flat = sorted_pairs.cpu().long(), pos_of.cpu().long(), chosen.cpu().reshape(-1).long()
    assert torch.equal(sp[po], torch.arange(Pn)) and torch.equal(flat[sp], flat.sort().values)
    tl = tiles.cpu().view(-1, 3)[:int(meta[0])]
    covered = torch.cat([torch.arange(int(f), int(f) + int(m)) for _, f, m in tl])
    assert torch.equal(covered, torch.arange(int((flat < n_real).sum())))
    assert all(bool((flat[sp][int(f):int(f) + int(m)] == int(e)).all()) and 0 < int(m) <= rows for e, f, m in tl)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,D,F,E,top,shared", [(37, 64, 24, 6, 3, 24), (1, 32, 8, 2, 2, None), (300, 96, 48, 4, 2, 40), (5, 40, 13, 9, 1, 16), (5, 40, 16, 9, 2, 16), (16, 64, 32, 7, 1, 32), (20, 64, 32, 16, 3, 32), (700, 64, 24, 30, 4, 64), (400, 64, 160, 5, 2, None)])
def test_experts_without_gates_beside_a_shared_one(dtype, T, D, F, E, top, shared):
    """Few tokens, tiles of 16 rows and of 64: the part's own result, the result added to a stream, and the sum left to the pass that reads it."""
    from levanter_amd.parts import BuildEnv, PartSpec, TensorSpec, part_class
    from levanter_amd.parts.embedding import nested_tensors
    from levanter_amd.parts.base import StepContext

    mlp = P.experts_mlp(ff=F, experts=E, top=top, shared=shared)
    cfg = P.make_config(vocab=8, width=D, layers=[{**P.biased_layer(), "mlp": mlp}])
    W = P.random_weights(cfg, F)
    g = torch.Generator().manual_seed(T)
    h = bfn(torch.randn(T, D, generator=g))
    # a token far from a tie between the last chosen and the first left out, so that the choice is the same in every arithmetic
    z = (h @ W["l0.mlp.router"].T).sort(-1, descending=True).values
    clear = torch.ones(T, dtype=torch.bool) if top == E else (z[:, top - 1] - z[:, top]) > 1e-3
    want = P.experts(h, W, "l0.mlp", mlp)
    names = {"router.weight": "l0.mlp.router", **{f"experts.{e}.{n}.weight": f"l0.mlp.e{e}.{n}" for e in range(E) for n in ("up", "down")}}
    own = lambda d: {k: TensorSpec(v, tuple(W[v].shape)) for k, v in d.items()}
    sh = None if shared is None else PartSpec("dense_mlp", {"dim": D, "inner_dim": shared, "activation": "relu_squared"},
                                              own({f"{n}.weight": f"l0.mlp.shared.{n}" for n in ("up", "down")}), family="feed_forward")
    spec = PartSpec("routed_experts", {"dim": D, "inner_dim": F, "n_experts": E, "top": top, "score": "softmax_chosen", "gated": False, "activation": "relu_squared",
                                       "correction": False, "shared": sh}, own(names), family="feed_forward")
    part = part_class("routed_experts", "feed_forward")(spec, nested_tensors(spec, {k: v.to(dtype) for k, v in W.items()}), BuildEnv(dtype, torch.device(DEV), K()))
    ctx = StepContext(kernels=K(), dtype=dtype, device=torch.device(DEV), n_tokens=T, tokens=None, attention=None, seq_slots=None, host={})
    limits = tol(dtype, f32=1e-4, bf16=6e-2)
    y = torch.full((T, D), float("nan"), device=DEV)
    part.compute(dev(h, dtype), y, ctx)
    torch.testing.assert_close(y.cpu().double()[clear], want[clear], **limits)
    x0 = torch.randn(T, D, generator=g)
    x = dev(x0)
    part.forward(dev(h, dtype), x, ctx)
    torch.testing.assert_close(x.cpu().double()[clear], (x0.double() + want)[clear], **limits)
    y = torch.full((T, D), float("nan"), device=DEV)
    left = part.compute_unsummed(dev(h, dtype), y, ctx)
    # a shared expert of the experts' size (filled up to a multiple of 8) is the last choice of every token where the experts have few rows each
    assert left.alone == (shared is None or (shared == (F + 7) // 8 * 8 and T * (top + 1) < 12 * (E + 1)))
    product = ctx.take_product_pending(y)
    x, nw = dev(x0), torch.ones(D, device=DEV)
    K().finish(K().sum_norm_step(x, alpha=2.0, y=None if left.alone or product is not None else y, product=product, experts=left, write_norm=(nw, None, 1e-5, False), defer=True))
    torch.testing.assert_close(x.cpu().double()[clear], P.norm_after_sum(x0.double(), want, 2.0, torch.ones(D, dtype=torch.float64), 1e-5)[clear], **limits)
    assert int(clear.sum()) >= T // 2


# ---- attention over shuffled pages -----------------------------------------------------------------------------------------------------
def run_attention(dtype, H, G, dk, dv, runs, scale, q, k, v, slopes, sinks, ps=16, seed=0):
    """Keys and values of every request in shuffled pages that hold NaN where nothing was written."""
    kern = K()
    kv_lens = [kv for _, kv in runs]
    n_pages = sum((n + ps - 1) // ps for n in kv_lens) + 3
    bt = random_block_tables(kv_lens, ps, n_pages, seed, DEV)
    k_pages = torch.full((n_pages, G * dk * ps), float("nan"), dtype=dtype, device=DEV)
    v_pages = torch.full((n_pages, G * dv * ps), float("nan"), dtype=dtype, device=DEV)
    for i, n in enumerate(kv_lens):
        dest = ints([int(bt[i, p // ps]) * ps + p % ps for p in range(n)])
        kern.kv_write(dev(k[i].reshape(n, -1), dtype), dev(v[i].reshape(n, -1), dtype), k_pages, v_pages, dest, G, dk, ps, value_dim=dv)
    meta = make_meta(runs, DEV)
    qq = dev(torch.cat([x.reshape(x.shape[0], -1) for x in q]), dtype)
    o = torch.empty(qq.shape[0], H, 1, dv, dtype=torch.float32, device=DEV)
    kern.attention_values(qq, o, k_pages, v_pages, meta, n_heads=H, n_kv_heads=G, head_dim=dk, value_dim=dv, all_value_heads=False, page_size=ps, scale=scale,
                          window=None, block_tables=bt, slopes=None if slopes is None else dev(torch.tensor(slopes)), sinks=None if sinks is None else dev(sinks))
    return o.view(qq.shape[0], H, dv).cpu().double()


def plain_attention(H, G, dk, dv, runs, scale, q, k, v, slopes, sinks):
    outs = []
    for i, (q_len, kv_len) in enumerate(runs):
        full_q = torch.zeros(kv_len, H, dk, dtype=torch.float64)
        full_q[kv_len - q_len:] = q[i]
        outs.append(P.sink_attention(full_q, k[i], v[i], scale, slopes or [0.0] * H, torch.full((H,), -300.0, dtype=torch.float64) if sinks is None else sinks)[kv_len - q_len:])
    return torch.cat(outs)


RUNS = [(70, 70), (1, 130), (19, 83), (1, 1), (2, 2), (1, 17), (130, 261), (1, 48), (1, 241), (5, 245), (1, 500), (64, 320)]  # (queries, keys after the step)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,dk,dv", [(4, 2, 32, 16), (6, 3, 64, 64), (3, 3, 48, 32), (6, 1, 24, 16), (2, 1, 128, 64), (34, 2, 32, 32)])
def test_attention_with_a_distance_term_and_sinks(dtype, H, G, dk, dv):
    g = torch.Generator().manual_seed(H * 100 + dk)
    q, k, v = ([bfn(torch.randn(r[i], n, d, generator=g)) for r in RUNS] for i, n, d in ((0, H, dk), (1, G, dk), (1, G, dv)))
    sinks = torch.randn(H, generator=g).double() * 2 + 1
    sinks[0] = 30.0  # takes nearly all the weight
    slopes = P.distance_slopes(H)
    args = (H, G, dk, dv, RUNS, 2.0 / math.sqrt(dk), q, k, v, slopes, sinks)
    got, want = run_attention(dtype, *args, seed=dk), plain_attention(*args)
    torch.testing.assert_close(got, want, **tol(dtype, f32=3e-5, bf16=3e-2))
    assert float(want[:, 0].abs().max()) < 1e-3
    # a term that grows with the key's position instead of falling with the distance is another result where there is a sink
    shifted = plain_attention(*args[:-2], [0.0] * H, sinks)
    assert float((shifted - want).abs().max()) > 0.3 and float((plain_attention(*args[:-1], None) - want).abs().max()) > 0.3


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,R,dr", [(5, 32, 16), (16, 112, 32), (8, 224, 32), (3, 256, 16), (2, 48, 8)])
def test_attention_over_latents(dtype, H, R, dr):
    """One key of latent and rotated part for all heads, the latent as the value; the largest sizes take other kernels."""
    g = torch.Generator().manual_seed(H * 100 + R)
    dk = R + dr
    q, k = ([bfn(torch.randn(r[i], n, dk, generator=g)) for r in RUNS] for i, n in ((0, H), (1, 1)))
    v = [x[:, :, :R].contiguous() for x in k]
    args = (H, 1, dk, R, RUNS, 2.0 / math.sqrt(dk), q, k, v, None, None)
    torch.testing.assert_close(run_attention(dtype, *args, seed=R), plain_attention(*args), **tol(dtype, f32=3e-5, bf16=3e-2))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("single", [True, False])
@pytest.mark.parametrize("ps", [16, 64])
@pytest.mark.parametrize("latent", [True, False])
def test_a_far_key_among_hundreds_at_page_borders(dtype, single, ps, latent):
    """A key whose score stands out against the sink, the distance term and all other keys, at the first and last places of pages and of the
    sequence."""
    n = 900
    H, G, dk, dv = (4, 1, 144, 112) if latent else (4, 2, 64, 32)
    slopes, sinks = (None, None) if latent else ([2.0 ** -8, 2.0 ** -7, 0.5, 0.25], torch.full((H,), 10.0, dtype=torch.float64))
    g = torch.Generator().manual_seed(5)
    for j in (0, 1, ps - 1, ps, 13 * ps - 1, 512, n - 2, n - 1):
        kk, qq, vv = bfn(torch.randn(n, G, dk, generator=g) * 0.05), bfn(torch.randn(n, H, dk, generator=g)), bfn(torch.randn(n, G, dv, generator=g) * 0.1)
        kk[j, 0] = qq[n - 1, 1]
        vv[j, 0] = 100.0
        ql = 1 if single else 200
        args = (H, G, dk, dv, [(ql, n)], 1.0, [qq[n - ql:]], [kk], [vv], slopes, sinks)
        got = run_attention(dtype, *args, ps=ps, seed=j)
        torch.testing.assert_close(got, plain_attention(*args), **tol(dtype, f32=3e-5, bf16=3e-2))
        assert bool((got[-1, 1] > 90).all()), f"key {j}"


# ---- whole models -----------------------------------------------------------------------------------------------------------------
def middle():
    """Middle sizes for the GPU alone: heads of 64 and 128, a latent of 192 with a rotated part of 64, several tiles of experts a prompt."""
    return P.make_config(vocab=1000, width=256, eps=1e-6, alpha=2.2, logit_scale=0.3, layers=[
        P.biased_layer(heads=8, kv_heads=2, dim=64, vdim=64, q_temp=(0.3, 100), mlp=P.experts_mlp(ff=128, experts=8, top=2, shared=128)),
        P.latent_layer(heads=8, dim=64, rot_dim=64, vdim=64, kv_rank=192, q_rank=128, base=500000.0, scaling=(4.0, 200, 32.0, 1.0), mlp=P.experts_mlp(ff=64, experts=16, top=4, shared=96)),
        P.biased_layer(heads=4, kv_heads=4, dim=128, vdim=32, q_temp=(0.2, 33), mlp=None),
        P.latent_layer(heads=20, dim=32, rot_dim=16, vdim=32, kv_rank=64, q_rank=96, base=1000.0, scaling=None, mlp=P.experts_mlp(ff=256, experts=3, top=1, shared=None)),
    ])


def sharp():
    """Configuration A with queries scaled up: single keys, near and far, take most of the weight."""
    raw, seed = KEL["A"]
    W = P.random_weights(raw, seed)
    for n in list(W):
        if n.endswith("mix.q.norm") or n.endswith("mix.uq"):
            W[n] = bfn(W[n] * 3.0)
    return copy.deepcopy(raw), W


def model_folder(name, tmp, store):
    if name == "sharp":
        raw, W = sharp()
    else:
        raw, seed = (middle(), 31) if name == "middle" else KEL[name]
        W = P.random_weights(raw, seed)
    return raw, W, P.write_folder(raw, W, os.path.join(str(tmp), name), store)


CLOSE = 0.08  # router logits have a spread of about 1.5; bfloat16 moves them by a few hundredths


def logits_and_clear_places(W, raw, tokens):
    """The plain logits, and the places where no router's choice is a close call."""
    with P.close_calls() as margins:
        logits = P.plain_logits(W, raw, tokens)
    clear = torch.ones(len(tokens), dtype=torch.bool)
    for m in margins:
        clear &= m > CLOSE
    return logits, clear


def row_error(got, want):
    """Difference of two rows of logits, mean taken off, relative to the spread of the wanted row."""
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    return (d.pow(2).mean(-1).sqrt() / want.std(-1)).max().item()


LENGTHS = {"A": [70, 45, 100, 37, 64, 33], "B": [90, 130, 41, 200, 64, 17], "C": [40, 12, 150, 3], "D": [33, 50, 41, 64, 80], "middle": [520, 340, 45], "sharp": [150, 64, 300, 47]}


@pytest.mark.parametrize("name,dtype", [(n, d) for n in list(KEL) + ["middle"] for d in ("float32", "bfloat16")] + [("sharp", "float32")])
def test_trace_run_all_cuttings(name, dtype, tmp_path):
    """Whole prompts, the last 32 tokens one by one, portions down to two tokens, and twice mixed with other requests in a pool of exactly
    the peak need (pages and slots are used again), through ``bin/trace_run``."""
    from test_gpu_replay import read_step, run_trace

    raw, W, d = model_folder(name, tmp_path, torch.float32 if dtype == "float32" else torch.bfloat16)
    reqs = TR.random_requests(raw["vocab"], LENGTHS[name], 21)
    both = {rid: logits_and_clear_places(W, raw, t) for rid, t in reqs.items()}
    plain = {rid: b[0] for rid, b in both.items()}
    steps = TR.number(TR.trace_whole(reqs) + TR.trace_prefill_then_singles(reqs) + TR.trace_portions(reqs)
                      + TR.trace_mixed(reqs, seed=3) + TR.trace_mixed(reqs, seed=4, prefix="n"))
    out = run_trace(d, dtype, steps, TR.peak_tokens(steps), extra=("--max-seqs", "4"))
    want = TR.expected_rows(steps, lambda rid: plain[rid[1:]])
    if dtype == "float32":
        limit_of = {rid: torch.full((len(t), 1), 2e-4 if name != "sharp" else 2e-3) for rid, t in reqs.items()}
    else:  # three times what rounding the products' inputs and results alone does at the position (at least what it does at one in ten)
        limit_of = {}
        for rid, t in reqs.items():
            with P.rounded_products():
                rounded = P.plain_logits(W, raw, t)
            err = torch.tensor([row_error(rounded[i:i + 1], plain[rid][i:i + 1]) for i in range(len(t))])
            clear = both[rid][1]
            assert float(clear.double().mean()) > 0.4
            limit = 3 * err.clamp(min=float(err[clear].quantile(0.9)))
            limit[~clear] = math.inf  # where a choice of experts nearly ties, another rounding may choose another one
            limit_of[rid] = limit.view(-1, 1)
    limits = TR.expected_rows(steps, lambda rid: limit_of[rid[1:]])
    worst, rows, over = 0.0, 0, []
    for s in steps:
        k = s["step"]
        assert (k in want) == os.path.exists(os.path.join(out, f"{k}.f32"))
        if k not in want:
            continue
        got = read_step(out, k, raw["vocab"]).double()
        for r in range(got.shape[0]):
            err = row_error(got[r:r + 1], want[k][r:r + 1])
            assert math.isfinite(err)
            rows += math.isfinite(float(limits[k][r]))
            if not err < float(limits[k][r]):
                over.append(f"step {k} row {r}: {err}")
            elif math.isfinite(float(limits[k][r])):
                worst = max(worst, err)
    print(f"kelasun {name} {dtype}: worst relative row error {worst:.3e} over {rows} rows, {len(over)} over the limit")
    # a token that has got another expert may be heard by later ones: in bfloat16 one row in a hundred may miss the limit for that
    assert rows >= 100 and len(over) <= (rows // 100 if dtype == "bfloat16" else 0), over[:10]


def _engine(d, dtype, **kw):
    from levanter_amd.config import InferenceEngineConfig
    from levanter_amd.engine import InferenceEngine

    cfg = InferenceEngineConfig(**{**dict(max_seqs=4, page_size=16, max_pages_per_seq=32, compute_dtype=dtype), **kw})
    return InferenceEngine.from_pretrained(d, cfg)


def check_greedy(W, raw, prompt, generated, dtype):
    """Every token whose two best logits are clearly apart (and, in bfloat16, whose experts are no close call) is the plain argmax."""
    logits, places = logits_and_clear_places(W, raw, list(prompt) + list(generated))
    clear = 0
    for i, tok in enumerate(generated):
        row = logits[len(prompt) - 1 + i]
        top = row.topk(2).values
        sure = dtype == "float32" or bool(places[len(prompt) - 1 + i])
        if sure and float(top[0] - top[1]) > (1e-3 if dtype == "float32" else 0.2) * float(row.std()):
            clear += 1
            assert int(row.argmax()) == tok, f"generated token {i}"
    return clear


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_entry_point(dtype, tmp_path):
    from levanter_amd.engine import Request

    raw, W, d = model_folder("A", tmp_path, torch.float32 if dtype == "float32" else torch.bfloat16)
    g = torch.Generator().manual_seed(0)
    prompts = [torch.randint(0, raw["vocab"], (n,), generator=g).tolist() for n in (5, 17, 33, 1)]
    engine = _engine(d, dtype)
    res = engine.generate([Request(prompt_tokens=p, request_id=i, max_new_tokens=20) for i, p in enumerate(prompts)])
    assert [len(t) for t in res.tokens] == [20] * 4 and res.finish_reasons == ["length"] * 4
    clear = sum(check_greedy(W, raw, p, out, dtype) for p, out in zip(prompts, res.tokens))
    print(f"greedy {dtype}: {clear} of 80 positions decided clearly")
    assert clear >= (76 if dtype == "float32" else 20)
    engine.cache.check_invariants()
    assert engine.cache.n_free_slots == 4


@pytest.mark.parametrize("name", ["A", "B"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_in_replayed_steps(name, dtype, tmp_path):
    """One prompt token, then 300 decoded ones, from the third step on replayed from a graph. Then the first tokens of sequences of one, two and
    three tokens in one batch, in slots and pages that were used before."""
    from levanter_amd.engine import Request

    raw, W, d = model_folder(name, tmp_path, torch.float32 if dtype == "float32" else torch.bfloat16)
    engine = _engine(d, dtype, max_pages=40)
    assert engine.model.graph_safe
    res = engine.generate([Request(prompt_tokens=[7], request_id=0, max_new_tokens=300)])
    out = res.tokens[0]
    assert len(out) == 300
    clear = check_greedy(W, raw, [7], out, dtype)
    print(f"long decoding {name} {dtype}: {clear} of 300 positions decided clearly")
    assert clear >= (280 if dtype == "float32" else 60)
    res = engine.generate([Request(prompt_tokens=p, request_id=i + 1, max_new_tokens=3) for i, p in enumerate(([5], [9, 4], [1, 2, 3]))])
    for p, o in zip(([5], [9, 4], [1, 2, 3]), res.tokens):
        check_greedy(W, raw, p, o, dtype)
    engine.cache.check_invariants()


def test_the_command_line_generates_from_a_folder(tmp_path):
    """``python -m levanter_amd.main.sample_lm`` on a Kelasun folder: greedy tokens are the plain implementation's."""
    import json
    import re
    import subprocess
    import sys

    raw, W, d = model_folder("B", tmp_path, torch.float32)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    prompts = [[3, 14, 15, 9, 2], [6]]
    p = subprocess.run([sys.executable, "-m", "levanter_amd.main.sample_lm", "--hf_checkpoint", d, "--prompt_ids", json.dumps(prompts),
                        "--temperature", "0", "--max_new_tokens", "12", "--n_rounds", "1", "--engine.compute_dtype", "float32",
                        "--engine.max_seqs", "2", "--engine.max_pages_per_seq", "4"], capture_output=True, text=True, cwd=root, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    found = re.findall(r"round 0 sequence (\d+) \(12 tokens, length\): (\[.*\])", p.stdout)
    assert len(found) == 2
    for i, toks in found:
        check_greedy(W, raw, prompts[int(i)], json.loads(toks), "float32")
