"""The dynamic tanh norm's kernels alone against plain float64: the norm, what is added to the stream through it, products that
take their result into the stream themselves (few and many rows, every way such a product can run), a token's own gated
input, and the routed experts whose weights are a softmax over the chosen logits (dense and grouped products)."""
import pytest
import torch

import plain_gisedra as pg

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
BF16, F32, F64 = torch.bfloat16, torch.float32, torch.float64


@pytest.fixture(scope="module")
def ops():
    from mini_llm_amd.kernels import ops as o
    return o


def _norm(g, D):
    return torch.tensor([0.4 + 0.3 * float(torch.rand(1, generator=g))]), 1.0 + 0.2 * torch.randn(D, generator=g), 0.2 * torch.randn(D, generator=g)


def _dev(n):
    return None if n is None else tuple(t.to(DEV) for t in n)


def _plain(n, v):
    return v if n is None else pg.dynamic_tanh(v, {"n": n[1].to(F64), "n.b": n[2].to(F64), "n.alpha": n[0].to(F64)}, "n")


@pytest.mark.parametrize("D", [5, 64, 1000, 2056])
def test_the_norm(ops, D):
    g = torch.Generator().manual_seed(D)
    x = 3 * torch.randn(7, D, generator=g)
    x[0, 0], x[1, 1], x[2, 2] = 1e6, -1e6, 0.0
    n = _norm(g, D)
    rows = torch.tensor([6, 0, 0, 3], dtype=torch.int32)
    ref = _plain(n, x.to(F64))
    for dtype, tol in ((F32, 1e-6), (BF16, 1e-2)):
        out = ops.tanh_norm(x.to(DEV), _dev(n), torch.empty(7, D, dtype=dtype, device=DEV))
        assert (out.cpu().double() - ref).abs().max() <= tol
        picked = ops.tanh_norm(x.to(DEV), _dev(n), torch.empty(4, D, dtype=dtype, device=DEV), rows.to(DEV))
        assert torch.equal(picked, out[rows.long().to(DEV)])


@pytest.mark.parametrize("T,D", [(1, 7), (3, 64), (70, 1030), (300, 768)])
@pytest.mark.parametrize("with_norm,with_x0,with_step,copied", [(True, False, False, 2), (False, True, True, 1), (True, True, True, 0), (False, False, True, 2)])
def test_added_to_the_stream(ops, T, D, with_norm, with_x0, with_step, copied):
    g = torch.Generator().manual_seed(T + D)
    x, y, x0, step = torch.randn(T, D, generator=g), 2 * torch.randn(T, D, generator=g), torch.randn(T, D, generator=g), torch.randn(D, generator=g)
    n, nx = _norm(g, D), _norm(g, D)
    copy = torch.full((T, D), float("nan"), dtype=BF16, device=DEV) if copied else None
    out = ops.stream_add(x.to(DEV), y.to(DEV) if with_norm else None, _dev(n) if with_norm else None, x0.to(DEV) if with_x0 else None,
                         step.to(DEV) if with_step else None, copy, _dev(nx) if copied == 2 else None, precise=True)
    ref = x.to(F64) + (_plain(n, y.to(F64)) if with_norm else 0) + (x0.to(F64) if with_x0 else 0) + (step.to(F64) if with_step else 0)
    assert (out.cpu().double() - ref).abs().max() <= 2e-6
    if copied:
        want = _plain(nx if copied == 2 else None, ref)
        assert (copy.cpu().double() - want).abs().max() <= 0.01 * want.abs().max()


@pytest.mark.parametrize("M", [1, 8, 9, 16, 17, 33, 64, 100, 300])
@pytest.mark.parametrize("N,K", [(48, 64), (768, 768), (330, 1152), (768, 5632), (4500, 256), (100, 40), (72, 36)])
def test_products_through_norms(ops, M, N, K):
    """Few rows (one tile or two a workgroup, workgroups that share a tile's K), many rows, sizes whose rows are no multiple of
    anything, and a K that the matrix-core kernels do not read; norms on both sides, one or none, with a bias and without."""
    g = torch.Generator().manual_seed(M * 7 + N + K)
    a = torch.randn(M, K, generator=g).to(BF16)
    w = (torch.randn(N, K, generator=g) / K ** 0.5).to(BF16)
    bias = torch.randn(N, generator=g)
    prod = a.to(F64) @ w.to(F64).T
    for with_bias, n, nx, copied in ((False, _norm(g, N), _norm(g, N), True), (True, _norm(g, N), None, True), (False, None, _norm(g, N), True), (True, _norm(g, N), None, False)):
        x = torch.randn(M, N, generator=g)
        copy = torch.full((M, N), float("nan"), dtype=BF16, device=DEV) if copied else None
        y = torch.full((M, N), float("nan"), device=DEV)
        out = ops.linear_stream_add(a.to(DEV), w.to(DEV), x.to(DEV), bias.to(DEV) if with_bias else None, y, _dev(n), copy, _dev(nx))
        ref = x.to(F64) + _plain(n, prod + (bias.to(F64) if with_bias else 0))
        assert (out.cpu().double() - ref).abs().max() <= 2e-4, (with_bias, n is None)
        if copied:
            want = _plain(nx, ref)
            assert (copy.cpu().double() - want).abs().max() <= 0.01 * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("D,dim", [(32, 1), (64, 16), (320, 13), (768, 64), (1024, 32), (1600, 40), (2048, 64)])
@pytest.mark.parametrize("T", [1, 8, 9, 70, 400])
def test_a_tokens_own_input(ops, D, dim, T):
    g = torch.Generator().manual_seed(D + dim + T)
    x = torch.randn(T, D, generator=g)
    xb = x.to(BF16)
    gate = (torch.randn(dim, D, generator=g) / D ** 0.5).to(BF16)
    proj = (torch.randn(D, dim, generator=g) / dim ** 0.5).to(BF16)
    weight = 1.0 + 0.1 * torch.randn(D, generator=g)
    table = torch.randn(19, 3 * dim + 2, generator=g).to(BF16)
    ids = torch.randint(0, 19, (T,), generator=g).to(torch.int32)
    col0 = dim + 1
    nx = _norm(g, D)
    # two of the tokens are fed: their ids are an earlier step's
    src = torch.full((T,), -1, dtype=torch.int32)
    prev = torch.tensor([18, 0, 7], dtype=torch.int32)
    src[0] = 2
    used = ids.clone()
    used[0] = 7
    copy = torch.full((T, D), float("nan"), dtype=BF16, device=DEV)
    out = ops.token_side(x.to(DEV), xb.to(DEV), gate.to(DEV), proj.to(DEV), weight.to(DEV), 1e-5, ids.to(DEV), table.to(DEV), col0, copy, _dev(nx),
                         src.to(DEV), prev.to(DEV))
    z = pg.gelu_tanh(xb.to(F64) @ gate.to(F64).T) * table.to(F64)[used.long(), col0:col0 + dim]
    y = z.to(BF16).to(F64) @ proj.to(F64).T
    ref = x.to(F64) + pg.unit_rms(y, 1e-5) * weight.to(F64)
    err = (out.cpu().double() - ref).abs()
    # (the kernel's z may round to the other bfloat16 neighbour)
    assert err.max() <= 4e-2 and err.mean() <= 4e-3
    want = _plain(nx, out.cpu().double())
    assert (copy.cpu().double() - want).abs().max() <= 0.01 * want.abs().max()


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("joined", [False, True])
@pytest.mark.parametrize("experts,top,ff,D,T", [(5, 2, 24, 48, 9), (3, 3, 7, 45, 70), (1, 1, 32, 48, 1), (70, 3, 8, 64, 33), (6, 1, 16, 64, 40),
                                                (5, 2, 24, 48, 300), (16, 2, 96, 256, 700), (70, 8, 16, 64, 333), (200, 4, 8, 40, 260), (4, 2, 136, 72, 193),
                                                (12, 3, 72, 200, 192)])
def test_gated_experts_weighed_over_the_chosen(ops, dtype, joined, experts, top, ff, D, T):
    """The feed-forward alone: few rows, many rows multiplied densely, and many rows as grouped products (from 192 tokens on in
    bfloat16, where at most half of the experts are chosen): tiles that are not full, experts that nobody chose, more experts
    than a wavefront has lanes, hidden widths and widths that are no multiple of a tile. The result is added to what the stream
    holds."""
    import parts_face as pf
    g = torch.Generator().manual_seed(experts + T)
    w = {"router": (0.4 * torch.randn(experts, D, generator=g)).to(dtype).to(F64), "router.b": 0.5 * torch.randn(experts, generator=g).to(F64)}
    if experts > 4:
        w["router.b"][3] = -60.0                     # an expert that nobody chooses
    for e in range(experts):
        for n, s in (("gate", (ff, D)), ("up", (ff, D)), ("down", (D, ff))):
            w[f"e{e}.{n}"] = (0.15 * torch.randn(*s, generator=g)).to(dtype).to(F64)
    rows = [w[f"e{e}.{n}"] for e in range(experts) for n in ("gate", "up")] + [w["router"]]
    both = torch.cat(rows, dim=0).to(dtype).to(DEV).contiguous()
    down = torch.cat([w[f"e{e}.down"] for e in range(experts)], dim=1).to(dtype).to(DEV).contiguous()
    n = 2 * experts * ff
    bias = w["router.b"].float().to(DEV)
    params = pf.Params(dtype=pf.DT[dtype], experts=experts, ff=ff, top=top, activation="silu_glu", router="softmax_chosen", up__weight=both[:n],
                       down__weight=down, router__bias=bias)
    params.set("router", both[n:])
    if joined:
        params.set("up_router.weight", both)
        params.set("up_router.bias", torch.cat([torch.zeros(n, device=DEV), bias]))
    part = pf.FeedForward("routed_experts", params)
    h = torch.randn(T, D, generator=g).to(dtype)
    x0 = torch.randn(T, D, generator=g)
    ops.reset_seen()
    for _ in range(2):                               # (twice: what the first call left behind does not reach the second)
        x = part.forward(h.to(DEV), x0.clone().to(DEV))
    grouped = dtype == BF16 and T >= 192 and 2 * top <= experts
    assert ops.seen("grouped_experts") == (2 if grouped else 0)
    z = pg.router_logits(h.to(F64), w, "")
    ref = x0.to(F64) + pg.routed_experts(h.to(F64), w, "", {"router": {"experts": experts, "top": top}})
    err = (x.cpu().double() - ref).abs().amax(dim=1)
    srt = z.sort(dim=-1, descending=True).values
    keep = torch.ones(T, dtype=torch.bool) if top >= experts else (srt[:, top - 1] - srt[:, top]) > (1e-5 if dtype == F32 else 1e-4)
    assert keep.float().mean() > 0.9
    scale = float((ref - x0.to(F64)).abs().max())
    assert err[keep].max() <= (1e-5 if dtype == F32 else 2.5e-2) * max(1.0, scale), (float(err[keep].max()), scale)
