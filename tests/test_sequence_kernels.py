"""gfx950 kernels of the layer-listed decoders against the fp32 reference ops,
in bf16 and in float32, over head sizes that hit every kernel and every
padding: equal and unequal key/value widths, odd widths, groups of 1 to 8."""
import pytest
import torch

from aurora_amd import ops
from aurora_amd.ops import sequence, torch_ref

pytestmark = pytest.mark.gpu

DTYPES = [torch.bfloat16, torch.float32]


def close(a, b, dtype, scale=1.0):
    tol = (2e-2 if dtype == torch.bfloat16 else 3e-5) * scale
    a, b = a.float().cpu(), b.float().cpu()
    assert torch.isfinite(a).all()
    err = (a - b).norm() / b.norm().clamp(min=1e-6)
    worst = (a - b).abs().max() / b.abs().max().clamp(min=1e-6)
    assert err < tol and worst < 4 * tol, (float(err), float(worst))


def rnd(*shape, dtype=torch.float32, scale=1.0):
    return (torch.randn(*shape) * scale).to(dtype)


def gpu(*ts):
    return [t.cuda() for t in ts]


# ------------------------------------------------------------ residual norm

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [512, 50, 1028])
@pytest.mark.parametrize("kind", ["plain", "delta", "moe", "gated"])
def test_residual_rmsnorm(dtype, W, kind):
    T, top = 7, 3
    x, w, step = rnd(T, W), rnd(W, scale=0.2), rnd(W)
    args = {}
    if kind == "delta":
        args["delta"] = rnd(T, W, dtype=dtype)
        args["step"] = step
    if kind == "moe":
        args["moe"] = (rnd(T * top, W, dtype=dtype),
                       torch.randperm(T * top).view(T, top).int(),
                       torch.rand(T, top).softmax(-1))
    if kind == "gated":  # the pre-activations are columns of a wider product
        args["delta"] = rnd(T, W, dtype=dtype)
        args["gate"] = (rnd(T, W + 12, dtype=dtype)[:, :W], rnd(W))
    xr, xg = x.clone(), x.cuda()
    want = torch_ref.residual_rmsnorm(xr, w, 1e-5, dtype=dtype, **args)
    dev = {k: tuple(gpu(*v)) if isinstance(v, tuple) else v.cuda() for k, v in args.items()}
    got = ops.residual_rmsnorm(xg, w.cuda(), 1e-5, dtype=dtype, **dev)
    close(got, want, dtype)
    close(xg, xr, torch.float32)


# --------------------------------------------------------------- attention

def _segment(lens, starts, P, slots=None, decode=False, shuffle=True):
    """Packed sequences with ``lens`` new tokens after ``starts`` cached ones."""
    ctx = [a + b for a, b in zip(starts, lens)]
    need = [-(-c // P) for c in ctx]
    order = torch.randperm(sum(need)) if shuffle else torch.arange(sum(need))
    bt = torch.zeros(len(lens), max(need), dtype=torch.int32)
    n = 0
    for i, k in enumerate(need):
        bt[i, :k] = order[n:n + k].int()
        n += k
    cu = [0]
    for x in lens:
        cu.append(cu[-1] + x)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32)  # noqa: E731
    return ops.Segment(
        rows=slice(0, cu[-1]), block_tables=bt, context_lens=i32(ctx), starts=i32(starts),
        state_slots=i32(slots if slots is not None else list(range(len(lens)))),
        cu=None if decode else i32(cu), cu_host=None if decode else cu,
        ctx_host=ctx), sum(need)


def _to(seg, dev):
    mv = lambda t: None if t is None else t.to(dev)  # noqa: E731
    return ops.Segment(seg.rows, mv(seg.block_tables), mv(seg.context_lens), mv(seg.starts),
                       mv(seg.state_slots), mv(seg.cu), seg.cu_host, seg.ctx_host)


ATTN = [  # heads, kv_heads, dim, vdim, window
    (8, 2, 128, 128, 100), (4, 4, 64, 64, 33), (6, 2, 64, 96, 64), (8, 1, 40, 20, 129),
    (5, 1, 128, 64, 0), (14, 2, 112, 128, 257), (2, 1, 160, 24, 70), (3, 3, 20, 300, 65)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,e,window", ATTN)
@pytest.mark.parametrize("decode", [False, True])
def test_biased_attention(dtype, H, G, d, e, window, decode):
    P = 32
    lens = [1] * 4 if decode else [150, 2, 33, 64]
    starts = [0, 63, 500, 129] if decode else [0, 300, 129, 31]
    seg, pages = _segment(lens, starts, P, decode=decode)
    T = sum(lens)
    DK, DV = ops.cache_head_dims(d, e, dtype, "cuda")
    kc, vc = torch.zeros(pages, G, P, DK, dtype=dtype), torch.zeros(pages, G, P, DV, dtype=dtype)
    kc[..., :d] = rnd(pages, G, P, d, dtype=dtype)
    vc[..., :e] = rnd(pages, G, P, e, dtype=dtype)
    # the new tokens' own keys go through the fused write
    c = [8, 8 + H * d, 16 + (H + G) * d]
    proj, bias = rnd(T, c[2] + G * e + 5, dtype=dtype), rnd(H * d + G * (d + e))
    slots = torch.tensor([int(seg.block_tables[s, p // P]) * P + p % P
                          for s in range(len(lens))
                          for p in range(starts[s], starts[s] + lens[s])], dtype=torch.int32)
    kg, vg = kc.cuda(), vc.cuda()
    q = torch_ref.bias_kv_write(proj, c, bias, slots, kc, vc, H, G, d, e)
    qg = ops.bias_kv_write(proj.cuda(), c, bias.cuda(), slots.cuda(), kg, vg, H, G, d, e)
    close(qg, q, dtype)
    close(kg, kc, dtype)
    close(vg, vc, dtype)
    slopes = torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)])
    out = torch.zeros(T, 3 + H * e + 9, dtype=dtype)
    og = out.cuda()
    ops.biased_attention(qg, kg, vg, _to(seg, "cuda"), d ** -0.5, window, slopes.cuda(),
                         og, 3, e, 0.7)
    ops.biased_attention(q.float(), kc.float(), vc.float(), seg, d ** -0.5, window, slopes,
                         out, 3, e, 0.7)
    close(og, out, dtype)
    assert (og[:, :3] == 0).all() and (og[:, 3 + H * e:] == 0).all()


NORMED = [  # heads, kv_heads, dim, vdim, rotated dims, shared keys, whole norm, log bias
    (8, 2, 128, 128, 64, True, False, False), (4, 4, 64, 64, 64, True, False, False),
    (8, 2, 96, 40, 0, False, True, True), (6, 3, 72, 100, 16, False, False, True),
    (5, 1, 33, 33, 10, True, True, False), (14, 2, 112, 128, 0, False, True, True),
    (2, 1, 160, 24, 96, False, False, True), (16, 1, 128, 64, 8, False, True, True)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,e,rot,shared,whole,log", NORMED)
@pytest.mark.parametrize("decode", [False, True])
def test_normed_attention(dtype, H, G, d, e, rot, shared, whole, log, decode):
    """Normed, rotated heads through the cache, then attention with a logarithmic
    distance bias and a sink, or with neither."""
    P = 32
    lens = [1] * 5 if decode else [150, 2, 33, 64]
    starts = [0, 63, 500, 129, 1000] if decode else [0, 300, 129, 31]
    seg, pages = _segment(lens, starts, P, decode=decode)
    T = sum(lens)
    DK, DV = ops.cache_head_dims(d, e, dtype, "cuda")
    kc, vc = torch.zeros(pages, G, P, DK, dtype=dtype), torch.zeros(pages, G, P, DV, dtype=dtype)
    kc[..., :d] = rnd(pages, G, P, d, dtype=dtype)
    vc[..., :e] = rnd(pages, G, P, e, dtype=dtype)
    q0, k0 = 8, 8 + -(-H * d // 8) * 8
    v0 = k0 if shared else k0 + -(-G * d // 8) * 8
    proj = rnd(T, -(-(v0 + G * e) // 8) * 8, dtype=dtype)
    p = ops.NormedHeadsParams(
        H, G, d, e, q0, k0, v0, 1 + rnd(H * d if whole else d, scale=0.3),
        1 + rnd(G * d if whole else d, scale=0.3), whole, 1e-5,
        torch_ref.rope_cos_sin_cache(rot, 2048, 1e4) if rot else None,
        (0.3, 70) if log else None)
    where = [(s, q) for s in range(len(lens)) for q in range(starts[s], starts[s] + lens[s])]
    pos = torch.tensor([q for _, q in where], dtype=torch.int32)
    slots = torch.tensor([int(seg.block_tables[s, q // P]) * P + q % P for s, q in where],
                         dtype=torch.int32)
    if decode:
        slots[2] = -1  # an idle row writes nothing
    kg, vg = kc.cuda(), vc.cuda()
    q = ops.normed_qkv(proj, p, pos, slots, kc, vc)
    qg = ops.normed_qkv(*gpu(proj), _params_to(p, "cuda"), *gpu(pos, slots), kg, vg)
    close(qg, q, dtype)
    close(kg, kc, dtype)
    assert torch.equal(vg.cpu(), vc)
    slopes, rate, sink = (rnd(H).abs(), rnd(H).abs(), rnd(H)) if log else \
        (torch.zeros(H), None, None)
    out = torch.zeros(T, 3 + H * e + 9, dtype=dtype)
    og = out.cuda()
    dev = [None if t is None else t.cuda() for t in (rate, sink)]
    ops.biased_attention(qg, kg, vg, _to(seg, "cuda"), 2 * d ** -0.5, 0, slopes.cuda(),
                         og, 3, e, 0.7, *dev)
    ops.biased_attention(q.float(), kc.float(), vc.float(), seg, 2 * d ** -0.5, 0, slopes,
                         out, 3, e, 0.7, rate, sink)
    close(og, out, dtype)
    assert (og[:, :3] == 0).all() and (og[:, 3 + H * e:] == 0).all()


# -------------------------------------------------------------- recurrences

def _delta(H, G, d, e, taps, dtype, strong):
    at = [0, G * d + 8, 2 * G * d + 8]
    b0 = at[2] + H * e
    p = ops.DeltaRuleParams(
        H, G, d, e, taps, at[0], at[1], at[2], b0, rnd(2 * G * d + H * e, taps),
        rnd(H, scale=0.3) + (2.0 if strong else -1.0), rnd(H * d) - 1.0,
        1 + rnd(e, scale=0.1), 1e-5)
    return p, b0 + H + 3


def _params_to(p, dev):
    return type(p)(**{k: v.to(dev) if torch.is_tensor(v) else v for k, v in vars(p).items()})


DELTA = [  # heads, kv_heads, dim, vdim, taps
    (4, 2, 128, 128, 4), (3, 3, 32, 64, 4), (6, 2, 16, 24, 3), (2, 1, 20, 7, 2),
    (2, 2, 256, 256, 4), (1, 1, 40, 130, 1)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,e,taps", DELTA)
@pytest.mark.parametrize("strong", [False, True])
def test_delta_rule(dtype, H, G, d, e, taps, strong):
    p, C = _delta(H, G, d, e, taps, dtype, strong)
    pg = _params_to(p, "cuda")
    S, ring = rnd(6, H, d, e), rnd(6, taps, 2 * G * d + H * e, dtype=dtype)
    Sg, rg = S.cuda(), ring.cuda()
    # a step of portions (fresh ones among them), then two of single tokens,
    # one row idle
    for lens, starts, slots, dec in (
            ([37, 2, 16, 1], [0, 5, 100, 0], [4, 0, 2, 5], False),
            ([1, 1, 1, 1], [37, 7, 116, 1], [4, 0, 2, 5], True),
            ([1, 1, 1, 1], [38, 8, 0, 0], [4, 0, -1, 3], True)):
        seg, _ = _segment(lens, starts, 64, slots, dec)
        T = sum(lens)
        proj, z = rnd(T, C, dtype=dtype), rnd(T, H * (d + e), dtype=dtype)
        out = torch.zeros(T, 2 + H * e, dtype=dtype)
        og = out.cuda()
        ops.delta_rule(proj, z, p, S, ring, seg, out, 2, 0.5)
        ops.delta_rule(proj.cuda(), z.cuda(), pg, Sg, rg, _to(seg, "cuda"), og, 2, 0.5)
        close(og, out, dtype)
        close(Sg, S, torch.float32, 3.0)
        assert torch.equal(rg.cpu(), ring)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,e,taps", DELTA)
@pytest.mark.parametrize("strong", [False, True])
def test_head_delta_rule(dtype, H, G, d, e, taps, strong):
    up = lambda n: -(-n // 8) * 8  # noqa: E731
    at = [0]
    for n in (G * d, G * d, H * e, H, H, H * e):
        at.append(at[-1] + up(n))
    p = ops.HeadDeltaParams(
        H, G, d, e, taps, *at[:6], rnd(2 * G * d + H * e, taps),
        rnd(H, scale=0.3) + (2.0 if strong else -1.0), rnd(H) - 1.0, 1 + rnd(e, scale=0.1),
        1e-5)
    pg = _params_to(p, "cuda")
    S, ring = rnd(6, H, d, e), rnd(6, taps, 2 * G * d + H * e, dtype=dtype)
    Sg, rg = S.cuda(), ring.cuda()
    for lens, starts, slots, dec in (
            ([37, 2, 16, 1], [0, 5, 100, 0], [4, 0, 2, 5], False),
            ([1, 1, 1, 1], [37, 7, 116, 1], [4, 0, 2, 5], True),
            ([1, 1, 1, 1], [38, 8, 0, 0], [4, 0, -1, 3], True)):
        seg, _ = _segment(lens, starts, 64, slots, dec)
        proj = rnd(sum(lens), at[6], dtype=dtype)
        out = torch.zeros(sum(lens), 2 + H * e, dtype=dtype)
        og = out.cuda()
        ops.head_delta_rule(proj, p, S, ring, seg, out, 2, 0.5)
        ops.head_delta_rule(proj.cuda(), pg, Sg, rg, _to(seg, "cuda"), og, 2, 0.5)
        close(og, out, dtype)
        close(Sg, S, torch.float32, 3.0)
        assert torch.equal(rg.cpu(), ring)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,e", [(4, 128, 128), (3, 32, 48), (3, 20, 7), (2, 256, 256),
                                   (1, 48, 30), (2, 16, 15), (1, 1, 1), (2, 64, 300)])
@pytest.mark.parametrize("forget", [5.0, -6.0])
def test_matrix_memory(dtype, H, d, e, forget):
    """Portions short and long (more tokens than the gates' scan takes at once), then
    single tokens; memories that keep nearly all or nothing."""
    up = lambda n: -(-n // 8) * 8  # noqa: E731
    at = [0]
    for n in (H * d, H * d, H * e, H, H, H * e):
        at.append(at[-1] + up(n))
    p = ops.MatrixMemoryParams(H, d, e, *at[:6], rnd(H) + 1, rnd(H) + forget,
                               1 + rnd(H * e, scale=0.2), 7.0, 1e-5)
    pg = _params_to(p, "cuda")
    S, N, M = rnd(6, H, d, e), rnd(6, H, d) + 2, rnd(6, H).abs()
    Sg, Ng, Mg = gpu(S, N, M)
    for lens, starts, slots, dec in (
            ([37, 2, 16, 1, 1100], [0, 5, 100, 0, 1], [4, 0, 2, 5, 1], False),
            ([1, 1, 1, 1], [37, 7, 116, 1], [4, 0, 2, 5], True),
            ([1, 1, 1, 1], [38, 8, 0, 0], [4, 0, -1, 3], True)):
        seg, _ = _segment(lens, starts, 64, slots, dec)
        proj = rnd(sum(lens), at[6], dtype=dtype)
        out = torch.zeros(sum(lens), 2 + H * e, dtype=dtype)
        og = out.cuda()
        ops.matrix_memory(proj, p, S, N, M, seg, out, 2, 0.5)
        ops.matrix_memory(proj.cuda(), pg, Sg, Ng, Mg, _to(seg, "cuda"), og, 2, 0.5)
        close(og, out, dtype, 3.0)
        close(Mg, M, torch.float32)
        close(Sg, S, torch.float32, 6.0)
        close(Ng, N, torch.float32, 6.0)
        for a, b in ((Sg, S), (Ng, N), (Mg, M)):  # the next step starts from equal ones
            a.copy_(b)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,e,rot", [(4, 128, 128, 128), (3, 32, 48, 32), (3, 20, 12, 8),
                                       (2, 256, 256, 64), (1, 48, 30, 48)])
def test_retention(dtype, H, d, e, rot):
    n, at = H * d, [8, 8 + H * d, 8 + 2 * H * d]
    g0 = at[2] + H * e
    p = ops.RetentionParams(
        H, d, e, rot, *at, g0, 1 - 2.0 ** -(1.0 + 2 * torch.arange(H)),
        torch_ref.rope_cos_sin_cache(rot, 4096, 1e4), 1e-5)
    pg = _params_to(p, "cuda")
    S = rnd(6, H, d, e)
    Sg = S.cuda()
    for lens, starts, slots, dec in (
            ([50, 2, 31, 1], [0, 2000, 100, 0], [4, 0, 2, 5], False),
            ([1, 1, 1, 1], [50, 2002, 0, 1], [4, 0, -1, 5], True)):
        seg, _ = _segment(lens, starts, 64, slots, dec)
        T = sum(lens)
        proj = rnd(T, g0 + H * e, dtype=dtype)
        out = torch.zeros(T, H * e, dtype=dtype)
        og = out.cuda()
        ops.retention(proj, p, S, seg, out)
        ops.retention(proj.cuda(), pg, Sg, _to(seg, "cuda"), og)
        close(og, out, dtype)
        close(Sg, S, torch.float32, 3.0)


# ------------------------------------------------------------------ experts

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,F,E,top", [
    (1, 512, 256, 8, 2), (5, 50, 20, 3, 3), (64, 128, 64, 70, 4), (300, 256, 128, 4, 1),
    (700, 192, 320, 6, 2), (33, 96, 48, 5, 5), (3000, 64, 5760, 2, 2)])
def test_routed_experts(dtype, T, W, F, E, top):
    h = rnd(T, W, dtype=dtype)
    router, bias = rnd(E, W, dtype=dtype, scale=W ** -0.5), rnd(E, scale=0.3)
    gu, dn = rnd(E, 2 * F, W, dtype=dtype, scale=W ** -0.5), rnd(E, W, F, dtype=dtype, scale=F ** -0.5)
    sel, wt = torch_ref.moe_route(h, router, bias, top)
    m = sequence._hip("test")
    sg, wg = m.moe_route(*gpu(h, router, bias), top)
    assert torch.equal(sg.cpu().sort(-1).values, sel.sort(-1).values)
    close(wg, wt, torch.float32)
    y, place = torch_ref.moe_clamped_glu(h, sel, gu, dn, 0.9, 1.702)
    yg, pg = m.moe_clamped_glu(*gpu(h), sel.cuda(), *gpu(gu, dn), 0.9, 1.702, 1.0)
    assert sorted(pg.flatten().tolist()) == list(range(T * top))
    close(yg.cpu()[pg.cpu().long()], y[place.long()], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,E,groups,keep,top", [
    (40, 64, 12, 2, 1, 2), (5, 50, 6, 6, 3, 3), (33, 128, 512, 8, 4, 10), (17, 72, 70, 1, 1, 4),
    (64, 320, 9, 3, 2, 6), (1, 8, 1, 1, 1, 1), (20, 64, 130, 65, 7, 14)])
def test_grouped_router(dtype, T, W, E, groups, keep, top):
    h, router = rnd(T, W, dtype=dtype), rnd(E, W, dtype=dtype, scale=2 * W ** -0.5)
    corr = rnd(E, scale=0.3) - 1.0  # choice scores of both signs
    args = (top, groups, keep, 2.5)
    sel, wt = torch_ref.moe_route_grouped(h, router, corr, *args)
    sg, wg = sequence._hip("test").moe_route_grouped(*gpu(h, router, corr), *args)
    assert torch.equal(sg.cpu().sort(-1).values, sel.sort(-1).values)
    order = (x.argsort(-1) for x in (sg.cpu(), sel))
    close(wg.cpu().gather(1, next(order)), wt.gather(1, next(order)), torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W,F,E,top", [(64, 128, 64, 7, 2), (5, 50, 20, 3, 3)])
def test_plain_glu_experts(dtype, T, W, F, E, top):
    h = rnd(T, W, dtype=dtype, scale=8.0)  # beyond any clamp
    gu, dn = rnd(E, 2 * F, W, dtype=dtype, scale=W ** -0.5), rnd(E, W, F, dtype=dtype, scale=F ** -0.5)
    sel = torch.rand(T, E).topk(top).indices.int()
    args = (float("inf"), 1.0, 0.0)
    y, place = sequence.expert_rows(h, sel, gu, dn, *args)
    yg, pg = sequence.expert_rows(*gpu(h, sel, gu, dn), *args)
    close(yg.cpu()[pg.cpu().long()], y[place.long()], dtype)


# --------------------------------------------------------------- output norms

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,W", [(7, 512), (5, 50), (3, 2052), (300, 1028)])
@pytest.mark.parametrize("kind", ["delta", "moe", "both"])
@pytest.mark.parametrize("depth", [0, 1, 6])
@pytest.mark.parametrize("final", [False, True])
def test_output_norm(dtype, T, W, kind, depth, final):
    src, w, b = rnd(T, W), 1 + rnd(W, scale=0.2), rnd(W)
    top, args = 3, {}
    if kind != "moe":
        args["delta"] = rnd(T, W, dtype=dtype) + 3.0  # a mean that matters
    if kind != "delta":
        args["moe"] = (rnd(T * top, W, dtype=dtype),
                       torch.randperm(T * top).view(T, top).int(),
                       torch.rand(T, top).softmax(-1))
    if kind == "both":
        args["gate"] = rnd(T, 11, dtype=dtype)[:, 4]
    if final:
        args["final"] = (1 + rnd(W, scale=0.2), rnd(W))
    dev = {k: tuple(gpu(*v)) if isinstance(v, tuple) else v.cuda() for k, v in args.items()}
    room = (depth + 1, depth)[final]  # the last result is not kept
    kept = rnd(room, T, W)
    kg = kept.cuda()
    if depth:
        coefs = rnd(depth + 1)
        args["depth"], dev["depth"] = (kept, coefs), (kg, coefs.cuda())
    x, xg = torch.empty(T, W), torch.empty(T, W, device="cuda")
    want = torch_ref.output_norm(src, x, w, b, 1e-5, dtype=dtype, **args)
    got = ops.output_norm(src.cuda(), xg, w.cuda(), b.cuda(), 1e-5, dtype=dtype, **dev)
    close(got, want, dtype)
    close(xg, x, torch.float32)
    if depth:
        close(kg, kept, torch.float32)
    # in place
    xg = src.cuda()
    ops.output_norm(xg, xg, w.cuda(), b.cuda(), 1e-5, dtype=dtype, **dev)
    close(xg, x, torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("F", [256, 36, 5])
def test_gelu_and_silu_glu(dtype, F):
    z = torch.cat([rnd(9, 2 * F + 3), rnd(9, 2 * F + 3, scale=1e-3),
                   rnd(9, 2 * F + 3, scale=8.0)]).to(dtype)
    close(ops.silu_glu(z.cuda(), F), ops.silu_glu(z.float(), F), dtype)
    for x in (z, z[:, :F], z[:, :2 * F].contiguous()):
        close(ops.gelu(x.cuda()), ops.gelu(x.float()), dtype)


# ------------------------------------- embeddings, input convolution, activation

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [288, 50])
def test_embed_pairs(dtype, W):
    V, B = 200, 31
    table, pairs, w = rnd(V, W, dtype=dtype), rnd(B + 1, W, dtype=dtype), rnd(W)
    prev = torch.randint(0, V, (6, 1), dtype=torch.int32)
    pg = prev.cuda()
    # factors whose products leave 32 bits behind
    mul = (2 ** 33 + 7, 2 ** 31 - 1)
    for lens, starts, slots, dec in (
            ([37, 2, 16, 1, 2], [0, 5, 100, 0, 1], [4, 0, 2, 5, 1], False),
            ([1, 1, 1, 1], [37, 7, 0, 0], [4, 0, -1, 3], True)):
        seg, _ = _segment(lens, starts, 64, slots, dec)
        ids = torch.randint(0, V, (sum(lens),))
        want = ops.embed_pairs(ids, table, 3.5, pairs, *mul, w, 1e-5, prev, [seg])
        got = ops.embed_pairs(ids.cuda(), table.cuda(), 3.5, pairs.cuda(), *mul, w.cuda(),
                              1e-5, pg, [_to(seg, "cuda")])
        close(got, want, torch.float32)
        assert torch.equal(pg.cpu(), prev)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [288, 50, 2056])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 6, 7, 16])
def test_short_conv_and_its_fused_form(dtype, W, taps):
    w, nw = rnd(taps, W, scale=0.5), rnd(W)
    ring = rnd(6, taps - 1, W, dtype=dtype)
    rg = ring.cuda()
    for lens, starts, slots, dec in (
            ([37, 2, 16, 1, 33], [0, 5, 100, 0, 2], [4, 0, 2, 5, 1], False),
            ([1, 1, 1, 1], [37, 7, 116, 1], [4, 0, 2, 5], True),
            ([1, 1, 1, 1], [38, 8, 0, 0], [4, 0, -1, 3], True)):
        seg, _ = _segment(lens, starts, 64, slots, dec)
        x = rnd(sum(lens), W)
        delta, gate = rnd(*x.shape, dtype=dtype), (rnd(*x.shape, dtype=dtype), rnd(W))
        xg = x.cuda()
        kw = dict(dtype=dtype, offset=0.0)
        h, u = ops.residual_rmsnorm_conv(x, nw, 1e-5, w, ring, [seg], delta=delta, gate=gate, **kw)
        hg, ug = ops.residual_rmsnorm_conv(
            xg, nw.cuda(), 1e-5, w.cuda(), rg, [_to(seg, "cuda")], delta=delta.cuda(),
            gate=(gate[0].cuda(), gate[1].cuda()), **kw)
        close(hg, h, dtype)
        close(ug, u, dtype)
        close(rg, ring, dtype) if taps > 1 else None
        rg.copy_(ring)  # the next step starts from equal pasts
    # portions beside single tokens: one segment after the other
    seg, _ = _segment([20, 3], [0, 9], 64, [1, 2])
    one, _ = _segment([1, 1], [4, 30], 64, [3, 0], True)
    one.rows = slice(23, 25)
    x = rnd(25, W)
    xg = x.cuda()
    h, u = ops.residual_rmsnorm_conv(x, nw, 1e-5, w, ring, [seg, one], **kw)
    hg, ug = ops.residual_rmsnorm_conv(xg, nw.cuda(), 1e-5, w.cuda(), rg,
                                       [_to(seg, "cuda"), _to(one, "cuda")], **kw)
    close(ug, u, dtype)
    close(rg, ring, dtype) if taps > 1 else None


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("F", [256, 36])
def test_xielu(dtype, F):
    z = torch.cat([rnd(9, F), rnd(9, F, scale=1e-3), rnd(9, F, scale=30.0)]).to(dtype)
    wide = torch.cat([z, z], 1)
    for act in ([0.3, -0.7], [-40.0, 30.0]):
        a = torch.tensor(act)
        want = ops.xielu(z.float(), a).to(dtype)
        close(ops.xielu(wide.cuda()[:, F:], a.cuda()), want, dtype)
        close(ops.xielu(z.cuda(), a.cuda()), want, dtype)


# ---------------------------------------------------------- latent attention

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H,K,N", [(1, 3, 64, 128), (17, 2, 512, 64), (40, 5, 256, 96),
                                     (64, 1, 32, 32), (150, 4, 128, 512), (70, 2, 320, 128)])
def test_head_linear(dtype, T, H, K, N):
    x, w = rnd(T, 8 + H * K, dtype=dtype), rnd(H, N, K, dtype=dtype, scale=K ** -0.5)
    gate = rnd(T, H + 2, dtype=dtype)[:, :H]
    xh = x[:, 8:].unflatten(1, (H, K))
    want = torch.einsum("thk,hnk->thn", xh.float(), w.float())
    xg = x.cuda()[:, 8:].unflatten(1, (H, K))
    close(sequence.head_linear(xg, w.cuda()), want, dtype)
    out = torch.zeros(T, H * N, dtype=dtype, device="cuda")
    sequence.head_linear(xg, w.cuda(), gate.cuda(), out.unflatten(1, (H, N)))
    close(out.cpu().unflatten(1, (H, N)), want * torch.sigmoid(gate.float()).unsqueeze(-1), dtype)


LATENT = [  # heads, dim, vdim, rank
    (5, 64, 64, 128), (3, 20, 100, 50), (16, 128, 128, 512), (17, 64, 128, 256),
    (40, 128, 64, 300), (1, 160, 72, 384), (6, 32, 32, 520), (2, 128, 128, 700), (33, 40, 24, 64)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,e,rank", LATENT)
@pytest.mark.parametrize("regime", ["decode", "portions", "long", "many"])
def test_latent_attention(dtype, H, d, e, rank, regime, monkeypatch):
    """Padded sizes as the mixer makes them; each regime's own form, and for
    portions both."""
    P = 48
    decode = regime in ("decode", "many")
    lens, starts = {"decode": ([1] * 4, [0, 63, 500, 129]),
                    "many": ([1] * 70, [(37 * i) % 200 for i in range(70)]),
                    "portions": ([2, 33, 7, 64], [300, 129, 0, 31]),
                    "long": ([200, 300], [0, 70])}[regime]
    seg, pages = _segment(lens, starts, P, decode=decode)
    T, R = sum(lens), ops.latent_width(rank)
    D, E = ops.latent_head_width(d), ops.latent_head_width(e)
    cache = torch.zeros(pages, 1, P, R, dtype=dtype)
    cache[..., :rank] = rnd(pages, 1, P, rank, dtype=dtype)
    c0 = H * D
    g0 = c0 + -(-rank // 8) * 8
    proj = rnd(T, g0 + -(-H // 8) * 8, dtype=dtype)
    w = rnd(rank)
    slots = torch.tensor([int(seg.block_tables[s, p // P]) * P + p % P
                          for s in range(len(lens))
                          for p in range(starts[s], starts[s] + lens[s])], dtype=torch.int32)
    cg = cache.cuda()
    ops.latent_write(proj, c0, rank, w, 1e-5, slots, cache)
    ops.latent_write(proj.cuda(), c0, rank, w.cuda(), 1e-5, slots.cuda(), cg)
    close(cg, cache, dtype)
    cg.copy_(cache)
    uk, uv = torch.zeros(H, D, R, dtype=dtype), torch.zeros(H, E, R, dtype=dtype)
    uk[:, :d, :rank] = rnd(H, d, rank, dtype=dtype, scale=rank ** -0.5)
    uv[:, :e, :rank] = rnd(H, e, rank, dtype=dtype, scale=rank ** -0.5)
    p = ops.LatentParams(H, D, E, 2.0 * d ** -0.5, 0, g0, uk,
                         uk.transpose(1, 2).contiguous(), uv, rnd(H, scale=2.0))
    out = torch.zeros(T, H * E, dtype=dtype)
    ops.latent_attention(proj, p, cache, seg, out)
    pg, sg = _params_to(p, "cuda"), _to(seg, "cuda")
    for expand in [False] if decode else [False, True]:
        if expand and (D > 128 or E > 128 or R not in sequence.MATRIX_LATENT_WIDTHS):
            continue
        monkeypatch.setattr(sequence, "expand_latents", lambda *a: expand)
        og = torch.zeros(T, H * E, dtype=dtype, device="cuda")
        ops.latent_attention(proj.cuda(), pg, cg, sg, og)
        close(og, out, dtype)
