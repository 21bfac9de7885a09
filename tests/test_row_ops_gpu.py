"""HIP kernels of the tanh-norm / delta-rule layers against the reference ops
(f32 on the CPU): every kernel variant a shape can select, strided inputs,
padding rows, reused slots."""

from __future__ import annotations

import pytest
import torch

from vllm_tgis_adapter_amd import ops
from vllm_tgis_adapter_amd.ops import reference as ref

pytestmark = pytest.mark.gpu
DEV = "cuda"
BF = torch.bfloat16
DTYPES = [torch.float32, BF]


def _rand(g, *shape, dtype=torch.float32, std=1.0):
    return (torch.randn(*shape, generator=g) * std).to(dtype)


def _gen(seed):
    return torch.Generator().manual_seed(seed)


def _i32(v):
    return torch.tensor(v, dtype=torch.int32)


def _near(got, want, dtype, scale=1.0):
    tol = (2e-5 if dtype == torch.float32 else 1.2e-2) * scale * max(1.0, float(want.abs().max()))
    err = float((got.float().cpu() - want.float()).abs().max())
    assert err < tol, err


# sequences of a step: rows of each, tokens including them, state slots (-1: a
# padding row)
STEPS = {
    "portions": ([5, 17, 1, 40, 2], [5, 30, 9, 40, 2], [3, 0, 4, 1, 2]),
    "single": ([1, 1, 1, 1], [1, 7, 2, 40], [2, 0, 3, 1]),
    "padded": ([1, 1, 1], [9, 1, 0], [1, 0, -1]),
    "gap": ([2, 0, 6], [10, 4, 6], [0, 2, 1]),       # a sequence that brings nothing
}


def _step(name):
    rows, lens, slots = STEPS[name]
    loc = [0]
    for n in rows:
        loc.append(loc[-1] + n)
    return loc[-1], _i32(loc), _i32(lens), _i32(slots)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,width", [(3, 4096), (1500, 256), (7, 30), (2, 1), (1030, 100)])
@pytest.mark.parametrize("two", [False, True])
def test_stream_add_tanh_norm(dtype, rows, width, two):
    g = _gen(rows + width)
    x, a, b = (_rand(g, rows, width) for _ in range(3))
    a, b = (a * 3).to(dtype), b.to(dtype)
    n1 = (0.8, _rand(g, width), _rand(g, width))
    n2 = (1.3, _rand(g, width), _rand(g, width))
    d = lambda n: (n[0], n[1].to(DEV), n[2].to(DEV))
    want = x.clone()
    nxt_want = ref.stream_add_tanh_norm(want, a, b if two else None, n1, n2, torch.float32)
    xs = x.to(DEV)
    nxt = ops.stream_add_tanh_norm(xs, a.to(DEV), d(n1), b=b.to(DEV) if two else None,
                                   next_norm=d(n2), out_dtype=dtype)
    _near(xs, want, torch.float32)
    _near(nxt, nxt_want, dtype)
    # without a next norm, and the next norm alone
    xs = x.to(DEV)
    assert ops.stream_add_tanh_norm(xs, a.to(DEV), d(n1), b=b.to(DEV) if two else None) is None
    _near(xs, want, torch.float32)
    nxt = ops.stream_add_tanh_norm(xs, None, None, next_norm=d(n2), out_dtype=dtype)
    _near(nxt, nxt_want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mix", [False, True])
@pytest.mark.parametrize("rows,heads,kv_heads,dim,vdim,pad", [
    (5, 8, 2, 32, 16, 0), (2050, 4, 4, 16, 8, 8), (3, 32, 8, 128, 128, 0), (4, 3, 1, 6, 10, 3),
    (2, 64, 16, 192, 128, 0), (3, 1, 1, 8, 8, 0), (2, 96, 96, 128, 128, 0)])
def test_wide_norm_cache_write(dtype, mix, rows, heads, kv_heads, dim, vdim, pad):
    g = _gen(rows + heads * dim)
    c = heads * dim + kv_heads * (dim + vdim)
    wide = _rand(g, rows, c + pad, dtype=dtype)
    proj = wide[:, :c]
    bias, qw = _rand(g, c), _rand(g, heads * dim)
    kw = _rand(g, kv_heads * dim)
    bs = 16
    nb = (rows + bs - 1) // bs + 1
    slots = torch.randperm(nb * bs, generator=g)[:rows]
    slots[rows // 2] = -1                     # a padding row
    kc, vc = _rand(g, nb, bs, kv_heads, dim, dtype=dtype), _rand(g, nb, bs, kv_heads, vdim, dtype=dtype)
    vf = _rand(g, nb, bs, kv_heads, vdim, dtype=dtype) if mix else None
    args = (heads, kv_heads, dim, vdim, 1e-5)
    kr, vr, kg, vg = kc.clone(), vc.clone(), kc.to(DEV), vc.to(DEV)
    want = ref.wide_norm_cache_write(proj, bias, *args, qw, kw, vf, 0.3, kr, vr, slots)
    got = ops.wide_norm_cache_write(
        wide.to(DEV)[:, :c], bias.to(DEV), *args, qw.to(DEV), kw.to(DEV),
        None if vf is None else vf.to(DEV), 0.3, kg, vg, slots.to(DEV))
    for a, b in ((got, want), (kg, kr), (vg, vr)):
        _near(a, b, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("step", sorted(STEPS))
@pytest.mark.parametrize("heads,groups,dim,vdim", [
    (4, 2, 32, 32), (4, 4, 64, 24), (6, 2, 128, 128), (2, 1, 16, 200), (2, 2, 256, 64),
    (3, 1, 40, 8), (3, 3, 5, 7), (2, 1, 300, 33)])
@pytest.mark.parametrize("general", [False, True])
def test_delta_gated(dtype, step, heads, groups, dim, vdim, general):
    g = _gen(dim * 7 + vdim)
    t, loc, lens, slots = _step(step)
    c = 2 * groups * dim + heads * vdim
    qkv = _rand(g, t, c, dtype=dtype)
    side = _rand(g, t, heads * vdim + 2 * heads + 4, dtype=dtype)
    state = _rand(g, 6, heads, vdim, dim, std=0.3)
    a_log, dt_bias = _rand(g, heads, std=0.5), _rand(g, heads)
    norm = _rand(g, vdim).repeat(heads)
    gd, hv = groups * dim, heads * vdim

    def run(f, qkv, side, *rest):
        return f(qkv[:, :gd].view(t, groups, dim), qkv[:, gd:2 * gd].view(t, groups, dim),
                 qkv[:, 2 * gd:].view(t, heads, vdim), side[:, hv:hv + heads],
                 side[:, hv + heads:hv + 2 * heads], *rest)

    sw = state.clone()
    o = run(ref.delta_scan, qkv, side, a_log, dt_bias, sw, loc, lens, slots)
    want = ref.gated_group_norm(o, side[:, :hv], norm, heads, 1e-5, False, torch.float32, True)
    want[slots.repeat_interleave(loc.diff()) < 0] = 0.0
    sg = state.to(DEV)
    sd = side.to(DEV)
    got = run(ops.delta_gated, qkv.to(DEV), sd, a_log.to(DEV), dt_bias.to(DEV), sd[:, :hv],
              norm.to(DEV), 1e-5, sg, loc.to(DEV), lens.to(DEV), slots.to(DEV), general)
    assert not torch.isnan(got).any()
    _near(got, want, dtype, scale=3.0)
    _near(sg, sw, torch.float32, scale=3.0)


@pytest.mark.parametrize("general", [False, True])
def test_delta_with_vanishing_decay(general):
    """Decays down to zero: nothing divides by the product of decays once it is
    small, and what was written before a zero is gone."""
    g = _gen(3)
    t, heads, dim, vdim = 60, 2, 32, 32
    q, k, v = _rand(g, t, 1, dim), _rand(g, t, 1, dim), _rand(g, t, heads, vdim)
    b_pre = _rand(g, t, heads)
    a_pre = torch.full((t, heads), -4.0)
    a_pre[::7] = 30.0          # exp(-e^2 * 30): zero in f32
    a_pre[5::11, 1] = 1.0
    a_log, dt_bias = torch.full((heads,), 2.0), torch.zeros(heads)
    loc, lens, slots = _i32([0, t]), _i32([t]), _i32([0])
    norm, gate = torch.ones(heads * vdim), torch.full((t, heads * vdim), 3.0)
    sw = torch.zeros(1, heads, vdim, dim)
    o = ref.delta_scan(q, k, v, b_pre, a_pre, a_log, dt_bias, sw, loc, lens, slots)
    want = ref.gated_group_norm(o, gate, norm, heads, 1e-5, False, torch.float32, True)
    d = lambda x: x.to(DEV)
    sg = torch.full_like(sw, 9.0).to(DEV)
    got = ops.delta_gated(d(q), d(k), d(v), d(b_pre), d(a_pre), d(a_log), d(dt_bias), d(gate),
                          d(norm), 1e-5, sg, d(loc), d(lens), d(slots), general)
    _near(got, want, torch.float32, scale=3.0)
    _near(sg, sw, torch.float32, scale=3.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("step", sorted(STEPS))
@pytest.mark.parametrize("width,taps", [(64, 2), (40, 3), (2056, 4), (24, 5), (12, 4), (8, 1)])
@pytest.mark.parametrize("add_input", [False, True])
def test_short_convolution_walk(dtype, step, width, taps, add_input):
    """The row-walking kernel (2..4 taps, widths in multiples of 8) and the other
    one; single-row steps advance the state in the same launch."""
    g = _gen(width + taps)
    t, loc, lens, slots = _step(step)
    reps = 40 if step == "portions" else 1      # long enough for the 16-row walk
    if reps > 1:
        rows = [n * reps for n in STEPS[step][0]]
        lens = _i32([a + n - m for a, n, m in zip(STEPS[step][1], rows, STEPS[step][0])])
        loc = torch.cat([torch.zeros(1, dtype=torch.int32),
                         torch.cumsum(_i32(rows), 0).to(torch.int32)])
        t = int(loc[-1])
    wide = _rand(g, t, width + 16, dtype=dtype)
    w, bias = _rand(g, width, taps), _rand(g, width)
    st = _rand(g, 6, taps - 1, width, dtype=dtype)
    sw, sg = st.clone(), st.to(DEV)
    want = ref.causal_conv_state(wide[:, 8:8 + width], w, sw, loc, lens, slots, add_input, bias, "silu")
    got = ops.causal_conv_state(wide.to(DEV)[:, 8:8 + width], w.to(DEV), sg, loc.to(DEV),
                                lens.to(DEV), slots.to(DEV), add_input, bias.to(DEV), "silu",
                                has_portions=step in ("portions", "gap"))
    _near(got, want, dtype)
    assert torch.equal(sg.cpu(), sw)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,experts,ff", [(5, 0, 24), (300, 0, 3584), (4, 6, 8), (3, 5, 7)])
def test_clamped_glu(dtype, rows, experts, ff):
    g = _gen(rows + ff)
    gu = _rand(g, rows, max(experts, 1) * 2 * ff, dtype=dtype, std=3.0)
    scale = torch.rand(rows, experts, generator=g) if experts else None
    if experts:
        scale[:, 1] = 0.0
    want = ref.clamped_glu(gu.float(), 1.5, scale)
    got = ops.clamped_glu(gu.to(DEV), 1.5, None if scale is None else scale.to(DEV))
    _near(got, want, dtype)
    if experts:
        assert float(got.view(rows, experts, ff)[:, 1].abs().max()) == 0.0


def test_grouped_clamped_experts_match_reference():
    g = _gen(9)
    e, k, n, t = 5, 256, 128, 300
    x, w = _rand(g, t, k, dtype=BF), _rand(g, e, 2 * n, k, dtype=BF, std=k ** -0.5)
    seg = _i32([0, 0, 130, 131, 290, 300])
    want = ref.moe_gemm(x, w, seg, True, "clamped", 0.6)
    got = ops.moe_gemm(x.to(DEV), w.to(DEV), seg.to(DEV), True, act="clamped", limit=0.6)
    _near(got, want, BF)


@pytest.mark.parametrize("rows_dtype", DTYPES)
@pytest.mark.parametrize("w_dtype", DTYPES)
@pytest.mark.parametrize("rows,experts,width", [
    (1, 16, 64), (40, 5, 96), (17, 32, 4096), (300, 64, 256), (9, 48, 1024), (5, 100, 512),
    (3, 7, 30)])
def test_router_logits(rows_dtype, w_dtype, rows, experts, width):
    g = _gen(experts + width)
    h = _rand(g, rows, width, dtype=rows_dtype)
    w = _rand(g, experts, width, dtype=w_dtype, std=width ** -0.5)
    want = (h.double() @ w.double().T).float()
    got = ops.router_logits(h.to(DEV), w.to(DEV)).cpu()
    assert got.dtype == torch.float32
    assert float((got - want).abs().max()) < 5e-6 * max(1.0, float(want.abs().max()))


@pytest.mark.parametrize("experts,top,groups,keep", [
    (16, 3, 4, 2), (16, 4, 1, 1), (12, 2, 3, 1), (64, 6, 8, 3), (6, 4, 6, 4), (40, 5, 5, 2),
    (32, 1, 16, 1), (128, 8, 8, 4), (96, 3, 2, 1), (2, 1, 2, 1), (1, 1, 1, 1)])
@pytest.mark.parametrize("renorm", [False, True])
def test_routing(experts, top, groups, keep, renorm):
    g = _gen(experts * 3 + top)
    rows, width = 203, 64
    h, w = _rand(g, rows, width, dtype=BF), _rand(g, experts, width, dtype=BF, std=0.2)
    corr = _rand(g, experts, std=0.3) - 0.5
    z = ops.router_logits(h.to(DEV), w.to(DEV))
    rule = (groups, keep, renorm, 1.7)
    want = ref.moe_route_sigmoid(z.cpu(), top, corr, *rule)
    for got in (ops.moe_route_sigmoid(z, top, corr.to(DEV), *rule),
                ops.route_experts(h.to(DEV), w.to(DEV), top, corr.to(DEV), *rule)):
        assert torch.equal(got[1].cpu(), want[1])
        for i in (0, 2):
            assert float((got[i].cpu() - want[i]).abs().max()) < 1e-5
    # without a correction
    want = ref.moe_route_sigmoid(z.cpu(), top, None, *rule)
    got = ops.route_experts(h.to(DEV), w.to(DEV), top, None, *rule)
    assert torch.equal(got[1].cpu(), want[1])


@pytest.mark.parametrize("tokens,top,experts", [(1, 1, 1), (300, 4, 16), (1024, 4, 200),
                                               (1025, 4, 16), (37, 3, 130), (2000, 3, 512)])
def test_pairs_grouped_by_expert(tokens, top, experts):
    """Both ways of placing the pairs (one workgroup up to 4096 pairs)."""
    g = _gen(tokens)
    ids = torch.stack([torch.randperm(experts + 2, generator=g)[:top] for _ in range(tokens)])
    ids = ids.to(torch.int32)                     # the last two ids are identity experts
    h = _rand(g, tokens, 16, dtype=BF)
    xs, pos, seg = (t.cpu() for t in ops.moe_sort(ids.to(DEV), experts, h.to(DEV)))
    counts = torch.bincount(ids[ids < experts].long(), minlength=experts)
    assert torch.equal(seg.diff().long(), counts) and int(seg[0]) == 0
    real = ids < experts
    rows = pos[real].long()
    assert rows.unique().numel() == rows.numel()              # nobody shares a row
    e = ids[real].long()
    assert bool((rows >= seg[e]).all()) and bool((rows < seg[e + 1]).all())
    token = torch.arange(tokens).unsqueeze(1).expand(-1, top)[real]
    assert torch.equal(xs[rows], h[token])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("general", [False, True])
@pytest.mark.parametrize("cap", [0.0, 8.0, 50.0, 90.0])
@pytest.mark.parametrize("heads,kv,dim,vdim", [(4, 2, 64, 64), (6, 2, 96, 64), (8, 1, 128, 128),
                                               (2, 2, 192, 128), (4, 2, 24, 40)])
def test_capped_attention(dtype, general, cap, heads, kv, dim, vdim):
    """Prompt portions and single queries; scores on both sides of the forms the
    kernels choose between; every head with a sink of its own."""
    g = _gen(dim + vdim)
    bs, rows, lens = 16, [70, 3, 260], [150, 33, 260]
    nb = sum((n + bs - 1) // bs for n in lens)
    order = torch.randperm(nb, generator=g)
    tables = torch.zeros(3, max((n + bs - 1) // bs for n in lens), dtype=torch.int32)
    at = 0
    for i, n in enumerate(lens):
        k = (n + bs - 1) // bs
        tables[i, :k] = order[at:at + k]
        at += k
    kc, vc = _rand(g, nb, bs, kv, dim, dtype=dtype), _rand(g, nb, bs, kv, vdim, dtype=dtype)
    q = _rand(g, sum(rows), heads, dim, dtype=dtype)
    sinks = _rand(g, heads, std=3.0)
    qsl = _i32([0, 70, 73, 333])
    d = lambda x: x.to(DEV)
    for scale in (0.2 / dim ** 0.5, 1.5 / dim ** 0.5, 8.0 / dim ** 0.5):
        for window in (0, 45):
            want = ref.paged_attention(q.float(), kc.float(), vc.float(), tables, qsl, _i32(lens),
                                       scale, window, sinks, cap)
            out = torch.empty(q.shape[0], heads, vdim, dtype=dtype, device=DEV)
            ops.gqa_attention_prefill(d(q), d(kc), d(vc), d(tables), d(qsl), d(_i32(lens)), scale,
                                      260, out=out, window=window, sinks=d(sinks), softcap=cap,
                                      general=general)
            _near(out, want, dtype)
            last = qsl[1:].long() - 1
            one = torch.empty(3, heads, vdim, dtype=dtype, device=DEV)
            ops.gqa_attention_decode(d(q[last]), d(kc), d(vc), d(tables), d(_i32(lens)), scale,
                                     out=one, window=window, sinks=d(sinks), softcap=cap,
                                     general=general)
            _near(one, want[last], dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_scale_logits(dtype):
    x = _rand(_gen(1), 7, 1003, dtype=dtype)
    got = ops.scale_logits(x.to(DEV), 0.37).cpu()
    assert got.dtype == torch.float32 and torch.allclose(got, x.float() * 0.37)
