"""HIP kernels of the grouped residual norm, the rotation table, the attention
inputs (bias, short convolution, norms, rotations, cache write), pooled
key/value blocks, attention over a window plus a prefix, gated linear attention
and the biased silu gate against the plain-PyTorch reference ops, on sizes that
hit vector, scalar and matrix-core paths."""

import math

import pytest
import torch

from vllm_tgis_adapter_amd import ops
from vllm_tgis_adapter_amd.ops import reference as ref

pytestmark = pytest.mark.gpu

DEV = "cuda"
DTYPES = [torch.float32, torch.bfloat16]


def _close(a, b, dtype, what=""):
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    a, b = a.float().cpu(), b.float().cpu()
    assert a.shape == b.shape, what
    if a.numel() == 0:
        return
    scale = max(1.0, float(b.abs().max()))
    err = float((a - b).abs().max()) / scale
    assert err < tol, f"{what}: {err}"


def _i32(v):
    return torch.tensor(v, dtype=torch.int32)


def _dev(t):
    return None if t is None else t.to(DEV)


# sequences of a step: rows per sequence, length after the step, slot
SEQS = [
    ([3, 1, 5], [3, 9, 12], [2, 0, 3]),            # new, single token, continued portion
    ([1, 1, 1, 1], [1, 20, 7, 2], [1, -1, 0, 3]),  # decode rows, one padding row
    ([40], [40], [1]),
    ([2, 0, 6], [10, 4, 6], [0, 2, 1]),            # a sequence that brings nothing
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,groups", [(6, 3), (96, 2), (1000, 5), (1024, 1), (4096, 4),
                                          (4096, 2), (768, 16), (120, 20), (8192, 1),
                                          (12288, 2), (36864, 1)])
def test_stream_add_group_norm(dtype, width, groups):
    g = torch.Generator().manual_seed(width)
    t = 5
    x = torch.randn(t, width, generator=g)
    a, b = (torch.randn(t, width, generator=g).to(dtype) for _ in range(2))
    vec = [torch.randn(width, generator=g) for _ in range(5)]
    bias, wa, wb, w_out, next_w = vec
    for case in (dict(), dict(a_bias=bias), dict(b=b, wa=wa, wb=wb, mix=0.5),
                 dict(b=b, wa=wa, wb=wb, mix=0.3, a_bias=bias)):
        for nw in (next_w, None):
            xr, xg = x.clone(), x.clone().to(DEV)
            want = ref.stream_add_group_norm(xr, a, case.get("a_bias"), case.get("b"),
                                             case.get("wa"), case.get("wb"), w_out, groups, 1e-5,
                                             case.get("mix", 0.5), nw, dtype)
            kw = {k: _dev(v) if torch.is_tensor(v) else v for k, v in case.items()}
            got = ops.stream_add_group_norm(xg, a.to(DEV), w_out.to(DEV), groups, 1e-5,
                                            next_w=_dev(nw), out_dtype=dtype, **kw)
            _close(xg, xr, torch.float32, f"stream {sorted(case)}")
            assert (got is None) == (want is None)
            if want is not None:
                _close(got, want, dtype, f"next norm {sorted(case)}")
    want = ref.stream_add_group_norm(x.clone(), None, None, None, None, None, None, groups, 1e-5,
                                     0.5, next_w, dtype)
    got = ops.stream_add_group_norm(x.to(DEV), None, None, groups, 1e-5, next_w=next_w.to(DEV),
                                    out_dtype=dtype)
    _close(got, want, dtype, "norm alone")


def test_rotary_table():
    pos = torch.tensor([0, 1, 17, 1000, 30000])
    inv = torch.tensor([20.0 ** (-2.0 * i / 22) for i in range(11)])
    got = ops.rotary_table(pos.to(DEV), inv.to(DEV)).double().cpu()
    ang = (pos.float().unsqueeze(1) * inv.unsqueeze(0)).double()
    assert float((got[..., 0] - ang.cos()).abs().max()) < 1e-6
    assert float((got[..., 1] - ang.sin()).abs().max()) < 1e-6


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [0, 1, 2, 3, 4, 6])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,rot,vrot,pad", [
    (4, 2, 8, 12, 4, 12, 3), (3, 1, 10, 6, 0, 0, 0), (2, 2, 64, 64, 64, 64, 8),
    (8, 2, 128, 128, 128, 128, 8), (4, 4, 128, 128, 0, 0, 0), (4, 1, 96, 32, 32, 32, 16),
    (5, 5, 40, 48, 16, 48, 8), (2, 1, 128, 64, 64, 0, 8), (1, 1, 300, 20, 300, 20, 0),
    (34, 17, 16, 16, 16, 16, 0),
])
def test_attn_inputs_cache_write(dtype, taps, heads, kv_heads, dim, vdim, rot, vrot, pad):
    g = torch.Generator().manual_seed(taps)
    bs, blocks = 4, 30
    ch = heads * dim + kv_heads * (dim + vdim)
    for case, (rows, lens, slots) in enumerate(SEQS):
        t = sum(rows)
        proj = torch.randn(t, ch + pad, generator=g).to(dtype)
        bias = torch.randn(ch, generator=g) if case != 2 else None
        qw, kw = (torch.rand(dim, generator=g) + 0.5 for _ in range(2))
        if case % 2:
            qw = kw = None
        cw = torch.randn(taps, ch, generator=g) if taps else None
        state = torch.randn(4, max(taps - 1, 0), ch, generator=g).to(dtype) if taps else None
        pos = torch.cat([torch.arange(n - r, n) for r, n in zip(rows, lens)])
        tab = lambda n: ref.rotary_table(pos, torch.rand(n // 2, generator=g)) if n else None
        rt, vt = tab(rot), tab(vrot)
        sm = torch.randperm(bs * blocks, generator=g)[:t]
        loc = _i32([0] + torch.tensor(rows).cumsum(0).tolist())
        if case == 1:
            sm[1] = -1                      # the padding row
        single = all(r == 1 for r in rows)
        real = torch.ones(t, dtype=torch.bool)
        real[[i for i in range(t) if single and slots[i] < 0]] = False

        def run(dev, portions):
            d = lambda x: None if x is None else x.to(dev)
            kc = torch.zeros(blocks, bs, kv_heads, dim, dtype=dtype, device=dev)
            vc = torch.zeros(blocks, bs, kv_heads, vdim, dtype=dtype, device=dev)
            st = None if state is None else state.clone().to(dev)
            q = ops.attn_inputs_cache_write(
                d(proj)[:, :ch], d(bias), heads, kv_heads, dim, vdim, 1e-5, d(qw), d(kw), d(cw),
                st, d(rt), d(vt), kc, vc, d(sm), d(loc), d(_i32(lens)), d(_i32(slots)),
                has_portions=portions)
            if st is not None:     # rows kept for positions before the start mean nothing
                st = torch.cat([st[s, max(0, taps - 1 - n):].flatten()
                                for s, n in zip(slots, lens) if s >= 0])
            return q[real.to(dev)], kc, vc, st

        want = run("cpu", True)
        for portions in ([True, False] if single else [True]):
            got = run(DEV, portions)
            for gg, ww, what in zip(got, want, ("queries", "key cache", "value cache", "state")):
                if ww is not None:
                    _close(gg, ww, dtype, f"{what} case {case}")


@pytest.mark.parametrize("long", [1100, 3300])
def test_attn_inputs_many_rows_in_one_workgroup(long):
    """Rows enough for the kernel to walk eight or sixteen of them per
    workgroup, with sequences that begin and end inside such a run."""
    g = torch.Generator().manual_seed(1)
    rows = [5, 1, 900, 2, 3, long, 70]
    lens = [5, 4, 900, 9, 3, long + 3, 70]
    slots = [0, 3, 1, 2, 5, 4, 6]
    heads, kvh, dim, taps, bs = 2, 1, 32, 3, 16
    t, ch = sum(rows), (2 + 1 + 1) * 32
    assert t >= 2048
    proj = torch.randn(t, ch, generator=g).to(torch.bfloat16)
    state = torch.randn(7, taps - 1, ch, generator=g).to(torch.bfloat16)
    bias, cw = torch.randn(ch, generator=g), torch.randn(taps, ch, generator=g)
    w = torch.ones(dim)
    pos = torch.cat([torch.arange(n - r, n) for r, n in zip(rows, lens)])
    tab = ref.rotary_table(pos, torch.rand(16, generator=g))
    loc = _i32([0] + torch.tensor(rows).cumsum(0).tolist())
    outs = []
    for dev in ("cpu", DEV):
        kc = torch.zeros(t // bs + 1, bs, kvh, dim, dtype=torch.bfloat16, device=dev)
        vc, st = torch.zeros_like(kc), state.clone().to(dev)
        q = ops.attn_inputs_cache_write(
            proj.to(dev), bias.to(dev), heads, kvh, dim, dim, 1e-5, w.to(dev), w.to(dev),
            cw.to(dev), st, tab.to(dev), tab.to(dev), kc, vc, torch.arange(t, device=dev),
            loc.to(dev), _i32(lens).to(dev), _i32(slots).to(dev))
        outs.append((q, kc, vc, st))
    for gg, ww, what in zip(outs[1], outs[0], ("queries", "keys", "values", "state")):
        _close(gg, ww, torch.bfloat16, what)


def _paged(ctx_lens, kv_heads, dim, vdim, bs, pool, dtype, g):
    """Caches with scattered blocks; pooled entries filled by the reference."""
    nblk = [(n + bs - 1) // bs for n in ctx_lens]
    total = sum(nblk) + 2
    order = torch.randperm(total, generator=g).tolist()
    tables = torch.zeros(len(ctx_lens), max(max(nblk), 1), dtype=torch.int32)
    for i, n in enumerate(nblk):
        for j in range(n):
            tables[i, j] = order.pop()
    kc = torch.randn(total, bs, kv_heads, dim, generator=g).to(dtype)
    vc = torch.randn(total, bs, kv_heads, vdim, generator=g).to(dtype)
    kp = vp = None
    if pool:
        n = ref.pool_slots_per_block(bs, pool)
        kp = torch.full((total, n, kv_heads, dim), 7.0, dtype=dtype)
        vp = torch.full((total, n, kv_heads, vdim), 7.0, dtype=dtype)
        qsl = _i32([0] + torch.tensor(ctx_lens).cumsum(0).tolist())
        ref.pool_cache_write(kc, vc, kp, vp, pool, tables, qsl, _i32(ctx_lens))
    return kc, vc, kp, vp, tables


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kv_heads,dim,vdim", [(2, 16, 24), (1, 5, 3), (4, 128, 128)])
@pytest.mark.parametrize("pool,bs", [(4, 16), (16, 16), (5, 16), (40, 16), (1, 4), (3, 8),
                                     (24, 16)])
def test_pool_cache_write(dtype, kv_heads, dim, vdim, pool, bs):
    g = torch.Generator().manual_seed(pool)
    ctx = [130, 48, 7, 0, 96]
    new = [130, 3, 7, 0, 50]
    kc, vc, kp, vp, tables = _paged(ctx, kv_heads, dim, vdim, bs, pool, dtype, g)
    for rows, qsl in ((new, _i32([0] + torch.tensor(new).cumsum(0).tolist())), ([1] * 5, None)):
        kr, vr = torch.zeros_like(kp), torch.zeros_like(vp)
        ops.pool_cache_write(kc, vc, kr, vr, pool, tables, qsl, _i32(ctx), sum(rows))
        kg, vg = torch.zeros_like(kp).to(DEV), torch.zeros_like(vp).to(DEV)
        ops.pool_cache_write(kc.to(DEV), vc.to(DEV), kg, vg, pool, tables.to(DEV), _dev(qsl),
                             _i32(ctx).to(DEV), sum(rows))
        _close(kg, kr, dtype, "pooled keys")
        _close(vg, vr, dtype, "pooled values")


SHAPES = [(8, 2, 16, 24), (4, 4, 64, 64), (6, 2, 40, 300), (3, 3, 6, 514),
          (8, 4, 128, 128), (16, 2, 128, 128), (4, 1, 64, 64)]      # matrix-core shapes
PREFIXES = [(40, 0, 0), (40, 5, 0), (24, 100, 0), (1, 3, 0), (33, 0, 4), (16, 0, 16), (5, 0, 1),
            (50, 0, 24), (0, 0, 0), (300, 64, 0), (64, 0, 10), (130, 130, 0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window,keep,pool", PREFIXES)
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", SHAPES)
def test_span_attention(dtype, window, keep, pool, heads, kv_heads, dim, vdim):
    g = torch.Generator().manual_seed(window + 7 * pool + keep)
    bs = 16
    ctx = [7, 300, 33, 500, 410, 2]
    new = [7, 1, 33, 260, 3, 2]
    kc, vc, kp, vp, tables = _paged(ctx, kv_heads, dim, vdim, bs, pool, dtype, g)
    scale = 1.5 / math.sqrt(dim)
    for back in (False, True):
        if back and vdim % 2:
            continue
        # portions
        t = sum(new)
        q = torch.randn(t, heads, dim, generator=g).to(dtype)
        qsl = _i32([0] + torch.tensor(new).cumsum(0).tolist())
        tab = None
        if back:
            pos = torch.cat([torch.arange(c - n, c) for c, n in zip(ctx, new)])
            tab = ref.rotary_table(pos, torch.rand(vdim // 2, generator=g))
        want = ref.span_attention(q, kc, vc, kp, vp, tables, qsl, _i32(ctx), scale, window, keep,
                                  pool, tab)
        for general in (False, True):
            out = torch.empty(t, heads, vdim, dtype=dtype, device=DEV)
            ops.span_attention_prefill(
                q.to(DEV), kc.to(DEV), vc.to(DEV), _dev(kp), _dev(vp), tables.to(DEV),
                qsl.to(DEV), _i32(ctx).to(DEV), scale, max(new), window, keep, pool, _dev(tab),
                out=out, general=general)
            _close(out, want, dtype, f"portions back={back} general={general}")
        # one query each, one padding row
        lens = list(ctx)
        lens[2] = 0
        q = torch.randn(len(ctx), heads, dim, generator=g).to(dtype)
        tab = ref.rotary_table(_i32([max(n - 1, 0) for n in lens]),
                               torch.rand(vdim // 2, generator=g)) if back else None
        one = torch.arange(len(ctx) + 1, dtype=torch.int32)
        want = ref.span_attention(q, kc, vc, kp, vp, tables, one, _i32(lens), scale, window, keep,
                                  pool, tab)
        for general in (False, True):
            out = torch.empty(len(ctx), heads, vdim, dtype=dtype, device=DEV)
            ops.span_attention_decode(
                q.to(DEV), kc.to(DEV), vc.to(DEV), _dev(kp), _dev(vp), tables.to(DEV),
                _i32(lens).to(DEV), scale, window, keep, pool, _dev(tab), out=out,
                general=general)
            _close(out, want, dtype, f"decode back={back} general={general}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,vdim,rank", [(3, 6, 10, 5), (2, 64, 64, 16), (1, 128, 128, 16),
                                                 (2, 48, 33, 7), (1, 256, 20, 130),
                                                 (4, 16, 300, 1)])
@pytest.mark.parametrize("case", range(len(SEQS)))
def test_gla_scan(dtype, heads, dim, vdim, rank, case):
    rows, lens, slots = SEQS[case]
    g = torch.Generator().manual_seed(case)
    t = sum(rows)
    loc = _i32([0] + torch.tensor(rows).cumsum(0).tolist())
    a = heads * dim
    proj = torch.randn(t, 2 * a + heads * vdim + rank + 8, generator=g).to(dtype)
    a2 = torch.randn(rank, a, generator=g) / math.sqrt(rank)
    bias = torch.randn(a, generator=g)
    state = torch.randn(4, heads, vdim, dim, generator=g)

    def run(dev, fn):
        p, st = proj.to(dev), state.clone().to(dev)
        b = 2 * a + heads * vdim
        o = fn(p[:, :a].view(t, heads, dim), p[:, a:2 * a].view(t, heads, dim),
               p[:, 2 * a:b].view(t, heads, vdim), p[:, b:b + rank], a2.to(dev), bias.to(dev),
               1.0 / 7.0, dim ** -0.5, st, loc.to(dev), _i32(lens).to(dev), _i32(slots).to(dev))
        return o, st

    want, got = run("cpu", ref.gla_scan), run(DEV, ops.gla_scan)
    _close(got[0], want[0], torch.float32, "outputs")
    _close(got[1], want[1], torch.float32, "state")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,vdim,rank", [
    (3, 6, 10, 5),                                          # scan and norm apart
    (2, 64, 64, 16), (1, 128, 128, 16), (2, 56, 72, 12), (1, 256, 24, 40), (4, 16, 304, 3),
    (2, 32, 8, 1), (2, 40, 200, 64), (1, 136, 64, 17), (1, 96, 120, 70),
])
@pytest.mark.parametrize("case", range(len(SEQS)))
def test_gla_gated(dtype, heads, dim, vdim, rank, case):
    rows, lens, slots = SEQS[case]
    g = torch.Generator().manual_seed(case)
    t, a, vw = sum(rows), heads * dim, heads * vdim
    loc = _i32([0] + torch.tensor(rows).cumsum(0).tolist())
    proj = torch.randn(t, (2 * a + 2 * vw + rank + 15) // 8 * 8, generator=g).to(dtype)
    a2 = torch.randn(rank, a, generator=g) / math.sqrt(rank)
    bias = torch.randn(a, generator=g)
    norm = torch.rand(vw, generator=g) + 0.5
    state = torch.randn(4, heads, vdim, dim, generator=g)
    b, c = 2 * a + vw, 2 * a + 2 * vw

    def run(dev, **kw):
        p, st = proj.to(dev), state.clone().to(dev)
        out = ops.gla_gated(p[:, :a].view(t, heads, dim), p[:, a:2 * a].view(t, heads, dim),
                            p[:, 2 * a:b].view(t, heads, vdim), p[:, b:c], p[:, c:c + rank],
                            a2.to(dev), bias.to(dev), 1.0 / 7.0, dim ** -0.5, norm.to(dev), 1e-5,
                            st, loc.to(dev), _i32(lens).to(dev), _i32(slots).to(dev), **kw)
        return out, st

    want = run("cpu")
    for general in (False, True):
        got = run(DEV, general=general)
        _close(got[0], want[0], dtype, f"outputs general={general}")
        _close(got[1], want[1], torch.float32, f"state general={general}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [5, 96, 1032])
def test_silu_mul_bias(dtype, ff):
    g = torch.Generator().manual_seed(ff)
    gu = torch.randn(9, 2 * ff, generator=g).to(dtype)
    bias = torch.randn(2 * ff, generator=g)
    for b in (bias, None):
        _close(ops.silu_mul_bias(gu.to(DEV), _dev(b)), ref.silu_mul_bias(gu, b), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cols,groups", [(120, 4), (30, 3), (4096, 32), (6144, 2)])
def test_silu_gate_after_the_norm(dtype, cols, groups):
    g = torch.Generator().manual_seed(cols)
    y = torch.randn(7, cols, generator=g)
    gate = torch.randn(7, cols, generator=g).to(dtype)
    w = torch.rand(cols, generator=g) + 0.5
    got = ops.gated_group_norm(y.to(DEV), gate.to(DEV), w.to(DEV), groups, 1e-5, False, dtype,
                               silu_after=True)
    _close(got, ref.gated_group_norm(y, gate, w, groups, 1e-5, False, dtype, True), dtype)
