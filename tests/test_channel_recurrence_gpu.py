"""HIP kernels of ``csrc/channel_recurrence.hip`` (selective scan per channel, block-diagonal gates, gated linear unit
recurrence) and what other files gained beside them (rotation in front of a head norm, a projection's bias inside the
convolution, a decay per head in the delta rule, SiLU behind the per-head norm, a scaled output norm, gated GELU),
against the plain PyTorch fp32 form of the same op (``ops/torch_ref.py``)."""
import pytest
import torch

pytestmark = pytest.mark.gpu

from vllm_distributed_amd.ops import torch_ref  # noqa: E402

DTYPES = [torch.bfloat16, torch.float16, torch.float32]


def _hip():
    from vllm_distributed_amd.ops import hip
    hip.load()
    return hip


def _close(a, b, dtype, scale=1.0):
    tol = {torch.float32: 3e-5, torch.float16: 2e-3, torch.bfloat16: 1.2e-2}[dtype]
    err = (a.float() - b.float()).abs().max().item()
    assert err <= tol * scale, err


def _i32(*v):
    return torch.tensor(list(v), dtype=torch.int32, device="cuda")


def _batch(lens, ctx):
    """Sequences that bring ``lens[i]`` rows as the last positions of ``ctx[i] + lens[i]`` tokens."""
    qsl = [0]
    for n in lens:
        qsl.append(qsl[-1] + n)
    pos, seq = [], []
    for i, (n, c) in enumerate(zip(lens, ctx)):
        pos += list(range(c, c + n))
        seq += [i] * n
    return _i32(*qsl), _i32(*[c + n for n, c in zip(lens, ctx)]), _i32(*pos), _i32(*seq)


# lengths on both sides of the chunks of both scans; sequences that start and that go on
MIXED = ([1, 16, 2, 129, 17, 1, 300], [4, 0, 9, 0, 3, 0, 11])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("c,n", [(64, 16), (70, 5), (129, 1), (96, 24), (40, 32), (200, 64), (33, 100), (48, 200), (4096, 16)])
def test_channel_scan(dtype, c, n):
    hip = _hip()
    g = torch.Generator(device="cuda").manual_seed(c * 1000 + n)

    def rnd(*s, lo=-1.0, hi=1.0):
        return lo + (hi - lo) * torch.rand(*s, device="cuda", generator=g)
    a_log, bias, skip = rnd(c, n, lo=-1.0, hi=2.5), rnd(c, lo=-4.0, hi=0.5), rnd(c)
    for lens, ctx in ((MIXED if c < 4096 else ([40, 3], [0, 5])), ([1] * 5, [3, 0, 7, 2, 0])):
        qsl, sls, _, _ = _batch(lens, ctx)
        t = sum(lens)
        u, gate = rnd(t, c + 8).to(dtype)[:, :c], rnd(t, c, lo=-3, hi=3).to(dtype)
        bc = rnd(t, 2 * n + 3).to(dtype)
        slots = torch.randperm(9, device="cuda", generator=g)[:len(lens)].int()
        st0 = rnd(9, c, n)
        for dt, b, d, gt in ((rnd(t, c, lo=-3, hi=3), bias, skip, gate), (rnd(t, c).to(dtype), None, None, None)):
            s1, s2 = st0.clone(), st0.clone()
            got = hip.channel_scan(u, dt, bc, n, a_log, b, d, gt, s1, slots, qsl, sls, max(lens))
            want = torch_ref.channel_scan(u.float(), dt, bc, n, a_log, b, d, gt, s2, slots, qsl, sls)
            top = max(1.0, want.abs().max().item())
            _close(got, want, dtype, top)
            _close(s1, s2, torch.float32, 2 * max(1.0, s2.abs().max().item()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("blocks,n", [(2, 32), (3, 64), (1, 128), (5, 24), (3, 7), (1, 1), (16, 256)])
def test_gated_unit(dtype, blocks, n):
    hip = _hip()
    w = blocks * n
    g = torch.Generator(device="cuda").manual_seed(w)

    def rnd(*s, lo=-1.0, hi=1.0):
        return lo + (hi - lo) * torch.rand(*s, device="cuda", generator=g)
    ra, ri = (rnd(blocks, n, n) * 3 * n ** -0.5).to(dtype), (rnd(blocks, n, n) * 3 * n ** -0.5).to(dtype)
    rb, ib, gb, rate = rnd(w), rnd(w), rnd(w), rnd(w, lo=1e-3, hi=3.0)
    for lens, ctx in ((MIXED if w < 4096 else ([200, 3], [0, 5])), ([1] * 7, [3, 0, 7, 2, 0, 1, 0]), ([3, 1, 4], [0, 2, 1])):
        qsl, sls, _, _ = _batch(lens, ctx)
        t = sum(lens)
        u, wide = rnd(t, w).to(dtype), rnd(t, w + 12, lo=-3, hi=3).to(dtype)
        a, drive = hip.block_gates(u, ra, rb, ri, ib, rate)
        a_ref, drive_ref = torch_ref.block_gates(u, ra, rb, ri, ib, rate)
        _close(a, a_ref, torch.float32, 1)
        _close(drive, drive_ref, torch.float32, 4)
        slots = torch.randperm(9, device="cuda", generator=g)[:len(lens)].int()
        st0 = rnd(9, w)
        for gate in (wide[:, :w], wide[:, 4:4 + w]):
            s1, s2 = st0.clone(), st0.clone()
            got = hip.gated_unit_step(u, ra, rb, ri, ib, rate, gate, gb, s1, slots, qsl, sls, max(lens))
            want = torch_ref.gated_unit_step(u.float(), ra, rb, ri, ib, rate, gate.float(), gb, s2, slots, qsl, sls)
            _close(got, want, dtype, max(1.0, want.abs().max().item()))
            _close(s1, s2, torch.float32, 4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("h,g,d,dv,half,inter", [(4, 2, 32, 48, 12, True), (3, 3, 20, 10, 7, True), (8, 1, 64, 64, 32, True),
                                                 (6, 2, 128, 16, 3, True), (2, 1, 48, 24, 0, True), (4, 4, 64, 8, 16, False),
                                                 (16, 16, 128, 128, 64, True)])
def test_rotate_norm_cache(dtype, h, g, d, dv, half, inter):
    hip = _hip()
    gen = torch.Generator(device="cuda").manual_seed(h * d)
    t, bs, blocks = 23, 16, 5
    x = torch.randn(t, h * d + g * (d + dv) + 8, device="cuda", generator=gen).to(dtype)
    freq = torch.rand(half, device="cuda", generator=gen) if half else None
    pos = torch.randint(0, 5000, (t,), device="cuda", generator=gen).int()
    slots = torch.randperm(bs * blocks, device="cuda", generator=gen)[:t].int()
    slots[3] = -1
    for qn, kn in ((None, None), (torch.rand(d, device="cuda") + 0.5, torch.rand(d, device="cuda") + 0.5)):
        caches = [torch.zeros(blocks, g, bs, d, device="cuda", dtype=dtype),
                  torch.zeros(blocks, g, bs // 8, dv, 8, device="cuda", dtype=dtype)]
        ref = [c.clone() for c in caches]
        got = hip.rotate_norm_cache(x, h, g, d, dv, freq, 1.17, inter, 1e-5, qn, kn, pos, *caches, slots)
        want = torch_ref.rotate_norm_cache(x, h, g, d, dv, freq, 1.17, inter, 1e-5, qn, kn, pos, *ref, slots)
        # (angles of thousands of radians: their fp32 rounding alone is a few 1e-4)
        _close(got, want, dtype, 20 if dtype == torch.float32 else 3)
        _close(caches[0], ref[0], dtype, 20 if dtype == torch.float32 else 3)
        assert torch.equal(caches[1], ref[1])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("c,taps", [(24, 4), (70, 3), (512, 2), (33, 1)])
def test_convolution_adds_the_projections_bias_to_inputs_that_exist(dtype, c, taps):
    hip = _hip()
    g = torch.Generator(device="cuda").manual_seed(c + taps)
    wide = torch.randn(40, c + 16, device="cuda", generator=g).to(dtype)
    w = (torch.randn(taps, c, device="cuda", generator=g) * 0.5).to(dtype)
    bias, ib = torch.randn(c, device="cuda", generator=g), torch.randn(c, device="cuda", generator=g)
    st0 = torch.randn(7, max(taps - 1, 1), c, device="cuda", generator=g).to(dtype)
    for lens, ctx, multi in (([1, 5, 1, 9, 2], [3, 0, 0, 7, 1], True), ([1, 1, 1], [5, 0, 2], False)):
        qsl, sls, pos, seq = _batch(lens, ctx)
        slots = _i32(4, 0, 2, 5, 1)[:len(lens)]
        x = wide[:sum(lens), 8:8 + c]
        s1, s2 = st0.clone(), st0.clone()
        got = hip.short_conv_act(x, c, w, s1, slots, qsl, sls, seq if multi else None, pos, True, multi, bias, False, ib)
        want = torch_ref.short_conv_act(x, c, w, s2, slots, qsl, sls, True, bias, False, ib)
        _close(got, want, dtype, 8)
        if taps > 1:
            assert torch.equal(s1, s2)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("h,g,dim,vdim", [(4, 2, 16, 24), (3, 3, 30, 7), (2, 1, 64, 80), (6, 2, 128, 128), (4, 4, 200, 32), (2, 2, 1, 5)])
def test_delta_rule_with_a_decay_per_head(dtype, h, g, dim, vdim):
    hip = _hip()
    gen = torch.Generator(device="cuda").manual_seed(h * dim)
    for lens, ctx in (([1, 9, 2, 70, 8], [4, 0, 9, 3, 0]), ([1] * 5, [3, 0, 7, 2, 0])):
        qsl, sls, _, _ = _batch(lens, ctx)
        t = sum(lens)
        x = torch.randn(t, 2 * g * dim + h * vdim + 4, device="cuda", generator=gen).to(dtype)
        ba = torch.randn(t, 2 * h, device="cuda", generator=gen).to(dtype)
        a_log, dtb = torch.randn(h, device="cuda", generator=gen) - 1, torch.randn(h, device="cuda", generator=gen)
        slots = torch.randperm(9, device="cuda", generator=gen)[:len(lens)].int()
        st0 = torch.randn(9, h, dim, vdim, device="cuda", generator=gen)
        for parts in (0, 4, 8, 16):
            s1, s2 = st0.clone(), st0.clone()
            got = hip.gated_delta_rule(x, h, g, dim, vdim, ba[:, :h], ba[:, h:], dtb, a_log, s1, slots, qsl, sls, 1e-6,
                                       max(lens), parts)
            want = torch_ref.gated_delta_rule(x, h, g, dim, vdim, ba[:, :h], ba[:, h:], dtb, a_log, s2, slots, qsl, sls)
            _close(got, want, torch.float32, 2 * max(1.0, want.abs().max().item()))
            _close(s1, s2, torch.float32, 4 * max(1.0, s2.abs().max().item()))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,group", [(96, 24), (256, 64), (120, 120), (512, 0), (128, 128)])
def test_silu_behind_the_norm(dtype, n, group):
    hip = _hip()
    g = torch.Generator(device="cuda").manual_seed(n)
    o = torch.randn(13, n, device="cuda", generator=g)
    w = torch.rand(group or n, device="cuda", generator=g) + 0.5
    gate = (3 * torch.randn(13, n + 8, device="cuda", generator=g)).to(dtype)[:, 8:]
    buf = torch.zeros(13, n + 16, dtype=dtype, device="cuda")
    for silu in (True, False):
        want = torch_ref.gated_rms_norm(o, w, gate, 1e-5, dtype, group, 0.7, None, silu)
        _close(hip.gated_rms_norm(o, w, gate, 1e-5, dtype, group, 0.7, None, silu), want, dtype, 12)
        _close(hip.gated_rms_norm(o, w, gate, 1e-5, dtype, group, 0.7, buf[:, 8:8 + n], silu), want, dtype, 12)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("h", [100, 192, 2048])
def test_scaled_output_norm(dtype, h):
    hip = _hip()
    g = torch.Generator(device="cuda").manual_seed(h)
    y, x0 = torch.randn(9, h, device="cuda", generator=g).to(dtype), torch.randn(9, h, device="cuda", generator=g)
    pw, nw = torch.rand(h, device="cuda", generator=g) + 0.5, torch.rand(h, device="cuda", generator=g) + 0.5
    for normed in (True, False):
        x1, x2 = x0.clone(), x0.clone()
        got = hip.norm_add_norm(y, pw, x1, nw if normed else None, 1e-5, dtype, 0.0, normed, 0.37)
        want = torch_ref.norm_add_norm(y, pw, x2, nw if normed else None, 1e-5, dtype, 0.0, normed, 0.37)
        _close(x1, x2, torch.float32)
        _close(got, want, dtype, 4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("f", [24, 77, 1024])
def test_gelu_and_mul(dtype, f):
    hip = _hip()
    g = torch.Generator(device="cuda").manual_seed(f)
    x = 2 * torch.randn(11, 2 * f + 8, device="cuda", generator=g)
    for v in (x[:, :2 * f].to(dtype), x.to(dtype)[:, 8:]):
        for tanh in (True, False):
            want = torch_ref.gelu_and_mul(v, tanh)
            _close(hip.gelu_and_mul(v, tanh), want, dtype, max(1.0, want.abs().max().item()))


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float16])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5])
def test_convolution_over_many_rows(dtype, taps):
    """Enough rows that a thread walks several of them: sequences of every short length in between, of which some start
    and some go on, against the plain form."""
    hip = _hip()
    c = 64
    g = torch.Generator(device="cuda").manual_seed(taps)
    lens = [1, 2, 1, 3, 4, 5, 1, 1, 7, 8, 9, 31, 2, 600, 1, 3600, 1, 15]
    ctx = [5, 0, 0, 1, 2, 3, 1, 2, 0, 9, 1, 0, 3, 2, 0, 0, 4, 1]
    qsl, sls, pos, seq = _batch(lens, ctx)
    t = sum(lens)
    x = torch.randn(t, c + 8, device="cuda", generator=g).to(dtype)[:, 8:]
    w = (torch.randn(taps, c, device="cuda", generator=g) * 0.5).to(dtype)
    bias, ib = torch.randn(c, device="cuda", generator=g), torch.randn(c, device="cuda", generator=g)
    slots = torch.randperm(20, device="cuda", generator=g)[:len(lens)].int()
    st0 = torch.randn(20, max(taps - 1, 1), c, device="cuda", generator=g).to(dtype)
    for silu, b, res, inb in ((True, bias, False, ib), (False, None, True, None)):
        s1, s2 = st0.clone(), st0.clone()
        got = hip.short_conv_act(x, c, w, s1, slots, qsl, sls, seq, pos, silu, True, b, res, inb)
        want = torch_ref.short_conv_act(x, c, w, s2, slots, qsl, sls, silu, b, res, inb)
        _close(got, want, dtype, 8)
        if taps > 1:
            for i, (n, k) in enumerate(zip(lens, ctx)):            # (rows in front of a sequence's start are never read)
                seen = min(n + k, taps - 1)
                assert torch.equal(s1[slots[i], taps - 1 - seen:], s2[slots[i], taps - 1 - seen:]), i
