"""HIP kernels of gated linear attention (``low_rank_decay``, ``channel_decay_attention``), of experts that weigh their input
(``weighted_relu_squared``, ``moe_combine`` without weights), and the arguments that ``rotate_norm_cache`` (biases, no head
norm, queries only) and ``residual_rms`` (two normed outputs beside a plain one) gained, against the plain PyTorch fp32 form
of the same op (``ops/torch_ref.py``)."""
import pytest
import torch

pytestmark = pytest.mark.gpu

from vllm_distributed_amd.ops import torch_ref  # noqa: E402


def _hip():
    from vllm_distributed_amd.ops import hip
    hip.load()
    return hip


def _close(a, b, tol):
    err = (a.float() - b.float()).abs().max().item()
    assert err <= tol * max(1.0, b.float().abs().max().item()), err


def _i32(*v):
    return torch.tensor(list(v), dtype=torch.int32, device="cuda")


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("rows,rank,channels,tau", [(1, 16, 96, 16.0), (5, 8, 300, 1.0), (1100, 16, 256, 4.0), (37, 5, 31, 16.0),
                                                    (1030, 40, 70, 2.5), (3, 72, 513, 8.0), (2, 1, 1, 3.0)])
def test_low_rank_decay(dtype, rows, rank, channels, tau):
    hip = _hip()
    g = torch.Generator(device="cuda").manual_seed(rows + rank)
    wide = torch.randn(rows, rank + 8, device="cuda", generator=g).to(dtype)
    a = wide[:, 8:]
    w = (torch.randn(channels, rank, device="cuda", generator=g) * rank ** -0.5 * 3).to(dtype)
    bias = torch.randn(channels, device="cuda", generator=g) * 4
    got = hip.low_rank_decay(a, w, bias, tau)
    z = a.double() @ w.double().t() + bias.double()
    want = torch.exp(torch.nn.functional.logsigmoid(z) / tau)
    # what the recurrence multiplies up over time is the distance from one: it is held to its own size
    err = ((got.double() - want).abs() / (1e-7 + 3e-6 * (1.0 - want) + 3e-6 * want * (want < 0.9))).max().item()
    assert got.dtype == torch.float32 and err < 4.0, err
    _close(hip.low_rank_decay(a, w, None, tau), torch_ref.low_rank_decay(a, w, None, tau), 2e-6)


def _recurrence(heads, dim, vdim, t_sizes, starts, dtype, seed, extra=11):
    g = torch.Generator(device="cuda").manual_seed(seed)
    t = sum(t_sizes)
    x = torch.randn(t, heads * (2 * dim + vdim) + extra, device="cuda", generator=g).to(dtype)
    alpha = torch.rand(t, heads * dim, device="cuda", generator=g) ** 0.2
    state = torch.randn(len(t_sizes) + 2, heads, dim, vdim, device="cuda", generator=g)
    qsl = _i32(*[sum(t_sizes[:i]) for i in range(len(t_sizes) + 1)])
    lens = _i32(*[s + n for s, n in zip(starts, t_sizes)])
    slots = _i32(*range(len(t_sizes), 0, -1))
    return x, alpha, state, slots, qsl, lens


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("heads,dim,vdim", [(2, 16, 24), (1, 128, 128), (3, 48, 32), (2, 64, 64), (2, 20, 7), (1, 200, 130),
                                            (1, 256, 65), (2, 1, 1), (1, 33, 63)])
def test_channel_decay_attention(dtype, heads, dim, vdim):
    """Fresh and continued sequences of unequal length, both launch shapes, strided rows, key sizes on both sides of every
    tiling, odd value sizes."""
    hip = _hip()
    for t_sizes, starts in (([37, 1, 8, 2], [0, 5, 3, 0]), ([1, 1, 1, 1, 1], [4, 0, 9, 1, 700]), ([2, 1], [3, 0]), ([129], [0])):
        x, alpha, state, slots, qsl, lens = _recurrence(heads, dim, vdim, t_sizes, starts, dtype, heads * dim + vdim)
        for silu in (False, True):
            s1, s2 = state.clone(), state.clone()
            got = hip.decay_linear_attention(x, heads, dim, vdim, alpha, s1, slots, qsl, lens, silu, max(t_sizes), 0.3)
            want = torch_ref.decay_linear_attention(x, heads, dim, vdim, alpha, s2, slots, qsl, lens, silu, 0.3)
            _close(got, want, 1e-5)
            _close(s1, s2, 1e-5)
            untouched = [i for i in range(state.shape[0]) if i not in slots.tolist()]
            assert torch.equal(s1[untouched], state[untouched])
            s1 = state.clone()                         # (the launch for rows of unknown length)
            _close(hip.decay_linear_attention(x, heads, dim, vdim, alpha, s1, slots, qsl, lens, silu, 0, 0.3), want, 1e-5)


@pytest.mark.parametrize("heads,dim,vdim", [(8, 20, 70), (8, 64, 64), (4, 128, 128), (8, 130, 32)])
def test_many_sequences_in_one_launch(heads, dim, vdim):
    """Enough workgroups for the launch shape of crowded prompt steps: portions of one to nine rows."""
    hip = _hip()
    sizes = [1 + (7 * i) % 9 for i in range(66)]
    starts = [(5 * i) % 4 for i in range(66)]
    x, alpha, state, slots, qsl, lens = _recurrence(heads, dim, vdim, sizes, starts, torch.bfloat16, dim)
    s1, s2 = state.clone(), state.clone()
    got = hip.decay_linear_attention(x, heads, dim, vdim, alpha, s1, slots, qsl, lens, False, 9, 0.5)
    want = torch_ref.decay_linear_attention(x, heads, dim, vdim, alpha, s2, slots, qsl, lens, False, 0.5)
    _close(got, want, 1e-5)
    _close(s1, s2, 1e-5)


@pytest.mark.parametrize("heads,dim,vdim", [(2, 64, 64), (1, 128, 128), (3, 24, 40)])
def test_portions_leave_the_state_a_whole_pass_leaves(heads, dim, vdim):
    hip = _hip()
    x, alpha, state, slots, qsl, lens = _recurrence(heads, dim, vdim, [203], [0], torch.bfloat16, 5)
    s1, s2 = state.clone(), state.clone()
    whole = hip.decay_linear_attention(x, heads, dim, vdim, alpha, s1, slots, qsl, lens, False, 203, 1.0)
    out, at = [], 0
    for n in (1, 2, 7, 8, 9, 1, 1, 64, 17, 2, 91):
        out.append(hip.decay_linear_attention(x[at:at + n], heads, dim, vdim, alpha[at:at + n], s2, slots, _i32(0, n),
                                              _i32(at + n), False, n, 1.0))
        at += n
    assert at == 203
    _close(torch.cat(out), whole, 3e-6)
    _close(s2, s1, 3e-6)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("rows,f", [(1, 8), (9, 128), (40, 1408), (7, 99)])
def test_weighted_relu_squared(dtype, rows, f):
    hip = _hip()
    g = torch.Generator(device="cuda").manual_seed(f)
    wide = (torch.randn(rows + 3, f + 8, device="cuda", generator=g) * 2).to(dtype)
    inv = torch.randperm(rows + 3, device="cuda", generator=g)[:rows].to(torch.int32)
    topw = torch.rand(rows, device="cuda", generator=g) + 0.05
    got = hip.weighted_relu_squared(wide[:, :f], topw, inv)
    want = torch_ref.weighted_relu_squared(wide[:, :f], topw, inv)
    _close(got[inv.long()], want[inv.long()], 1e-6 if dtype == torch.float32 else 8e-3)


def test_combine_without_weights():
    hip = _hip()
    g = torch.Generator(device="cuda").manual_seed(3)
    t, k, h = 13, 3, 256
    y = torch.randn(t * k, h, device="cuda", generator=g).to(torch.bfloat16)
    topi = torch.randint(0, 8, (t, k), device="cuda", generator=g, dtype=torch.int32)
    inv = torch.randperm(t * k, device="cuda", generator=g).to(torch.int32)
    want = y[inv.long()].float().view(t, k, h).sum(1)
    _close(hip.moe_combine(y, None, topi, inv), want, 8e-3)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("h", [22, 192, 1000, 4096])
def test_two_normed_outputs_and_a_plain_one(dtype, h):
    hip = _hip()
    g = torch.Generator(device="cuda").manual_seed(h)
    x = torch.randn(7, h, device="cuda", generator=g) * 3
    w, w1, w2 = (torch.rand(h, device="cuda", generator=g) + 0.3 for _ in range(3))
    wide = torch.randn(7, 3 * h + 8, device="cuda", generator=g).to(dtype) * torch.tensor(
        [0.001, 0.1, 1, 3, 10, 100, 1], device="cuda").view(-1, 1).to(dtype)
    y, z, f = wide[:, :h], wide[:, h:2 * h], wide[:, 2 * h + 8:]
    for plain in (f, None):
        for second in ((z, w2), None):
            for normed in (True, False):
                r1, r2 = x.clone(), x.clone()
                o1 = hip.norm_add_norm(y, w1, r1, w, 1e-6, dtype, 0.0, normed, 0.5, second, plain)
                o2 = torch_ref.norm_add_norm(y, w1, r2, w, 1e-6, dtype, 0.0, normed, 0.5, second, plain)
                _close(r1, r2, 3e-6)
                _close(o1, o2, 1e-5 if dtype == torch.float32 else 8e-3)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("heads,groups,dim,vdim", [(4, 2, 64, 64), (3, 1, 20, 12), (2, 2, 48, 80), (8, 2, 128, 32), (1, 1, 8, 8)])
def test_heads_with_biases_with_and_without_norm(dtype, heads, groups, dim, vdim):
    hip = _hip()
    g = torch.Generator(device="cuda").manual_seed(dim)
    t, bs, nblk = 41, 16, 6
    c = (heads + groups) * dim + groups * vdim
    x = torch.randn(t, c + 8, device="cuda", generator=g).to(dtype)
    bias = torch.randn(c, device="cuda", generator=g)
    qn, kn = torch.rand(dim, device="cuda", generator=g) + 0.5, torch.rand(dim, device="cuda", generator=g) + 0.5
    pos = torch.arange(t, dtype=torch.int32, device="cuda")
    slot = torch.randperm(nblk * bs, device="cuda", generator=g)[:t].to(torch.int32)
    slot[3] = -1
    tol = 2e-6 if dtype == torch.float32 else 8e-3
    for b in (bias, None):
        for normed in (True, False):
            caches = [(torch.full((nblk, groups, bs, dim), 5.0, device="cuda", dtype=dtype),
                       torch.full((nblk, groups, bs // 8, vdim, 8), 5.0, device="cuda", dtype=dtype)) for _ in range(2)]
            args = (x, heads, groups, dim, vdim, None, 1.0, False, 1e-6, qn if normed else None, kn if normed else None, pos)
            q1 = hip.rotate_norm_cache(*args, *caches[0], slot, normed, b)
            q2 = torch_ref.rotate_norm_cache(*args, *caches[1], slot, normed, b)
            _close(q1, q2, tol)
            for a1, a2 in zip(*caches):
                _close(a1, a2, tol)
            qx = torch.cat([x[:, :heads * dim], x[:, -8:]], 1)             # queries only: nothing is cached
            args = (qx, heads, 0, dim, vdim, None, 1.0, False, 1e-6, qn if normed else None, None, pos)
            qb = None if b is None else b[:heads * dim].contiguous()
            _close(hip.rotate_norm_cache(*args, None, None, None, normed, qb), q2, tol)
