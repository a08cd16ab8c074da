"""Time gated linear attention (a decay per key channel) beside the gated delta rule and linear attention with a decay per
head at equal head sizes - prompt portions and decoded rows - and the low-rank decays, the head preparation and the
residual launch of a layer with two normed outputs.  ``python benchmarks/channel_decay_bench.py`` on a GPU box."""
import os
import sys

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
import torch  # noqa: E402

from vllm_distributed_amd.ops import hip  # noqa: E402


def timed(fn, reps=20):
    for _ in range(3):
        fn()
    torch.cuda.synchronize()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    for _ in range(reps):
        fn()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) * 1e3 / reps


def main():
    hip.load()
    dev, dt = "cuda", torch.bfloat16
    for heads, dim, vdim in ((16, 128, 128), (32, 64, 64)):
        for seqs, rows in ((1, 8192), (4, 2048), (8, 1024), (16, 512), (64, 128), (128, 1), (256, 1)):
            t = seqs * rows
            x = (torch.randn(t, 2 * heads * dim + heads * vdim, device=dev) * 0.5).to(dt)
            alpha = torch.rand(t, heads * dim, device=dev)
            decay = torch.full((heads,), 0.97, device=dev)
            beta, dtr = torch.randn(t, heads, device=dev).to(dt), torch.randn(t, heads * dim, device=dev).to(dt)
            dt_bias, a_log = torch.zeros(heads * dim, device=dev), torch.zeros(heads, device=dev) - 1.0
            state = torch.zeros(seqs + 1, heads, dim, vdim, device=dev)
            qsl = torch.arange(0, t + 1, rows, dtype=torch.int32, device=dev)
            lens = torch.full((seqs,), rows + 5, dtype=torch.int32, device=dev)
            slots = torch.arange(seqs, dtype=torch.int32, device=dev)
            a = timed(lambda: hip.decay_linear_attention(x, heads, dim, vdim, alpha, state, slots, qsl, lens, False, rows))
            b = timed(lambda: hip.decay_linear_attention(x, heads, dim, vdim, decay, state, slots, qsl, lens, False, rows))
            c = timed(lambda: hip.gated_delta_rule(x, heads, heads, dim, vdim, beta, dtr, dt_bias, a_log, state, slots, qsl,
                                                   lens, 1e-6, rows))
            print(f"H{heads} d{dim} v{vdim} {seqs:3d} x {rows:4d} rows:  decay per channel {a:8.1f} us   decay per head "
                  f"{b:8.1f} us   delta rule with its preparation {c:8.1f} us", flush=True)
    for t in (8192, 128):
        w = 2048
        a1, a2 = torch.randn(t, 16, device=dev).to(dt), torch.randn(w, 16, device=dev).to(dt)
        bias = torch.randn(w, device=dev)
        us = timed(lambda: hip.low_rank_decay(a1, a2, bias, 16.0))
        print(f"low_rank_decay {t} x {w}, rank 16: {us:8.1f} us", flush=True)
        x = torch.randn(t, w, device=dev)
        y, z, f = (torch.randn(t, w, device=dev).to(dt) for _ in range(3))
        g = torch.ones(w, device=dev)
        us = timed(lambda: hip.norm_add_norm(y, g, x, g, 1e-6, dt, 0.0, True, 0.5, (z, g), f))
        print(f"residual_rms {t} x {w}, two normed outputs and a plain one: {us:8.1f} us", flush=True)
        heads, groups, dim = 16, 4, 128
        qkv = torch.randn(t, (heads + 2 * groups) * dim, device=dev).to(dt)
        b = torch.randn((heads + 2 * groups) * dim, device=dev)
        n = torch.ones(dim, device=dev)
        pos = torch.arange(t, dtype=torch.int32, device=dev)
        kc = torch.zeros(t // 64 + 1, groups, 64, dim, device=dev, dtype=dt)
        vc = torch.zeros(t // 64 + 1, groups, 8, dim, 8, device=dev, dtype=dt)
        us = timed(lambda: hip.rotate_norm_cache(qkv, heads, groups, dim, dim, None, 1.0, False, 1e-6, n, n, pos, kc, vc, pos,
                                                 True, b))
        print(f"head preparation {t} rows, {heads} + {groups} heads of {dim}, biases, norms, cache: {us:8.1f} us", flush=True)


if __name__ == "__main__":
    main()
