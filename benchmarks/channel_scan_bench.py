"""Per-channel recurrences alone: ``channel_scan`` (selective scan, N states per channel), ``block_gates`` and
``gated_unit_scan`` / the one-launch decode step, at prompt and decode shapes.  Microseconds and the bytes that have to
move per second.

    python benchmarks/channel_scan_bench.py
"""
import os
import sys

import torch

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))

from vllm_distributed_amd.ops import hip  # noqa: E402


def timed(fn, n=20):
    for _ in range(3):
        fn()
    torch.cuda.synchronize()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    for _ in range(n):
        fn()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) * 1e3 / n


def main() -> None:
    hip.load()
    dev, bf = "cuda", torch.bfloat16
    i32 = dict(dtype=torch.int32, device=dev)
    for seqs, rows, c, n in ((8, 1024, 4096, 16), (4, 2048, 4096, 16), (1, 8192, 4096, 16), (8, 1024, 4096, 64), (128, 1, 4096, 16),
                             (128, 1, 4096, 64)):
        t = seqs * rows
        u, z = torch.randn(t, c, device=dev).to(bf), torch.randn(t, c, device=dev).to(bf)
        dt, bc = torch.randn(t, c, device=dev) - 3, torch.randn(t, 2 * n, device=dev).to(bf)
        al, db, sk = torch.rand(c, n, device=dev), torch.zeros(c, device=dev), torch.ones(c, device=dev)
        st, slots = torch.zeros(seqs, c, n, device=dev), torch.arange(seqs, **i32)
        qsl, sl = torch.arange(seqs + 1, **i32) * rows, torch.full((seqs,), rows + 1, **i32)
        us = timed(lambda: hip.channel_scan(u, dt, bc, n, al, db, sk, z, st, slots, qsl, sl, rows))
        gb = (t * c * 10 + 2 * seqs * c * n * 4) / 1e9
        print(f"channel_scan    {seqs:4d} x {rows:5d} rows, {c} channels, {n:3d} states: {us:8.1f} us  {gb / us * 1e3:6.2f} TB/s", flush=True)
    for seqs, rows, w, blk in ((8, 1024, 2048, 128), (1, 8192, 2048, 128), (8, 1024, 4096, 256), (128, 1, 2048, 128), (128, 1, 4096, 256)):
        t = seqs * rows
        u, y = torch.randn(t, w, device=dev).to(bf), torch.randn(t, w, device=dev).to(bf)
        ra, ri = ((torch.randn(w // blk, blk, blk, device=dev) * blk ** -0.5).to(bf) for _ in range(2))
        rb, rate = torch.zeros(w, device=dev), torch.rand(w, device=dev)
        st, slots = torch.zeros(seqs, w, device=dev), torch.arange(seqs, **i32)
        qsl, sl = torch.arange(seqs + 1, **i32) * rows, torch.full((seqs,), rows + 1, **i32)
        if rows == 1:
            us = timed(lambda: hip.gated_unit_step(u, ra, rb, ri, rb, rate, y, rb, st, slots, qsl, sl, 1))
            print(f"gated_unit_step {seqs:4d} x     1 rows, {w} channels in blocks of {blk}: {us:8.1f} us", flush=True)
            continue
        us = timed(lambda: hip.block_gates(u, ra, rb, ri, rb, rate))
        print(f"block_gates     {seqs:4d} x {rows:5d} rows, {w} channels in blocks of {blk}: {us:8.1f} us  {t * w * 10 / us / 1e6:6.2f} TB/s", flush=True)
        a, d = hip.block_gates(u, ra, rb, ri, rb, rate)
        us = timed(lambda: hip.gated_unit_scan(a, d, y, rb, st, slots, qsl, sl, rows))
        print(f"gated_unit_scan {seqs:4d} x {rows:5d} rows, {w} channels:                 {us:8.1f} us  {t * w * 12 / us / 1e6:6.2f} TB/s", flush=True)


if __name__ == "__main__":
    main()
