"""Vebusun configurations drawn at random with fixed seeds (widths, the order and kinds of layers, loops, head counts,
key, value and state sizes, inner ranks, taps, rotated dimensions, windows, first tokens, caps, decays, factors,
layers without feed-forward, constants present or absent), each stepped through a random mixed schedule on a pool at
the schedule's peak with four slots against the plain implementation. A row is held to the dtype's bound, or to three
times what rounding (float32 throughout; what the sublayers read in bfloat16) does to the plain statement itself at that
row where that is more: the first tokens of a recurrence hang on the sign of one dot product."""
import random

import pytest
import torch

import plain_vebusun as plain
from conftest import prompt_tokens
from gpu_helpers import make_engine, mixed_schedule, peak_pages
from tolerances import bound
from vebusun_models import delta, layer, left, parallel, right, runs_of, write_model

pytestmark = pytest.mark.gpu


def draw_config(seed):
    rng = random.Random(seed)
    width = rng.choice([32, 40, 60, 64, 96, 128, 160, 256])
    layers = []
    for _ in range(rng.randint(1, 5)):
        if rng.random() < 0.5:
            kv = rng.choice([1, 2, 3])
            mixer = delta(kv * rng.choice([1, 2, 3]), kv, rng.choice([8, 12, 16, 32, 64, 128, 160]),
                          rng.choice([8, 10, 16, 32, 64]), rng.choice([1, 2, 3, 4]))
        else:
            kv = rng.choice([1, 2, 4])
            dim = rng.choice([8, 16, 32, 48, 64, 96, 128]) if rng.random() < 0.8 else rng.choice([12, 24, 40])
            vdim = dim if rng.random() < 0.6 else rng.choice([8, 12, 16, 20, 32, 64])
            window = rng.choice([None, 1, 2, 7, 16, 33, 64, 100])
            a = left(kv * rng.choice([1, 2, 4]), kv, dim, vdim,
                     # mild scores: scores spread much wider than 1 / sqrt(dim) turn bfloat16's rounding of q and k
                     # into weight shifts of several percent whichever kernel runs: conditioning, no fault
                     scale=rng.choice([1.0, 0.5, 1.0 / 3.0]) / dim ** 0.5, softcap=rng.choice([None, 2.0, 10.0, 50.0]),
                     window=window, keep=rng.choice([None, 0, 1, 3, 16, 40, 70]) if window else None,
                     rot=rng.choice([None, dim, dim // 2 - (dim // 2) % 2, 2]) or None, base=rng.choice([100.0, 10000.0, 1e6]))
            heads = rng.choice([1, 2, 3, 4])
            b = right(heads, rng.choice([8, 16, 32, 64, 96]), rng.choice([8, 16, 24, 64]),
                      [rng.choice([1.0, 0.5, 0.9, 0.97, 0.999]) for _ in range(heads)])
            mixer = parallel(a, b, rng.choice([1.0, 0.6, 1.4]), rng.choice([1.0, 0.5, 1.2]))
        layers.append(layer(mixer, rng.choice([None, 8, 20, 32, 100, 256])))
    cfg = dict(architecture="Vebusun", vocab=rng.choice([50, 97, 300, 500]), width=width,
               norm=dict(eps=rng.choice([1e-6, 1e-5, 1e-3])), layers=layers)
    if rng.random() < 0.8:
        cfg["residual_mult"] = rng.choice([0.25, 0.5])
    if rng.random() < 0.7:
        cfg["embedding"] = dict(scale=rng.choice([0.5, 2.0, 3.3]))
    if rng.random() < 0.6:
        start = rng.randint(0, len(layers) - 1)
        cfg["loop"] = dict(start=start, stop=rng.randint(start, len(layers)), times=rng.choice([1, 2, 2, 3]))
    return cfg, (rng.choice([1, 4, 9, 16, 32]), rng.choice([1, 6, 8, 20]))


@pytest.mark.parametrize("seed", range(24))
def test_random_configuration_through_a_mixed_schedule(seed, tmp_path):
    from imparo_amd.engine import StepEntry
    cfg, ranks = draw_config(3000 + seed)
    d = write_model(cfg, seed, str(tmp_path / "m"), ranks=ranks)
    rng = random.Random(seed)
    lengths = [rng.choice([1, 2, 5, 30, 70, 130]) for _ in range(5)]
    prompts = [prompt_tokens(cfg["vocab"], n, 40 + i) for i, n in enumerate(lengths)]
    steps = mixed_schedule(rng, lengths, max_live=4, sizes=(1, 1, 1, 2, 2, 3, 5, 9, 16, 40, 70))
    page = rng.choice([8, 16, 64])
    ref, single = plain.PlainVebusun(d), plain.PlainVebusun(d, torch.float32)
    low = lambda p, dtype: single.logits(p) if dtype == "float32" else ref.logits(p, inputs_as=torch.bfloat16)
    all_ref = torch.cat([ref.logits(p) for p in prompts])
    scale = float(all_ref.abs().max())
    for dtype in ("float32", "bfloat16"):
        eng = make_engine(d, dtype, page_size=page, max_tokens=peak_pages(steps, page) * page, max_requests=4)
        got = {i: [] for i in range(len(lengths))}
        for entries, ends in steps:
            out = eng.step([StepEntry(rid, prompts[rid][lo:hi], list(range(hi - lo))) for rid, lo, hi in entries]).cpu()
            at = 0
            for rid, lo, hi in entries:
                got[rid].append(out[at:at + hi - lo])
                at += hi - lo
            for rid in ends:
                eng.release(rid)
        all_got = torch.cat([torch.cat(got[i]) for i in range(len(lengths))]).float()
        assert torch.isfinite(all_got).all(), f"seed {seed} {dtype}"
        row_err = (all_got - all_ref).abs().max(dim=-1).values / scale
        noise = (torch.cat([low(p, dtype) for p in prompts]) - all_ref).abs().max(dim=-1).values / scale
        allowed = torch.maximum(torch.full_like(row_err, bound(dtype, runs_of(cfg))), 3.0 * noise)
        bad = (row_err > allowed).nonzero()
        assert bad.numel() == 0, (f"seed {seed} {dtype}: row {int(bad[0])} of {row_err.shape[0]} misses by "
                                  f"{float(row_err[bad[0]]):.3g}, allowed {float(allowed[bad[0]]):.3g}; {bad.numel()} rows; {cfg}")
        eng.cache.check()
