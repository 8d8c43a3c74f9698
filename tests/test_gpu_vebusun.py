"""The Vebusun design in the engine against the plain implementation (tests/plain_vebusun.py): each mechanism's
kernels alone, whole prompts, stepwise decoding, portions down to two tokens, mixed batches on a pool at the
schedule's peak with slots used again, long decoding past every window, first tokens, other sizes and constants, keys
far away and just inside and just outside a window and the first tokens that stay, each singled out by one score,
generation through the entry point and the trace replay program."""
import copy
import json
import math
import os
import random
import subprocess

import numpy as np
import pytest
import torch

import plain_vebusun as plain
from conftest import ROOT, prompt_tokens
from gpu_helpers import hand_context, make_engine, mixed_schedule, peak_pages, step_all
from tolerances import bound, check_logits
from vebusun_models import CONFIGS, RANKS, random_weights, runs_of, write_model

pytestmark = pytest.mark.gpu
DEV = "cuda:0"


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    return {name: write_model(cfg, seed, str(tmp_path_factory.mktemp(f"vebusun_{name}")), ranks=RANKS[name])
            for name, (cfg, seed) in CONFIGS.items()}


class Yardstick:
    """The plain implementation in float64, and per row how far rounding moves the plain statement itself: in float32
    throughout, and with what every sublayer reads rounded to bfloat16. The first tokens of a recurrence, and heads
    whose result happens to be small, are badly conditioned (a norm stretches what is left to unit size), so a run
    is held to the general bound or to three times that rounding's effect at the row, whichever is larger."""

    def __init__(self, model_dir):
        self.exact, self.single = plain.PlainVebusun(model_dir), plain.PlainVebusun(model_dir, torch.float32)
        self._memo, self._noise = {}, {}

    def logits(self, tokens, order=None):
        key = tuple(tokens)
        if key not in self._memo:
            self._memo[key] = self.exact.logits(tokens)
        return self._memo[key]

    def noise(self, tokens, dtype="float32"):
        key = (tuple(tokens), dtype)
        if key not in self._noise:
            ref = self.logits(tokens)
            low = self.single.logits(tokens) if dtype == "float32" else self.exact.logits(tokens, inputs_as=torch.bfloat16)
            self._noise[key] = (low - ref).abs().max(dim=-1).values / float(ref.abs().max())
        return self._noise[key]

    def greedy(self, prompt, n):
        return self.exact.greedy(prompt, n)


@pytest.fixture(scope="module")
def plains(dirs):
    return {name: Yardstick(d) for name, d in dirs.items()}


def runs(name):
    return runs_of(CONFIGS[name][0])


def vocab(name):
    return CONFIGS[name][0]["vocab"]


def check(got, ref, what, rel, noise):
    """Every row within `rel` of the largest reference logit, or within three times its `noise` (Yardstick)."""
    got, ref = got.float().cpu(), ref.float().cpu()
    assert got.shape == ref.shape and torch.isfinite(got).all(), what
    row_err = (got - ref).abs().max(dim=-1).values / float(ref.abs().max())
    allowed = torch.maximum(torch.full_like(row_err, rel), 3.0 * noise[:row_err.shape[0]].float())
    over = (row_err > allowed).nonzero().flatten()
    assert over.numel() == 0, (f"{what}: row {int(over[0])} misses by {float(row_err[over[0]]):.3g}, allowed "
                               f"{float(allowed[over[0]]):.3g}; {over.numel()} of {got.shape[0]} rows")


def dev(t, dtype=torch.float32):
    return t.to(device=DEV, dtype=dtype).contiguous()


def i32(a):
    return torch.tensor(np.asarray(a, dtype=np.int32), device=DEV)


def near(got, want, rel, what=""):
    got, want = got.double().cpu(), want.double().cpu()
    assert got.shape == want.shape and torch.isfinite(got).all(), what
    assert float((got - want).abs().max()) <= rel * max(float(want.abs().max()), 1e-30), \
        f"{what}: {float((got - want).abs().max()):.3e} against {rel * float(want.abs().max()):.3e}"


# ------------------------------------------------------------------ the norm
@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,E", [(5, 64), (3, 37), (70, 1024), (1, 1), (300, 260)])
def test_norm_without_a_statistic(T, E, out_dtype):
    """tanh(alpha v) w + b with no delta, one, one in slices, two; written back or for chosen rows only."""
    from imparo_amd.kernels import ops
    g = torch.Generator().manual_seed(T + E)
    x, w, b = 2.0 * torch.randn(T, E, generator=g), torch.rand(E, generator=g) + 0.5, torch.randn(E, generator=g)
    one, many, more = torch.randn(T, E, generator=g), torch.randn(6, T, E, generator=g), torch.randn(2, T, E, generator=g)
    alpha = 0.63
    rel = 2e-6 if out_dtype == torch.float32 else 5e-3
    for deltas in ((), (one,), (many,), (one, many), (more, one)):
        v = x.double() + sum((d.double().sum(0) if d.dim() == 3 else d.double()) for d in deltas)
        want = torch.tanh(alpha * v) * w + b
        stream, out = dev(x), torch.empty(T, E, dtype=out_dtype, device=DEV)
        on = tuple(dev(d) for d in deltas)
        ops.dynamic_tanh(stream, alpha, dev(w), dev(b), out, on, write_back=bool(deltas))
        near(out.float(), want, rel)
        near(stream, v, 1e-6)
        rows = [T - 1, 0, T // 2]
        stream, out = dev(x), torch.empty(3, E, dtype=out_dtype, device=DEV)
        ops.dynamic_tanh(stream, alpha, dev(w), dev(b), out, on, rows=i32(rows))
        near(out.float(), want[rows], rel)
        assert torch.equal(stream.cpu(), x)


def test_two_pending_deltas_before_any_norm():
    """What two mixers side by side leave pending is added by every norm kind, in a launch of its own or in its own."""
    from imparo_amd.config.plan import PartSpec
    from imparo_amd.parts import part_class
    from imparo_amd.parts.base import Residual
    g = torch.Generator().manual_seed(2)
    T, E = 7, 48
    x, a, b, w = (torch.randn(T, E, generator=g), torch.randn(3, T, E, generator=g), torch.randn(T, E, generator=g),
                  torch.rand(E, generator=g) + 0.5)
    want = x.double() + a.double().sum(0) + b.double()
    ctx = hand_context([(0, T)], 16, 2, torch.float32, torch.device(DEV))
    for kind, params, normed in (("rms_norm", dict(width=E, eps=1e-5, tensor="n"), plain.unit_rms(want, 1e-5) * w),
                                 ("none", dict(width=E), want),
                                 ("dynamic_tanh", dict(width=E, tensor="n"), torch.tanh(0.7 * want) * w + w)):
        part = part_class("norm", kind)(PartSpec(kind, "", params), {"n": w, "n.b": w, "n.alpha": torch.tensor(0.7)},
                                        torch.device(DEV), torch.float32)
        res = Residual(dev(x), pending=(dev(a), dev(b)))
        out = part.forward(ctx, res, torch.float32, name=kind)
        near(out, normed, 3e-6, kind)
        near(res.x, want, 1e-6, kind)
        assert res.pending is None


# ------------------------------------------------------------------ products and gates
@pytest.mark.parametrize("m", [1, 5, 16, 17, 40, 64, 100, 300])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_gated_product_with_a_factor(m, dtype):
    """The gated epilogue times a constant, in every kernel the library chooses by the number of rows."""
    from imparo_amd.kernels import ops
    g = torch.Generator().manual_seed(m)
    for n, k in ((48, 64), (1024, 256)):
        x, w = torch.randn(m, k, generator=g).to(dtype), (torch.randn(n, k, generator=g) / math.sqrt(k)).to(dtype)
        y = x.double() @ w.double().T
        want = plain.silu(y[:, 0::2]) * y[:, 1::2] * 0.3
        out = torch.empty(m, n // 2, dtype=dtype, device=DEV)
        ops.gemm(dev(x, dtype), dev(w, dtype), out, swiglu=True, swiglu_scale=0.3)
        near(out.float(), want, 3e-6 if dtype == torch.float32 else 6e-3, f"{n} {k}")


@pytest.mark.parametrize("width,groups", [(64, 4), (640, 1), (36, 3), (2048, 1), (5, 5)])
def test_sigmoid_gate_and_norm_behind_the_heads(width, groups):
    from imparo_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    T, eps, off = 9, 1e-3, 4
    x, gate, w = torch.randn(T, width, generator=g), torch.randn(T, width + 9, generator=g), 0.5 + torch.rand(width, generator=g)
    want = plain.unit_rms(x.double().reshape(T, groups, -1), eps).reshape(T, width) * w * torch.sigmoid(gate[:, off:off + width].double())
    for dt, rel in ((torch.float32, 3e-6), (torch.bfloat16, 5e-3)):
        out = torch.empty(T, width, dtype=dt, device=DEV)
        ops.gated_group_norm(dev(x), dev(gate), off, dev(w), groups, eps, out, gate_first=False, gate_act="sigmoid")
        near(out.float(), want, rel)


@pytest.mark.parametrize("off,n,ld", [(0, 64, 64), (8, 20, 40), (3, 5, 11), (4, 7, 12)])
def test_silu_on_columns(off, n, ld):
    from imparo_amd.kernels import ops
    x = 3.0 * torch.randn(13, ld, generator=torch.Generator().manual_seed(n))
    rows = dev(x)
    ops.silu_columns(rows, off, n)
    want = x.double().clone()
    want[:, off:off + n] = plain.silu(want[:, off:off + n])
    near(rows, want, 2e-6)
    assert torch.equal(rows.cpu()[:, :off], x[:, :off]) and torch.equal(rows.cpu()[:, off + n:], x[:, off + n:])


# ------------------------------------------------------------------ recurrences
def plain_channel_walk(q, k, v, g, beta, S):
    """One head in float64: q, k, g [T, d], v [T, dv], beta [T], S [d, dv] -> (o [T, dv], S)."""
    out = []
    for t in range(q.shape[0]):
        S = g[t][:, None] * S
        S = S + torch.outer(k[t], beta[t] * (v[t] - S.T @ k[t]))
        out.append(S.T @ q[t])
    return torch.stack(out), S


@pytest.mark.parametrize("strength", [0.02, 1.0, 30.0])
@pytest.mark.parametrize("H,share,d,dv", [(2, 1, 16, 24), (4, 2, 20, 12), (1, 1, 1, 1), (2, 2, 128, 64), (3, 1, 48, 32),
                                          (1, 1, 136, 20), (2, 1, 512, 8), (6, 3, 64, 128), (2, 1, 7, 300)])
def test_channel_decay_recurrence_over_segments_in_used_slots(H, share, d, dv, strength):
    """Three requests in slots that held something else, fed in segments of one token, two, and long ones that are
    walked in chunks: results and states are those of one walk over all tokens. Decays from hardly any to gone within
    a token, beside one another in a head's channels."""
    from imparo_amd.kernels import ops
    g = torch.Generator().manual_seed(H * 1000 + d + dv)
    lens, slots, n_slots = [341, 7, 107], [5, 0, 3], 6
    cuts = [[1, 2, 300, 38], [7], [5, 1, 70, 31]]
    Hs, f64 = H // share, torch.float64
    unit = lambda t: t / t.norm(dim=-1, keepdim=True)
    data = []
    for n in lens:
        q, k = unit(torch.randn(n, Hs, d, generator=g)), unit(torch.randn(n, Hs, d, generator=g))
        data.append((q, k, torch.randn(n, H, dv, generator=g), torch.randn(n, H, generator=g),
                     torch.randn(n, H * d, generator=g)))
    rate = strength * (torch.rand(H, generator=g) + 0.1)
    bias = 3.0 * torch.randn(H * d, generator=g) - 1.0
    state = torch.randn(n_slots, H, d, dv, generator=g)
    want_o, want_S = [], []
    for r, (q, k, v, beta, step) in enumerate(data):
        outs, ends = [], []
        for h in range(H):
            dt = torch.nn.functional.softplus((step + bias)[:, h * d:(h + 1) * d].to(f64))
            o, S = plain_channel_walk(q[:, h // share].to(f64), k[:, h // share].to(f64), v[:, h].to(f64),
                                      torch.exp(-rate[h].to(f64) * dt), torch.sigmoid(beta[:, h].to(f64)), torch.zeros(d, dv, dtype=f64))
            outs.append(o)
            ends.append(S)
        want_o.append(torch.stack(outs, 1).reshape(lens[r], H * dv))
        want_S.append(torch.stack(ends))
    st = dev(state)
    for r in range(3):
        st[slots[r]].zero_()                # a request that has seen nothing starts from zero
    fed, got = [0, 0, 0], [[] for _ in lens]
    chunked = 0
    while any(fed[r] < lens[r] for r in range(3)):
        rows = [r for r in range(3) if fed[r] < lens[r]]
        seg = [cuts[r].pop(0) for r in rows]
        cat = lambda j: torch.cat([data[r][j][fed[r]:fed[r] + n].reshape(n, -1) for r, n in zip(rows, seg)])
        rows_t = dev(torch.cat([cat(0), cat(1), cat(2), cat(3)], dim=1))        # q | k | v | beta
        steps_t = dev(torch.cat([torch.full((sum(seg), 3), 9.0), cat(4)], dim=1))
        out = torch.full((rows_t.shape[0], H * dv), 7.0, device=DEV)
        chunk_tokens, max_chunks = ops.channel_delta_chunks(max(seg), d)
        chunked += chunk_tokens > 0
        scratch = torch.full((ops.channel_delta_scratch(len(rows), max_chunks, H, d),), float("nan"), device=DEV) if chunk_tokens else None
        ops.channel_delta_scan(rows_t, 0, share, rows_t, Hs * d, share, rows_t, 2 * Hs * d, steps_t, 3, dev(bias), dev(rate),
                               rows_t, 2 * Hs * d + H * dv, st, i32(np.cumsum([0] + seg[:-1])), i32(seg),
                               i32([slots[r] for r in rows]), out, H, d, dv, chunk_tokens=chunk_tokens, max_chunks=max_chunks,
                               scratch=scratch)
        at = 0
        for r, n in zip(rows, seg):
            got[r].append(out[at:at + n].cpu())
            at += n
            fed[r] += n
    assert chunked == (0 if d > 128 else 1)
    for r in range(3):
        near(torch.cat(got[r]), want_o[r], 2e-5, f"request {r}")
        near(st[slots[r]].cpu(), want_S[r], 2e-5, f"state {r}")
    untouched = [s for s in range(n_slots) if s not in slots]
    assert torch.equal(st[untouched].cpu(), state[untouched])


@pytest.mark.parametrize("H,d,dv", [(2, 16, 24), (3, 20, 12), (1, 1, 1), (2, 200, 8)])
def test_linear_attention_with_silu_on_the_way_in(H, d, dv):
    """Segments of one to seven tokens with SiLU on q, k and v inside the walk."""
    from imparo_amd.kernels import ops
    g = torch.Generator().manual_seed(d)
    T = 23
    x = torch.randn(T, H * (2 * d + dv) + 2, generator=g)
    decay = torch.rand(H, generator=g)
    q = plain.silu(x[:, :H * d].double()).reshape(T, H, d)
    k = plain.silu(x[:, H * d:2 * H * d].double()).reshape(T, H, d)
    v = plain.silu(x[:, 2 * H * d:2 * H * d + H * dv].double()).reshape(T, H, dv)
    S, want = torch.zeros(H, d, dv, dtype=torch.float64), []
    for t in range(T):
        S = decay.double()[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        want.append((S * q[t][:, :, None]).sum(1).reshape(-1))
    st, got, at = torch.zeros(3, H, d, dv, device=DEV), [], 0
    for n in (1, 2, 7, 1, 5, 7):
        out = torch.empty(n, H * dv, device=DEV)
        rows = dev(x[at:at + n])
        ops.decay_scan(rows, 0, 1, rows, H * d, 1, rows, 2 * H * d, st, i32([0]), i32([n]), i32([1]), out, H, d, dv,
                       decay_const=dev(decay), silu_in=True)
        got.append(out.cpu())
        at += n
    near(torch.cat(got), torch.stack(want), 1e-5)
    near(st[1], S, 1e-5)


# ------------------------------------------------------------------ attention
def attention_case(H, G, D, V, segments, page, dtype, window, keep=0, cap=None, sinks=False, out_scale=1.0, boost=None, seed=0,
                   kernel="wave", flip=None, parts=None):
    """q, k, v for rows given as (start, tokens) whose earlier positions are in the cache; pages in a shuffled order, the
    pages that no query of the row can see given back (their table entries are -1), and everything in the cache that
    is no visible key, stale pages included, is not a number. -> (kernel output [tokens, H * V], plain output). `boost`
    (row, key position): that key is made to match the row's last query, so that it takes most of the weight if it
    is seen. `flip` (query position, key position) of row 0: the plain statement with that entry of its mask
    turned over. `parts`: the prompt kernel's keys in that many parts."""
    from imparo_amd.kernels import ops
    g = torch.Generator().manual_seed(seed + D + V)
    bf = (lambda t: t.to(torch.bfloat16).float()) if dtype == torch.bfloat16 else (lambda t: t)
    scale = 1.0 / math.sqrt(D)
    n_pages = sum((p0 + n + page - 1) // page for p0, n in segments) + 3
    order = [p for p in torch.randperm(n_pages, generator=g).tolist() if p != 0]      # page 0 stays stale
    nan = float("nan")
    kc, vc = torch.full((n_pages, G, page, D), nan), torch.full((n_pages, G, page, V), nan)
    sink = 1.0 + torch.randn(H, generator=g) if sinks else None
    q_all, ref_all, tables = [], [], []
    for r, (p0, n) in enumerate(segments):
        L = p0 + n
        q, k, v = bf(torch.randn(L, H, D, generator=g)), bf(torch.randn(L, G, D, generator=g)), bf(torch.randn(L, G, V, generator=g))
        if boost is not None and boost[0] == r:
            k[boost[1]] = bf(q[L - 1, ::H // G] * 3.0)
        seen = plain.seen_mask(torch.arange(L), window, keep)
        if flip is not None and r == 0:
            seen[flip[0], flip[1]] = ~seen[flip[0], flip[1]]
        ref_all.append(out_scale * plain.capped_sink_attention(q.double(), k.double(), v.double(), seen, scale, cap,
                                                               None if sink is None else sink.double())[p0:].float())
        q_all.append(q[p0:])
        # what the row's queries can see: the first tokens and everything from its first query's window on
        low = 0 if window is None else max(0, p0 + 1 - window)
        pages = [order.pop() if (i * page < keep or (i + 1) * page > low) else -1 for i in range((L + page - 1) // page)]
        tables.append(pages)
        for p in range(L):
            if pages[p // page] >= 0 and (p >= low or p < keep):
                kc[pages[p // page], :, p % page] = k[p]
                vc[pages[p // page], :, p % page] = v[p]
    ctx = hand_context(segments, page, n_pages, dtype, torch.device(DEV), tables=tables)
    q = dev(torch.cat(q_all), dtype)
    out = torch.empty(q.shape[0], H * V, dtype=dtype, device=DEV)
    rule = ops.attention_rule(H, keep if window is not None else 0, cap, None if sink is None else dev(sink), out_scale)
    if kernel == "wave":
        ops.attention(q, dev(kc, dtype), dev(vc, dtype), out, ctx.positions, ctx.row_of_token, ctx.block_tables[0], scale, window,
                      rule=rule)
        return out.float().cpu(), torch.cat(ref_all)
    assert D == V and dtype == torch.bfloat16
    kd, vd = dev(kc, dtype), dev(vc.permute(0, 1, 3, 2), dtype)
    if ctx.n_single_rows:
        keys = ops.attention_ruled_keys(ctx.max_context, window, rule)
        splits = (keys + ops.decode_split() - 1) // ops.decode_split()
        part_o = torch.full((ctx.n_single_rows * H * splits * D,), nan, device=DEV)
        part_ml = torch.full((ctx.n_single_rows * H * splits * 2,), nan, device=DEV)
        ops.attention_decode(q, kd, vd, out, part_o, part_ml, ctx.single_rows, ctx.n_single_rows, ctx.seg_start,
                             ctx.positions, ctx.block_tables[0], scale, window, ctx.max_context, exact=True, rule=rule)
    if ctx.n_portion_rows:
        tiles = sum((n + 63) // 64 for n in ctx.host_seg_len if n > 1)
        part_o = part_ml = None
        if parts:
            part_o = torch.full((q.shape[0] * H * parts * D,), nan, device=DEV)
            part_ml = torch.full((q.shape[0] * H * parts * 2,), nan, device=DEV)
        ops.attention_prefill(q, kd, vd, out, ctx.portion_rows, ctx.n_portion_rows, tiles, ctx.seg_start, ctx.seg_len,
                              ctx.positions, ctx.block_tables[0], scale, window, part_o, part_ml, parts or 1, exact=True, rule=rule)
    return out.float().cpu(), torch.cat(ref_all)


RULES = [dict(window=24, keep=5, cap=2.0, sinks=True, out_scale=0.7), dict(window=None, cap=1.0), dict(window=33, sinks=True),
         dict(window=9, keep=40), dict(window=1, keep=1, cap=5.0, sinks=True), dict(window=70, keep=64, sinks=True, out_scale=-0.3),
         dict(window=1000, keep=100, cap=3.0), dict(window=3)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rule", range(len(RULES)))
@pytest.mark.parametrize("H,G,D,V,page", [(4, 2, 16, 32, 16), (3, 1, 24, 40, 64), (2, 1, 12, 20, 8)])
def test_attention_with_rules(H, G, D, V, page, rule, dtype):
    """A portion behind cached keys beside single tokens and a fresh prompt: windows, first tokens that stay, capped
    scores, sinks and a factor, alone and together."""
    got, ref = attention_case(H, G, D, V, [(150, 37), (299, 1), (0, 70), (63, 1), (0, 1)], page, dtype, **RULES[rule])
    near(got, ref, 3e-6 if dtype == torch.float32 else 1e-2)


@pytest.mark.parametrize("rule", range(len(RULES)))
@pytest.mark.parametrize("H,G,D,page", [(4, 2, 16, 16), (8, 2, 64, 64), (2, 2, 128, 32), (3, 1, 48, 64), (16, 4, 32, 64), (5, 5, 80, 16),
                                        (40, 2, 64, 128)])
def test_attention_with_rules_on_the_matrix_cores(H, G, D, page, rule):
    """The same through the matrix-core kernels: decode over one split and several (700 keys), the prompt kernels for
    head sizes in steps of 32 and of 16, pages smaller and larger than a tile."""
    segments = [(150, 37), (299, 1), (0, 70), (700, 1), (63, 1), (0, 1), (500, 130)]
    got, ref = attention_case(H, G, D, D, segments, page, torch.bfloat16, kernel="mfma", **RULES[rule])
    near(got, ref, 1e-2)


@pytest.mark.parametrize("rule", [0, 1, 5, 6])
@pytest.mark.parametrize("parts", [2, 3, 8])
def test_attention_with_rules_in_parts(rule, parts):
    """The prompt kernel's keys cut into parts (more parts than tiles of keys too) and merged."""
    got, ref = attention_case(8, 2, 64, 64, [(400, 90), (0, 20), (130, 64)], 64, torch.bfloat16, kernel="mfma", parts=parts, **RULES[rule])
    near(got, ref, 1e-2)


EDGES = [(24, 16, 5), (64, 64, 64), (65, 64, 63), (9, 8, 17), (1, 16, 1), (130, 64, 20), (100, 32, 65), (40, 16, 0)]


def edge_keys(L, window, keep):
    """(key, seen by the last query): just inside and just outside the window, the last of the first tokens and the next."""
    last = L - 1
    keys = [(last - window + 1, True), (last - window, last - window < keep)]
    if keep:
        keys += [(keep - 1, True), (keep, last - keep < window)]
    return sorted({(k, s) for k, s in keys if 0 <= k <= last})


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n_last", [1, 5])
@pytest.mark.parametrize("window,page,keep", EDGES)
def test_a_key_at_an_edge(window, page, keep, n_last, dtype):
    """A key just inside or just outside the window, or the last of the first tokens or the one after, carries most of
    the last query's weight if it is seen. The query is the last of a portion or a single decoded token."""
    shown = False
    for L in (keep + 2 * window + 3, keep + 3 * window + page, max(window, keep) + 2):
        for key, seen in edge_keys(L, window, keep):
            segs = [(L - min(n_last, L), min(n_last, L))]
            args = dict(window=window, keep=keep, sinks=True, boost=(0, key), seed=key)
            got, ref = attention_case(2, 1, 16, 24, segs, page, dtype, **args)
            near(got, ref, 3e-6 if dtype == torch.float32 else 1e-2, f"{L} {key} {seen}")
            if key != L - 1:       # the case shows the fault it is made for: that key seen where it must not be, or missed
                wrong = attention_case(2, 1, 16, 24, segs, page, dtype, flip=(L - 1, key), **args)[1]
                assert float((wrong[-1] - ref[-1]).abs().max()) > 0.2 * float(ref[-1].abs().max()), (L, key, seen)
                shown = True
    assert shown


@pytest.mark.parametrize("D", [16, 48, 64, 128])
@pytest.mark.parametrize("n_last", [1, 5, 70])
@pytest.mark.parametrize("window,page,keep", [e for e in EDGES if e[1] >= 16])
def test_a_key_at_an_edge_on_the_matrix_cores(window, page, keep, n_last, D):
    for L in (keep + 2 * window + 3, keep + 3 * window + page):
        for key, seen in edge_keys(L, window, keep):
            segs = [(L - min(n_last, L), min(n_last, L)), (40, 1)]
            got, ref = attention_case(4, 2, D, D, segs, page, torch.bfloat16, window=window, keep=keep, sinks=True, cap=9.0,
                                      boost=(0, key), seed=key, kernel="mfma")
            near(got, ref, 1e-2, f"{L} {key} {seen}")


@pytest.mark.parametrize("kernel,dtype", [("wave", torch.float32), ("wave", torch.bfloat16), ("mfma", torch.bfloat16)])
def test_a_far_key_among_hundreds(kernel, dtype):
    """A key 1,100 positions back inside a long window, and a first token that lies 1,100 positions before a short one."""
    for segs in ([(1150, 1), (880, 20)], [(1120, 31), (3, 1)]):
        for window, keep in ((1120, 4), (50, 64), (300, 64)):
            got, ref = attention_case(4, 2, 64, 64, segs, 64, dtype, window=window, keep=keep, cap=30.0, sinks=True, boost=(0, 47),
                                      kernel=kernel)
            near(got, ref, 3e-6 if dtype == torch.float32 else 1e-2)


def test_a_sink_that_outweighs_every_key():
    """Sinks far above and far below the scores: the result fades to nothing, or is what it is without a sink."""
    from imparo_amd.kernels import ops
    g = torch.Generator().manual_seed(1)
    q, k, v = torch.randn(3, 2, 16, generator=g), torch.randn(3, 2, 16, generator=g), torch.randn(3, 2, 16, generator=g)
    ctx = hand_context([(0, 3)], 16, 1, torch.float32, torch.device(DEV))
    kc, vc = torch.zeros(1, 2, 16, 16), torch.zeros(1, 2, 16, 16)
    kc[0, :, :3], vc[0, :, :3] = k.permute(1, 0, 2), v.permute(1, 0, 2)
    sink = torch.tensor([80.0, -90.0])
    out = torch.empty(3, 32, device=DEV)
    ops.attention(dev(q), dev(kc), dev(vc), out, ctx.positions, ctx.row_of_token, ctx.block_tables[0], 0.25, None,
                  rule=ops.attention_rule(2, sink=dev(sink)))
    seen = plain.seen_mask(torch.arange(3), None, 0)
    want = plain.capped_sink_attention(q.double(), k.double(), v.double(), seen, 0.25, None, sink.double())
    near(out[:, 16:], want[:, 16:], 2e-6)
    assert float(out[:, :16].abs().max()) < 1e-30


# ------------------------------------------------------------------ the model
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompt_and_stepwise(dirs, plains, name, dtype):
    """A prompt whole; then most of it whole and its last 50 tokens one by one (captured steps)."""
    from imparo_amd.engine import StepEntry
    tokens = prompt_tokens(vocab(name), 170, 7)
    ref = plains[name].logits(tokens)
    rel = bound(dtype, runs(name))
    eng = make_engine(dirs[name], dtype)
    whole = eng.step([StepEntry("w", tokens, list(range(170)))]).cpu()
    eng.release("w")
    noise = plains[name].noise(tokens, dtype)
    check(whole, ref, f"{name} whole", rel, noise)
    head = eng.step([StepEntry("d", tokens[:120], list(range(120)))]).cpu()
    tail = [eng.step([StepEntry("d", [t], [0])]).cpu() for t in tokens[120:]]
    eng.release("d")
    stepwise = torch.cat([head] + tail)
    check(stepwise, ref, f"{name} stepwise", rel, noise)
    if dtype == "float32":
        check(stepwise, whole, f"{name} stepwise against whole", 2e-6, noise)


@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_every_layer_alone(dirs, name, tmp_path):
    """The model cut behind its first, second, ... layer run: the first layer that differs from the plain
    implementation is named by the failing case."""
    from imparo_amd.engine import StepEntry
    cfg, seed = CONFIGS[name]
    tokens = prompt_tokens(cfg["vocab"], 40, 9)
    for k in range(1, len(cfg["layers"])):
        sub = dict(cfg, layers=cfg["layers"][:k])
        sub.pop("loop", None)
        d = write_model(sub, seed, str(tmp_path / f"cut{k}"), ranks=RANKS[name])
        got = make_engine(d, "float32").step([StepEntry("a", tokens, list(range(40)))]).cpu()
        y = Yardstick(d)
        check(got, y.logits(tokens), f"{name}: {k} layers", bound("float32", k), y.noise(tokens))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,page", [("A", 16), ("B", 8), ("C", 16), ("D", 64), ("E", 32)])
def test_portions_of_changing_size(dirs, plains, name, page, dtype):
    """Portions down to two tokens, cut inside pages, windows and conv histories, also without captured steps."""
    tokens = prompt_tokens(vocab(name), 160, 8)
    ref = plains[name].logits(tokens)
    noise = plains[name].noise(tokens, dtype)
    for cuts, graphs in (((2, 3, 17, 2, 1, 31, 1, 1, 5), True), ((64, 2, 9), False), ((1,), True), ((2,), False)):
        eng = make_engine(dirs[name], dtype, page_size=page, use_graphs=graphs)
        got = step_all(eng, "p", tokens if len(cuts) > 1 else tokens[:45], cuts)
        check(got, ref[:got.shape[0]], f"{name} cuts {cuts}", bound(dtype, runs(name)), noise)


@pytest.mark.parametrize("name", ["A", "C", "E"])
def test_a_long_portion_beside_a_short_one(dirs, plains, name):
    """Portions of 300 and 290 tokens (the recurrences walk such a step in chunks) beside one of 3 and a single token,
    then the rest: every request's logits are those of its whole prompt."""
    from imparo_amd.engine import StepEntry
    prompts = [prompt_tokens(vocab(name), n, 40 + i) for i, n in enumerate((330, 300, 9, 5))]
    eng = make_engine(dirs[name], "float32", page_size=16)
    cuts = [(300, 30), (290, 10), (3, 6), (1, 4)]
    got = [[] for _ in prompts]
    for step in range(2):
        entries = []
        for i, p in enumerate(prompts):
            lo = sum(cuts[i][:step])
            entries.append(StepEntry(i, p[lo:lo + cuts[i][step]], list(range(cuts[i][step]))))
        out = eng.step(entries).cpu()
        at = 0
        for i, e in enumerate(entries):
            got[i].append(out[at:at + len(e.tokens)])
            at += len(e.tokens)
    for i, p in enumerate(prompts):
        check(torch.cat(got[i]), plains[name].logits(p), f"{name} request {i}", bound("float32", runs(name)),
              plains[name].noise(p))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,page", [("A", 8), ("B", 8), ("D", 16), ("E", 16)])
def test_mixed_batches_on_a_full_pool(dirs, plains, name, page, dtype):
    """Six unequal requests, at most four live, portions beside single tokens, on a pool of exactly the schedule's
    peak and four slots: pages and state slots are used again. Each request's logits are those it has alone."""
    from imparo_amd.engine import StepEntry
    rng = random.Random(5)
    lengths = [70, 33, 1, 90, 2, 51]
    prompts = [prompt_tokens(vocab(name), n, 20 + i) for i, n in enumerate(lengths)]
    steps = mixed_schedule(rng, lengths, max_live=4)
    eng = make_engine(dirs[name], dtype, page_size=page, max_tokens=peak_pages(steps, page) * page, max_requests=4)
    got = {i: [] for i in range(len(lengths))}
    for entries, ends in steps:
        out = eng.step([StepEntry(rid, prompts[rid][lo:hi], list(range(hi - lo))) for rid, lo, hi in entries]).cpu()
        at = 0
        for rid, lo, hi in entries:
            got[rid].append(out[at:at + hi - lo])
            at += hi - lo
        for rid in ends:
            eng.release(rid)
    for i, p in enumerate(prompts):
        check(torch.cat(got[i]), plains[name].logits(p), f"{name} request {i}", bound(dtype, runs(name)),
              plains[name].noise(p, dtype))
    eng.cache.check()
    assert eng.free_pages() == [g.pool.n_pages for g in eng.cache.groups]


@pytest.mark.parametrize("name", ["A", "D"])
def test_long_decoding_and_first_tokens(dirs, plains, name):
    """One prompt token, then 330 single-token steps: decoded tokens leave every window, the cache gives back the pages
    behind it while those of the first tokens stay, and the recurrences run 331 steps on their states; and requests of
    one and of two tokens alone."""
    from imparo_amd.engine import StepEntry
    tokens = prompt_tokens(vocab(name), 331, 3)
    exact = plains[name].logits(tokens)
    page = 16
    for dtype in ("float32", "bfloat16"):
        eng = make_engine(dirs[name], dtype, page_size=page)
        got = torch.cat([eng.step([StepEntry("r", [t], [0])]).cpu() for t in tokens])
        noise = plains[name].noise(tokens, dtype)
        check(got, exact, "long decoding", bound(dtype, runs(name)), noise)
        for g, group in enumerate(eng.cache.groups):
            table = eng.cache.table(g, "r")
            first, window = -(-group.spec.keep_first // page), group.spec.window
            assert all(p >= 0 for p in table[:first]) and table[first] == -1
            assert sum(p >= 0 for p in table) <= first + window // page + 2
        eng.release("r")
        two = eng.step([StepEntry("x", tokens[:1], [0]), StepEntry("y", tokens[:2], [0, 1])]).cpu()
        check(two, torch.cat([exact[:1], exact[:2]]), "first tokens", bound(dtype, runs(name)),
              torch.cat([noise[:1], noise[:2]]))


def test_other_constants(dirs, tmp_path):
    """Values that a model may happen to make equal or 1: another multiplier, eps, scale, cap, window, number of first
    tokens, rotation, decay, factor and loop move the logits, and by what the plain implementation says."""
    from imparo_amd.engine import StepEntry
    cfg, seed = CONFIGS["A"]
    tokens = prompt_tokens(cfg["vocab"], 60, 4)
    base = make_engine(dirs["A"], "float32").step([StepEntry("a", tokens, list(range(60)))]).cpu()
    side = lambda c, s: c["layers"][1]["mixer"][s]
    changes = [
        lambda c: c.update(residual_mult=1.0),
        lambda c: c.pop("residual_mult"),
        lambda c: c["embedding"].update(scale=0.7),
        lambda c: c["norm"].update(eps=1e-1),
        lambda c: side(c, "left").update(scale=1.3),
        lambda c: side(c, "left").update(softcap=0.5),
        lambda c: side(c, "left").pop("softcap"),
        lambda c: side(c, "left")["mask"].update(size=3),
        lambda c: side(c, "left")["mask"].update(keep_first=0),
        lambda c: side(c, "left")["mask"].update(keep_first=30),
        lambda c: side(c, "left").pop("mask"),
        lambda c: side(c, "left")["rot"].update(base=33.0, dims=16),
        lambda c: side(c, "left").pop("rot"),
        lambda c: side(c, "right").update(decay=[0.1, 1.0, 0.5]),
        lambda c: c["layers"][1]["mixer"].update(left_scale=0.2),
        lambda c: c["layers"][1]["mixer"].update(right_scale=2.2),
        lambda c: c["loop"].update(times=3),
        lambda c: c["loop"].update(start=0, stop=4),
        lambda c: c.pop("loop"),
        lambda c: c["layers"][0].update(mlp=None),
    ]
    weights = random_weights(cfg, seed, RANKS["A"])
    for n, change in enumerate(changes):
        other = copy.deepcopy(cfg)
        change(other)
        d = str(tmp_path / f"other{n}")
        from imparo_amd.weights.safetensors_io import save_file
        os.makedirs(d)
        with open(os.path.join(d, "config.json"), "w") as f:
            json.dump(other, f)
        keep = {k: v for k, v in weights.items() if other["layers"][0]["mlp"] is not None or not k.startswith(("l0.mlp", "l0.norm2"))}
        save_file({k: v.to(torch.bfloat16).contiguous() for k, v in keep.items()}, os.path.join(d, "model.safetensors"))
        got = make_engine(d, "float32").step([StepEntry("a", tokens, list(range(60)))]).cpu()
        y = Yardstick(d)
        check(got, y.logits(tokens), f"change {n}", bound("float32", runs_of(other)), y.noise(tokens))
        assert float((got - base).abs().max()) > 0.01 * float(base.abs().max()), f"change {n} moves nothing"


def test_generation_through_the_entry_point(dirs, plains):
    from imparo_amd import generate
    prompts = [prompt_tokens(vocab("A"), n, 50 + n) for n in (1, 6, 29, 13, 40)]
    want = [plains["A"].greedy(p, 12) for p in prompts]
    assert all(len(set(w)) > 2 for w in want), f"the plain continuation hardly moves: {want}"
    assert generate(dirs["A"], prompts, max_tokens=12, dtype="float32", page_size=8) == want
    # three at a time under a small token budget: prompts in portions beside decoding rows
    os.environ["IMPARO_BATCH"] = "5"
    try:
        got = generate(dirs["A"], prompts, max_tokens=12, dtype="float32", page_size=8, parallel=3, max_batch_tokens=11)
    finally:
        del os.environ["IMPARO_BATCH"]
    assert got == want
    got16 = generate(dirs["A"], prompts, max_tokens=12, dtype="bfloat16", parallel=3)
    assert all(len(out) == 12 for out in got16)


def test_trace_replay_program(dirs, plains, tmp_path):
    tokens = prompt_tokens(vocab("B"), 45, 1)
    other = prompt_tokens(vocab("B"), 9, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": tokens[:20], "want": [0, 19]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": tokens[20:44], "want": []},
                                {"id": "b", "tokens": other, "want": [8]}], "end": ["b"]},
        {"step": 2, "entries": [{"id": "a", "tokens": tokens[44:], "want": [0]}], "end": ["a"]},
    ]
    out = tmp_path / "out"
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", dirs["B"], "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    V = vocab("B")
    ref, ref_other = plains["B"].logits(tokens), plains["B"].logits(other)
    read = lambda n: torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, V))
    check_logits(read(0), ref[[0, 19]], "float32", "step 0")
    check_logits(read(1), ref_other[[8]], "float32", "step 1")
    check_logits(read(2), ref[[44]], "float32", "step 2")


@pytest.mark.parametrize("taps", [2, 3, 4])
@pytest.mark.parametrize("out_dtype", [torch.float32, torch.bfloat16])
def test_short_conv_over_many_tokens(taps, out_dtype):
    """Segments of many sizes in one batch of many tokens, so that runs of tokens that share their loads hold the end of
    one segment and the start of another, beside histories left by earlier batches."""
    from imparo_amd.kernels import ops
    g = torch.Generator().manual_seed(taps)
    C, ld, off, slots = 70, 90, 3, [4, 1, 0, 6, 2]
    cuts = [[1, 70, 2], [3, 9, 65], [33, 1, 1], [50, 5, 17], [2, 2, 40]]
    w = torch.randn(C, taps, generator=g)
    rows = [torch.randn(sum(cut), ld, generator=g) for cut in cuts]
    want = [plain.silu(plain.causal_conv(x[:, off:off + C].double(), w.double())) for x in rows]
    st = dev(torch.randn(7, taps - 1, C, generator=g))
    for s in slots:
        st[s].zero_()
    got, fed = [[] for _ in cuts], [0] * len(cuts)
    for step in range(3):
        seg = [cut[step] for cut in cuts]
        u = dev(torch.cat([x[f:f + n] for x, f, n in zip(rows, fed, seg)]))
        assert u.shape[0] >= 64
        row_of = np.concatenate([[i] * n for i, n in enumerate(seg)])
        out = torch.empty(u.shape[0], C, dtype=out_dtype, device=DEV)
        ops.causal_conv(u, C, dev(w), None, st, i32(row_of), i32(np.cumsum([0] + seg[:-1])), i32(seg), i32(slots), out, silu=True,
                        u_off=off)
        for i, o in enumerate(torch.split(out.float().cpu(), seg)):
            got[i].append(o)
            fed[i] += seg[i]
    for i in range(len(cuts)):
        near(torch.cat(got[i]), want[i], 3e-6 if out_dtype == torch.float32 else 5e-3, f"request {i}")
