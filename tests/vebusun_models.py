"""Small Vebusun configurations with random weights, for tests. The weights are drawn so that every mechanism
matters: projections of unit gain, conv taps of unit size, norm weights away from one with biases, alphas that bend
the stream, sinks near the largest scores, decays that spread from slow to fast over the channels of a head; the
queries of the recurrences are drawn near their keys (see `near` below)."""
import json
import math
import os

import torch


def left(heads, kv_heads, dim, vdim, scale=None, softcap=None, window=None, keep=None, rot=None, base=10000.0):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale if scale is not None else 1.0 / math.sqrt(dim))
    if softcap is not None:
        m["softcap"] = softcap
    if window is not None:
        m["mask"] = dict(size=window)
        if keep is not None:
            m["mask"]["keep_first"] = keep
    if rot is not None:
        m["rot"] = dict(dims=rot, base=base)
    return m


def right(heads, dim, vdim, decay):
    return dict(heads=heads, dim=dim, vdim=vdim, decay=list(decay))


def parallel(l, r, left_scale=1.0, right_scale=1.0):
    return dict(type="parallel", mixer=dict(left=l, right=r, left_scale=left_scale, right_scale=right_scale))


def delta(heads, kv_heads, dim, vdim, conv):
    return dict(type="channel_delta", mixer=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv))


def layer(mixer, ff):
    return dict(mixer, mlp=None if ff is None else dict(kind="dense", ff=ff))


# A: both mixers; a rotation of part of a head; the first tokens kept beside a window; shared keys; a loop over the
# middle layers; a layer without feed-forward
CONFIG_A = dict(
    architecture="Vebusun", vocab=200, width=64, norm=dict(eps=1e-6), residual_mult=0.45, embedding=dict(scale=2.5),
    loop=dict(start=1, stop=3, times=2),
    layers=[
        layer(delta(4, 2, 16, 24, 4), 40),
        layer(parallel(left(4, 2, 16, 16, scale=0.4, softcap=6.0, window=21, keep=5, rot=8, base=500.0),
                       right(3, 16, 24, [0.7, 0.95, 0.999]), 1.3, 0.7), 48),
        layer(delta(2, 2, 24, 8, 3), None),
        layer(parallel(left(2, 1, 32, 32, softcap=3.0, window=40, keep=17, rot=32), right(1, 8, 40, [0.9]), 0.6, 1.2), 24),
    ])

# B: values that a model may happen to make equal or 1, or leave out: no multiplier, no factor on the embedding, one
# head, one state row, one tap, an inner rank of one, no mask, no first tokens, no cap, no rotation, decays of one
# and a half, a window of one position, factors of one
CONFIG_B = dict(
    architecture="Vebusun", vocab=300, width=96, norm=dict(eps=1e-5),
    layers=[
        layer(parallel(left(1, 1, 24, 40, scale=0.2), right(1, 1, 8, [1.0])), 100),
        layer(delta(1, 1, 8, 16, 1), 64),
        layer(parallel(left(6, 3, 16, 16, softcap=50.0, window=1, rot=16, base=100.0), right(2, 32, 16, [0.5, 1.0])), None),
        layer(delta(3, 1, 32, 8, 2), 40),
        layer(parallel(left(2, 2, 16, 16, window=1, keep=1), right(2, 16, 16, [0.5, 0.99])), 32),
    ])

# C: sizes that are no multiples of 8 (width, heads, keys, values, states, hidden widths), edges that cut pages
CONFIG_C = dict(
    architecture="Vebusun", vocab=70, width=36, norm=dict(eps=1e-4), residual_mult=0.8, embedding=dict(scale=0.9),
    loop=dict(start=0, stop=2, times=3),
    layers=[
        layer(delta(3, 3, 12, 10, 4), 28),
        layer(parallel(left(3, 1, 12, 20, softcap=4.0, window=5, keep=3, rot=4, base=50.0), right(3, 20, 12, [0.8, 0.9, 0.95]),
                       0.5, 0.9), 20),
        layer(delta(2, 1, 20, 12, 3), 12),
    ])

# D: sizes like a real model's layers in small: heads of 64 on the matrix cores, a window of 100 beside 70 first
# tokens, states of 128 rows, rows of 512 values normed whole
CONFIG_D = dict(
    architecture="Vebusun", vocab=500, width=128, norm=dict(eps=2e-5), residual_mult=0.4, embedding=dict(scale=3.0),
    layers=[
        layer(parallel(left(8, 2, 64, 64, scale=0.125, softcap=20.0, window=100, keep=70, rot=64, base=5e5),
                       right(4, 64, 128, [0.9, 0.97, 0.99, 0.999]), 0.9, 1.1), 256),
        layer(delta(4, 2, 128, 64, 4), 192),
        layer(parallel(left(4, 4, 128, 128, scale=0.09, softcap=15.0, window=64, keep=4, rot=64), right(2, 128, 32, [0.95, 0.98])), 64),
        layer(delta(2, 1, 64, 128, 4), None),
    ])

# E: head sizes in steps of 16 that are none of 32 (the other prompt kernel), and a head wider than the chunk form takes
CONFIG_E = dict(
    architecture="Vebusun", vocab=120, width=80, norm=dict(eps=1e-6), residual_mult=0.5, embedding=dict(scale=2.0),
    loop=dict(start=0, stop=1, times=2),
    layers=[
        layer(parallel(left(4, 2, 48, 48, softcap=9.0, window=33, keep=20, rot=24, base=2000.0), right(2, 24, 16, [0.85, 0.99]),
                       1.1, 0.8), 56),
        layer(delta(2, 1, 136, 16, 2), 40),
        layer(parallel(left(3, 3, 80, 80, softcap=9.0, window=70, keep=66, rot=80), right(1, 16, 16, [0.97])), None),
    ])

CONFIGS = {"A": (CONFIG_A, 51), "B": (CONFIG_B, 52), "C": (CONFIG_C, 53), "D": (CONFIG_D, 54), "E": (CONFIG_E, 55)}
RANKS = {"A": (12, 20), "B": (1, 1), "C": (5, 9), "D": (32, 24), "E": (16, 16)}       # inner ranks of decays and gates


def runs_of(config):
    loop = config.get("loop") or dict(start=0, stop=0, times=1)
    return len(config["layers"]) + (loop["stop"] - loop["start"]) * (loop["times"] - 1)


def random_weights(config, seed, ranks=(12, 20)):
    g = torch.Generator().manual_seed(seed)
    E, V = config["width"], config["vocab"]
    randn = lambda *shape: torch.randn(*shape, generator=g)
    rand = lambda *shape: torch.rand(*shape, generator=g)
    matrix = lambda out, inn: randn(out, inn) / math.sqrt(inn)
    weight = lambda n: 0.5 + rand(n)
    t = {"embed": randn(V, E), "head": randn(V, E) / math.sqrt(E)}

    def norm(name):
        t[name], t[name + ".b"], t[name + ".alpha"] = weight(E), 0.3 * randn(E), 0.4 + 0.4 * rand(())

    def near(a, b):
        # A recurrence's first token gives (k . q) u, which the norm behind the heads stretches to unit size: where
        # k . q happens to lie near zero, its sign, a matter of rounding, decides the token's result. The queries
        # are drawn near the keys, so that this dot product stays away from zero and float32 runs can be held to
        # the float32 bound at every row.
        t[a] = 0.8 * t[b] + 0.6 * t[a]

    norm("final.norm")
    for i, l in enumerate(config["layers"]):
        p, m = f"l{i}", l["mixer"]
        norm(f"{p}.norm1")
        x = f"{p}.mix"
        if l["type"] == "channel_delta":
            H, Hk, dk, dv, L = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
            for n, rows in (("q", Hk * dk), ("k", Hk * dk), ("v", H * dv)):
                t[f"{x}.{n}"], t[f"{x}.{n}.conv"] = matrix(rows, E), randn(rows, L) * (1.2 / math.sqrt(L))
            near(f"{x}.q", f"{x}.k")
            near(f"{x}.q.conv", f"{x}.k.conv")
            t[f"{x}.b"] = matrix(H, E)
            t[f"{x}.a1"], t[f"{x}.a2"] = matrix(ranks[0], E), matrix(H * dk, ranks[0])
            # channels of a head from hardly any decay to a forgetting within a token or two
            t[f"{x}.A_log"], t[f"{x}.dt_bias"] = 0.7 * randn(H) - 0.5, 3.0 * randn(H * dk) - 2.0
            t[f"{x}.g1"], t[f"{x}.g2"] = matrix(ranks[1], E), matrix(H * dv, ranks[1])
            t[f"{x}.norm"], t[f"{x}.o"] = weight(dv), matrix(E, H * dv)
        else:
            a, b = m["left"], m["right"]
            H, G, d, dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            for n, rows in (("q", H * d), ("k", G * d), ("v", G * dv)):
                t[f"{x}.left.{n}"] = matrix(rows, E)
            t[f"{x}.left.q.norm"], t[f"{x}.left.k.norm"] = weight(d), weight(d)
            t[f"{x}.left.sink"], t[f"{x}.left.o"] = 1.0 + 1.5 * randn(H), matrix(E, H * dv)
            H, d, dv = b["heads"], b["dim"], b["vdim"]
            t[f"{x}.right.q"], t[f"{x}.right.k"] = matrix(H * d, E), matrix(H * d, E)
            near(f"{x}.right.q", f"{x}.right.k")
            t[f"{x}.right.v"], t[f"{x}.right.g"], t[f"{x}.right.o"] = matrix(H * dv, E), matrix(H * dv, E), matrix(E, H * dv)
            t[f"{x}.right.norm"] = weight(H * dv)
        if l["mlp"] is not None:
            F = l["mlp"]["ff"]
            norm(f"{p}.norm2")
            t[f"{p}.mlp.gate"], t[f"{p}.mlp.up"], t[f"{p}.mlp.down"] = matrix(F, E), matrix(F, E), matrix(E, F)
    return t


def write_model(config, seed, out_dir, overrides=None, ranks=(12, 20)):
    """Writes config.json and model.safetensors (bfloat16) and returns the folder."""
    from imparo_amd.weights.safetensors_io import save_file
    tensors = random_weights(config, seed, ranks)
    tensors.update(overrides or {})
    os.makedirs(out_dir, exist_ok=True)
    with open(os.path.join(out_dir, "config.json"), "w") as f:
        json.dump(config, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in tensors.items()},
              os.path.join(out_dir, "model.safetensors"))
    return out_dir
