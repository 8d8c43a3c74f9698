"""The gated delta rule with one decay a head and key channel.

As the gated delta rule (gated_delta.py) up to the unit vectors: q and k of
[kv_heads, dim], v of [heads, vdim], a causal convolution per channel and SiLU
on each, q and k unit vectors per head, q times dim^(-1/2), b = sigmoid(Wb h)
one number a head. The decay comes through a bottleneck and is one number a head
and state row,

    g = exp(-exp(A_log_h) softplus(Wa2 (Wa1 h) + dt_bias)),      [heads, dim],

and acts on the rows of S:

    S <- diag(g) S;   u = b (v - S^T k);   S <- S + k u^T;   o = S^T q.

Each head's o is divided by its root mean square, multiplied by a weight that all
heads share and by sigmoid(Wg2 (Wg1 h)); the heads side by side go through the
output projection. `out_scale` multiplies the result (the norm's weight carries
it, float32). A request's state is S, float32, and the convs' last taps - 1
inputs. Decays, gates, unit vectors, the state and every sum of the recurrence
are float32 whatever the engine's dtype. The two inner ranks are the file's.

Parameters: width, heads, kv_heads, dim, vdim, taps, eps, out_scale, names.
"""
from __future__ import annotations

from typing import Dict

import torch

from ..cache.pages import FixedArray, FixedSpec
from ..config.plan import PartSpec
from ..kernels import ops
from ..weights.loader import FreeDim, TensorDecl
from .base import Declared, StepContext
from .gated_delta import UNIT_EPS
from .linear import Linear, place_projection, place_vector
from .registry import register_part

_DEFAULT_NAMES = dict(q="q", k="k", v="v", q_conv="q.conv", k_conv="k.conv", v_conv="v.conv", b="b", a1="a1", a2="a2",
                      A_log="A_log", dt_bias="dt_bias", g1="g1", g2="g2", norm="norm", o="o")


class ChannelDelta:
    role = "mixer"
    graph_safe = True     # launches kernels only: a step made of such parts can be captured

    @staticmethod
    def _names(spec: PartSpec) -> Dict[str, str]:
        names = dict(_DEFAULT_NAMES)
        names.update(spec.get("names") or {})
        return {k: f"{spec.prefix}.{v}" for k, v in names.items()}

    @classmethod
    def declare(cls, spec: PartSpec) -> Declared:
        n = cls._names(spec)
        E, H, Hk, dk, dv, L = spec["width"], spec["heads"], spec["kv_heads"], spec["dim"], spec["vdim"], spec["taps"]
        rank = FreeDim(max(dk, dv))
        return {
            n["q"]: (TensorDecl((Hk * dk, E)), "matrix"),
            n["k"]: (TensorDecl((Hk * dk, E)), "matrix"),
            n["v"]: (TensorDecl((H * dv, E)), "matrix"),
            n["q_conv"]: (TensorDecl((Hk * dk, L), "vector"), "conv"),
            n["k_conv"]: (TensorDecl((Hk * dk, L), "vector"), "conv"),
            n["v_conv"]: (TensorDecl((H * dv, L), "vector"), "conv"),
            n["b"]: (TensorDecl((H, E)), "matrix"),
            n["a1"]: (TensorDecl((rank, E)), "matrix"),
            n["a2"]: (TensorDecl((H * dk, rank)), "matrix"),
            n["A_log"]: (TensorDecl((H,), "vector"), "wide"),
            n["dt_bias"]: (TensorDecl((H * dk,), "vector"), "bias"),
            n["g1"]: (TensorDecl((rank, E)), "matrix"),
            n["g2"]: (TensorDecl((H * dv, rank)), "matrix"),
            n["norm"]: (TensorDecl((dv,), "vector"), "norm"),
            n["o"]: (TensorDecl((E, H * dv)), "matrix"),
        }

    def __init__(self, spec: PartSpec, tensors: Dict[str, torch.Tensor], device: torch.device,
                 engine_dtype: torch.dtype):
        n = self._names(spec)
        self.width, self.heads, self.kv_heads = spec["width"], spec["heads"], spec["kv_heads"]
        self.dim, self.vdim, self.taps = spec["dim"], spec["vdim"], spec["taps"]
        self.eps = float(spec["eps"])
        if self.heads % self.kv_heads:
            raise ValueError(f"{self.heads} heads cannot share {self.kv_heads} query/key heads evenly")
        if not 1 <= self.taps <= 64:
            raise ValueError(f"the conv kernels take 1 to 64 taps, got {self.taps}")
        if self.dim > ops.DECAY_SCAN_MAX_DIM:
            raise ValueError(f"the recurrence kernel takes up to {ops.DECAY_SCAN_MAX_DIM} state rows a head, got {self.dim}")
        H, Hk, dk, dv = self.heads, self.kv_heads, self.dim, self.vdim
        for low, high in (("a1", "a2"), ("g1", "g2")):
            if tensors[n[low]].shape[0] != tensors[n[high]].shape[1]:
                raise ValueError(f"{n[low]} gives {tensors[n[low]].shape[0]} numbers and {n[high]} reads {tensors[n[high]].shape[1]}")
        self.conv_channels = 2 * Hk * dk + H * dv

        def side(*names):
            ws = [tensors[n[x]] for x in names]
            return ws if len({w.dtype for w in ws}) == 1 else [w.to(torch.float32) for w in ws]

        # one projection for q | k | v | b: the same dot products, one launch
        self.proj = Linear(place_projection(torch.cat(side("q", "k", "v", "b"), dim=0), engine_dtype, device))
        # The two bottlenecks side by side: one projection down, and one up whose matrix has a block for each (the
        # other block's columns are zero and add nothing). Filled up with rows of zero weight to a multiple of 8
        # inner numbers, which the bfloat16 kernels walk.
        a1, g1, a2, g2 = side("a1", "g1", "a2", "g2")
        ra, rg = a1.shape[0], g1.shape[0]
        fill = (-(ra + rg)) % 8
        self.low = Linear(place_projection(torch.cat([a1, g1, a1.new_zeros(fill, self.width)], dim=0), engine_dtype, device))
        high = a2.new_zeros(H * dk + H * dv, ra + rg + fill)
        high[:H * dk, :ra] = a2
        high[H * dk:, ra:ra + rg] = g2
        self.high = Linear(place_projection(high, engine_dtype, device))
        if self.low.in_dtype != self.proj.in_dtype:
            raise ValueError("the projections of a mixer's input are stored in one dtype")
        self.conv_weight = place_vector(torch.cat([tensors[n[x]].to(torch.float32).reshape(-1, self.taps)
                                                   for x in ("q_conv", "k_conv", "v_conv")], dim=0), device)
        self.dt_bias = place_vector(tensors[n["dt_bias"]], device)
        self.rate = place_vector(torch.exp(tensors[n["A_log"]].to(torch.float32)), device)
        self.norm = place_vector(tensors[n["norm"]].to(torch.float32).repeat(H) * float(spec.get("out_scale", 1.0)), device)
        self.out = Linear(place_projection(tensors[n["o"]], engine_dtype, device))

    @property
    def in_dtype(self) -> torch.dtype:
        return self.proj.in_dtype

    def cache_spec(self, page_size: int) -> FixedSpec:
        arrays = (FixedArray("state", (self.heads, self.dim, self.vdim), "float32", 0.0),)
        if self.taps > 1:
            arrays += (FixedArray("conv", (self.taps - 1, self.conv_channels), "float32", 0.0),)
        return FixedSpec(arrays=arrays)

    def forward(self, ctx: StepContext, site: int, owns_cache: bool, h: torch.Tensor) -> torch.Tensor:
        if not owns_cache:
            raise ValueError("a recurrence's state cannot be read from another layer")
        T, H, Hk, dk, dv, C = h.shape[0], self.heads, self.kv_heads, self.dim, self.vdim, self.conv_channels
        state = ctx.fixed_arrays(site)
        rows = self.proj(ctx, h, torch.float32, "delta_rows", alias="mixer_in")              # q k v | b
        low = self.low(ctx, h, self.high.in_dtype, "delta_low")
        steps = self.high(ctx, low, torch.float32, "delta_steps")                            # decays' steps | gate
        qkv = ctx.workspace.get("delta_qkv", (T, C), torch.float32)
        ops.causal_conv(rows, C, self.conv_weight, None, state.get("conv"), ctx.row_of_token, ctx.seg_start,
                        ctx.seg_len, ctx.slot, qkv, silu=True, single_tokens=ctx.max_seg_len == 1)
        # q and k heads as unit vectors; the queries carry dim^(-1/2)
        ops.head_prepare(qkv, 0, 2 * Hk, dk, unit=True, unit_eps=UNIT_EPS, n_first=Hk, scale_first=float(dk) ** -0.5)
        o = ctx.workspace.get("delta_o", (T, H * dv), torch.float32)
        # a long portion: the rule in chunks (a triangle solved a chunk, side by side; then the chunks in order)
        chunk_tokens, max_chunks = ops.channel_delta_chunks(ctx.max_seg_len, dk)
        scratch = None
        if chunk_tokens:
            scratch = ctx.workspace.get("channel_delta_chunks",
                                        (ops.channel_delta_scratch(ctx.n_rows, max_chunks, H, dk),), torch.float32)
        ops.channel_delta_scan(qkv, 0, H // Hk, qkv, Hk * dk, H // Hk, qkv, 2 * Hk * dk, steps, 0, self.dt_bias, self.rate,
                               rows, C, state["state"], ctx.seg_start, ctx.seg_len, ctx.slot, o, H, dk, dv,
                               chunk_tokens=chunk_tokens, max_chunks=max_chunks, scratch=scratch)
        gated = ctx.workspace.get("delta_gated", (T, H * dv), self.out.in_dtype, alias="mixer_mid")
        ops.gated_group_norm(o, steps, H * dk, self.norm, H, self.eps, gated, gate_first=False, gate_act="sigmoid")
        return self.out(ctx, gated, torch.float32, "mixer_out", sliced_ok=True, into=ctx.stream)


register_part("mixer", "channel_delta", ChannelDelta)
