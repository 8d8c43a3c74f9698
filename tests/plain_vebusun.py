"""A plain, slow statement of the Vebusun design: float64 (or float32), whole
sequences, no cache, one function per mechanism. It shares no code with the
engine: tests hold the engine against it.

Notation: a sequence is a [tokens, width] matrix; positions count from 0; a
linear weight is [out, in] and applied as x @ W.T; `w` maps tensor names to
tensors and `L` is a layer's prefix ("l3").
"""
from __future__ import annotations

import json
import os
import struct
from typing import Dict, List, Optional

import numpy as np
import torch


def read_tensors(path: str, dtype=torch.float64) -> Dict[str, torch.Tensor]:
    """A safetensors file by hand: 8 bytes of length, a JSON header, raw data."""
    with open(path, "rb") as f:
        (n,) = struct.unpack("<Q", f.read(8))
        header = json.loads(f.read(n))
        data = f.read()
    out = {}
    for name, meta in header.items():
        if name == "__metadata__":
            continue
        a, b = meta["data_offsets"]
        raw = np.frombuffer(data[a:b], dtype=np.uint8)
        if meta["dtype"] == "BF16":
            wide = raw.view(np.uint16).astype(np.uint32) << 16
            t = torch.from_numpy(wide.view(np.float32).copy())
        elif meta["dtype"] == "F32":
            t = torch.from_numpy(raw.view(np.float32).copy())
        else:
            raise ValueError(meta["dtype"])
        out[name] = t.reshape(meta["shape"]).to(dtype)
    return out


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.where(z > 30, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def unit_rms(x, eps):
    """x divided by its root mean square over the last dimension, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def dynamic_tanh(x, w, name: str):
    """A norm without a statistic: tanh(alpha x) w + b with one alpha for the row."""
    return torch.tanh(w[f"{name}.alpha"] * x) * w[name] + w[f"{name}.b"]


def causal_conv(u, taps_w):
    """u [tokens, channels], taps_w [channels, taps]; the last tap is the current token's and there
    are zeros before the start."""
    T, C = u.shape
    K = taps_w.shape[1]
    padded = torch.cat([u.new_zeros(K - 1, C), u], dim=0)
    y = u.new_zeros(T, C)
    for j in range(K):
        y = y + padded[j:j + T] * taps_w[:, j]
    return y


def turn_halves(x, positions, dims: int, base: float):
    """x [tokens, heads, dim]: dimension i turns with i + dims/2, over the first `dims` dimensions."""
    if not dims:
        return x
    half = dims // 2
    i = torch.arange(half, dtype=torch.float64)
    freq = torch.pow(torch.tensor(float(base), dtype=torch.float64), -2.0 * i / dims).to(x.dtype)
    a = positions.to(x.dtype)[:, None, None] * freq[None, None, :]
    c, s = torch.cos(a), torch.sin(a)
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., dims:]], dim=-1)


def seen_mask(positions, size: Optional[int], keep_first: int):
    """seen[i, j]: j is not after i, and lies in i's window or among the first tokens, which stay."""
    i, j = positions[:, None], positions[None, :]
    seen = j <= i
    if size is not None:
        seen = seen & ((i - j < size) | (j < keep_first))
    return seen


def capped_sink_attention(q, k, v, seen, scale: float, softcap: Optional[float], sink):
    """q [T, H, d] over k [T, G, d], v [T, G, dv]; scores go through softcap * tanh(s / softcap); the softmax's
    denominator also holds exp(sink) of the head, which has no key and no value. -> [T, H * dv]."""
    H, G = q.shape[1], k.shape[1]
    out = []
    for hd in range(H):
        g = hd // (H // G)
        s = (q[:, hd] @ k[:, g].T) * scale
        if softcap is not None:
            s = softcap * torch.tanh(s / softcap)
        s = s.masked_fill(~seen, float("-inf"))
        if sink is not None:
            s = torch.cat([s, sink[hd].expand(s.shape[0], 1)], dim=1)
        p = torch.softmax(s, dim=-1)
        out.append(p[:, :k.shape[0]] @ v[:, g])
    return torch.cat(out, dim=-1)


def window_attention(h, positions, w, P: str, mx: dict, eps: float):
    T = h.shape[0]
    H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q = (h @ w[f"{P}.q"].T).reshape(T, H, d)
    k = (h @ w[f"{P}.k"].T).reshape(T, G, d)
    v = (h @ w[f"{P}.v"].T).reshape(T, G, dv)
    q = unit_rms(q, eps) * w[f"{P}.q.norm"]
    k = unit_rms(k, eps) * w[f"{P}.k.norm"]
    rot = mx.get("rot") or {"dims": 0, "base": 1.0}
    q = turn_halves(q, positions, rot["dims"], rot["base"])
    k = turn_halves(k, positions, rot["dims"], rot["base"])
    mask = mx.get("mask") or {}
    seen = seen_mask(positions, mask.get("size"), mask.get("keep_first", 0))
    return capped_sink_attention(q, k, v, seen, mx["scale"], mx.get("softcap"), w.get(f"{P}.sink")) @ w[f"{P}.o"].T


def decayed_linear_attention(h, w, P: str, mx: dict, eps: float):
    """S <- decay S + k v^T, o = S^T q with SiLU on q, k and v; the row normed whole, a sigmoid gate."""
    T = h.shape[0]
    H, d, dv = mx["heads"], mx["dim"], mx["vdim"]
    q = silu(h @ w[f"{P}.q"].T).reshape(T, H, d)
    k = silu(h @ w[f"{P}.k"].T).reshape(T, H, d)
    v = silu(h @ w[f"{P}.v"].T).reshape(T, H, dv)
    decay = torch.tensor(mx["decay"], dtype=torch.float64).to(h.dtype)
    S = h.new_zeros(H, d, dv)
    o = h.new_zeros(T, H, dv)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    o = unit_rms(o.reshape(T, H * dv), eps) * w[f"{P}.norm"] * torch.sigmoid(h @ w[f"{P}.g"].T)
    return o @ w[f"{P}.o"].T


def side_by_side(h, positions, w, L: str, mx: dict, eps: float):
    return (mx["left_scale"] * window_attention(h, positions, w, f"{L}.mix.left", mx["left"], eps)
            + mx["right_scale"] * decayed_linear_attention(h, w, f"{L}.mix.right", mx["right"], eps))


def channel_delta(h, w, L: str, mx: dict, eps: float):
    """The gated delta rule with one decay a head and key channel: S <- diag(g) S; u = beta (v - S^T k);
    S <- S + k u^T; o = S^T q."""
    T = h.shape[0]
    H, Hk, dk, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    P = f"{L}.mix"
    q = silu(causal_conv(h @ w[f"{P}.q"].T, w[f"{P}.q.conv"])).reshape(T, Hk, dk)
    k = silu(causal_conv(h @ w[f"{P}.k"].T, w[f"{P}.k.conv"])).reshape(T, Hk, dk)
    v = silu(causal_conv(h @ w[f"{P}.v"].T, w[f"{P}.v.conv"])).reshape(T, H, dv)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * dk ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    per = H // Hk
    q, k = q.repeat_interleave(per, dim=1), k.repeat_interleave(per, dim=1)
    beta = torch.sigmoid(h @ w[f"{P}.b"].T)                                             # [T, H]
    step = softplus((h @ w[f"{P}.a1"].T) @ w[f"{P}.a2"].T + w[f"{P}.dt_bias"]).reshape(T, H, dk)
    g = torch.exp(-torch.exp(w[f"{P}.A_log"])[None, :, None] * step)                    # [T, H, dk]
    S = h.new_zeros(H, dk, dv)
    o = h.new_zeros(T, H, dv)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    o = (unit_rms(o, eps) * w[f"{P}.norm"]).reshape(T, H * dv)
    o = o * torch.sigmoid((h @ w[f"{P}.g1"].T) @ w[f"{P}.g2"].T)
    return o @ w[f"{P}.o"].T


def silu_unit(h, w, P: str):
    return (silu(h @ w[f"{P}.gate"].T) * (h @ w[f"{P}.up"].T)) @ w[f"{P}.down"].T


def run_order(cfg: dict) -> List[int]:
    n = len(cfg["layers"])
    loop = cfg.get("loop") or {"start": 0, "stop": 0, "times": 1}
    inside = list(range(loop["start"], loop["stop"]))
    return list(range(loop["start"])) + inside * loop["times"] + list(range(loop["stop"], n))


def forward(cfg: dict, w, tokens: List[int], dtype=torch.float64, layers_out: Optional[list] = None, order=None,
            inputs_as: Optional[torch.dtype] = None):
    """Logits [tokens, vocab] of one sequence from position 0. `inputs_as`: what every sublayer and the head read is
    rounded to that dtype first (how much such rounding alone moves the logits)."""
    def norm(x, name):
        y = dynamic_tanh(x, w, name)
        return y if inputs_as is None else y.to(inputs_as).to(y.dtype)

    eps, m = cfg["norm"]["eps"], cfg.get("residual_mult", 1.0)
    positions = torch.arange(len(tokens))
    x = w["embed"][torch.tensor(tokens)].to(dtype) * (cfg.get("embedding") or {}).get("scale", 1.0)
    for i in (run_order(cfg) if order is None else order):
        layer = cfg["layers"][i]
        L, kind, mx = f"l{i}", layer["type"], layer["mixer"]
        h = norm(x, f"{L}.norm1")
        if kind == "parallel":
            y = side_by_side(h, positions, w, L, mx, eps)
        elif kind == "channel_delta":
            y = channel_delta(h, w, L, mx, eps)
        else:
            raise ValueError(kind)
        x = x + m * y
        if layer.get("mlp") is not None:
            x = x + m * silu_unit(norm(x, f"{L}.norm2"), w, f"{L}.mlp")
        if layers_out is not None:
            layers_out.append(x.clone())
    return norm(x, "final.norm") @ w["head"].T


class PlainVebusun:
    def __init__(self, model_dir: str, dtype=torch.float64):
        with open(os.path.join(model_dir, "config.json")) as f:
            self.cfg = json.load(f)
        self.dtype = dtype
        self.w = read_tensors(os.path.join(model_dir, "model.safetensors"), dtype)

    def logits(self, tokens: List[int], order=None, layers_out: Optional[list] = None,
               inputs_as: Optional[torch.dtype] = None) -> torch.Tensor:
        return forward(self.cfg, self.w, list(tokens), self.dtype, layers_out, order, inputs_as).to(torch.float32)

    def greedy(self, prompt: List[int], n: int) -> List[int]:
        tokens, out = list(prompt), []
        for _ in range(n):
            nxt = int(self.logits(tokens)[-1].argmax())
            out.append(nxt)
            tokens.append(nxt)
        return out
