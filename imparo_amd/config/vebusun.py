"""Typed Vebusun configuration and its plan.

A Vebusun model is a pre-norm decoder whose layers are listed one by one in
config.json (`layers`: each with a `type`, the `mixer`'s sizes and an `mlp` or
null), a run of which (`loop`) is gone through several times in a row with the
same weights and a cache or state of its own a pass. The norm computes no
statistic: tanh(alpha x) w + b. Each sublayer's result is multiplied by
`residual_mult` before it joins the stream, and the embedding's rows by
`embedding.scale`.

Mixers: `parallel` (two side by side on one input, `left_scale` and
`right_scale` times their results summed: softmax attention with head norms, a
rotation in halves of part of a head, capped scores, a window beside which the
first tokens stay visible, and a learned sink a head; and lightning attention,
linear attention with SiLU on q, k and v and a fixed decay a head) and
`channel_delta` (the gated delta rule with one decay a head and key channel).
Feed-forward: `dense`, a SwiGLU unit. Every size and every constant that may
differ between models comes from the file or a tensor's shape; what the file
leaves out (a mask, a rotation, a cap, a loop, an mlp) is not there.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from .errors import BadValue, Inconsistent, MissingKey
from .mepapel import _object, _rotation
from .plan import LayerCall, LayerPlan, ModelPlan, PartSpec
from .tumadra import _int, _num

ARCHITECTURE = "Vebusun"
MIXER_KINDS = ("parallel", "channel_delta")
MAX_POSITION = 1 << 30        # positions are int32 and enter only through angles and masks

_DELTA_KEYS = ("heads", "kv_heads", "dim", "vdim", "conv")
_LEFT_KEYS = ("heads", "kv_heads", "dim", "vdim")
_RIGHT_KEYS = ("heads", "dim", "vdim")


@dataclass
class VebusunLayer:
    type: str
    mixer: Dict[str, Any]
    ff: Optional[int]          # the feed-forward's hidden width, None: no feed-forward


@dataclass
class VebusunConfig:
    vocab: int
    width: int
    layers: List[VebusunLayer]
    norm_eps: float
    embedding_scale: float = 1.0
    residual_mult: float = 1.0
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 1
    raw: Dict[str, Any] = field(default_factory=dict)
    unread_keys: List[str] = field(default_factory=list)

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "VebusunConfig":
        for key in ("vocab", "width", "layers", "norm"):
            if key not in d:
                raise MissingKey(f"config.json: required key {key!r} is missing")
        if not isinstance(d["norm"], dict):
            raise BadValue("config.json: norm must be an object with eps")
        if not isinstance(d["layers"], list) or not d["layers"]:
            raise BadValue("config.json: layers must be a non-empty list")
        embedding = _object(d, "embedding", "the model", required=False) or {}
        cfg = cls(vocab=_int(d, "vocab", "the model"), width=_int(d, "width", "the model"),
                  layers=[cls._layer(i, entry) for i, entry in enumerate(d["layers"])],
                  norm_eps=_num(d["norm"], "eps", "norm"),
                  embedding_scale=_num(embedding, "scale", "embedding") if "scale" in embedding else 1.0,
                  residual_mult=_num(d, "residual_mult", "the model") if "residual_mult" in d else 1.0, raw=d)
        loop = _object(d, "loop", "the model", required=False)
        if loop is not None:
            cfg.loop_start, cfg.loop_stop = _int(loop, "start", "loop", 0), _int(loop, "stop", "loop", 0)
            cfg.loop_times = _int(loop, "times", "loop", 1)
        known = {"architecture", "architectures", "vocab", "width", "layers", "norm", "residual_mult", "embedding", "loop"}
        cfg.unread_keys = sorted(k for k in d if k not in known)
        if cfg.norm_eps <= 0:
            raise BadValue("norm.eps must be positive")
        if not 0 <= cfg.loop_start <= cfg.loop_stop <= len(cfg.layers):
            raise Inconsistent(f"loop {cfg.loop_start}..{cfg.loop_stop} does not lie inside {len(cfg.layers)} layers")
        return cfg

    @staticmethod
    def _layer(i: int, entry: Any) -> VebusunLayer:
        where = f"layers[{i}]"
        if not isinstance(entry, dict) or "type" not in entry or "mixer" not in entry:
            raise BadValue(f"config.json: {where} must be an object with type, mixer and mlp")
        kind = entry["type"]
        if kind not in MIXER_KINDS:
            raise BadValue(f"config.json: {where}.type is {kind!r}; known mixers are {', '.join(MIXER_KINDS)}")
        mixer = entry["mixer"]
        if not isinstance(mixer, dict):
            raise BadValue(f"config.json: {where}.mixer must be an object")
        w = f"{where}.mixer"
        if kind == "channel_delta":
            parsed = {key: _int(mixer, key, w) for key in _DELTA_KEYS}
            if parsed["heads"] % parsed["kv_heads"]:
                raise Inconsistent(f"{w}: {parsed['heads']} heads on {parsed['kv_heads']} query/key heads")
        else:
            parsed = dict(left=VebusunConfig._left(_object(mixer, "left", w), f"{w}.left"),
                          right=VebusunConfig._right(_object(mixer, "right", w), f"{w}.right"),
                          left_scale=_num(mixer, "left_scale", w), right_scale=_num(mixer, "right_scale", w))
        mlp = _object(entry, "mlp", where, required=False)
        ff = None
        if mlp is not None:
            if mlp.get("kind") != "dense":
                raise BadValue(f"config.json: {where}.mlp.kind is {mlp.get('kind')!r}; only 'dense' is known")
            ff = _int(mlp, "ff", f"{where}.mlp")
        return VebusunLayer(kind, parsed, ff)

    @staticmethod
    def _left(m: Dict[str, Any], w: str) -> Dict[str, Any]:
        out = {key: _int(m, key, w) for key in _LEFT_KEYS}
        if out["heads"] % out["kv_heads"]:
            raise Inconsistent(f"{w}: {out['heads']} heads on {out['kv_heads']} key/value heads")
        mask = _object(m, "mask", w, required=False)
        out.update(scale=_num(m, "scale", w), rot=_rotation(m, w, out["dim"]), softcap=None, window=None, keep_first=0)
        if m.get("softcap") is not None:
            out["softcap"] = _num(m, "softcap", w)
            if not out["softcap"] > 0:
                raise BadValue(f"config.json: {w}.softcap must be positive")
        if mask is not None:
            out["window"] = _int(mask, "size", f"{w}.mask")
            out["keep_first"] = _int(mask, "keep_first", f"{w}.mask", 0) if mask.get("keep_first") is not None else 0
        return out

    @staticmethod
    def _right(m: Dict[str, Any], w: str) -> Dict[str, Any]:
        out: Dict[str, Any] = {key: _int(m, key, w) for key in _RIGHT_KEYS}
        decay = m.get("decay")
        if not isinstance(decay, list) or len(decay) != out["heads"] or any(
                isinstance(x, bool) or not isinstance(x, (int, float)) or not math.isfinite(x) for x in decay):
            raise BadValue(f"config.json: {w}.decay must be a list of one number a head")
        out["decay"] = [float(x) for x in decay]
        return out

    def order(self) -> List[int]:
        """Layers in the order they run: those of the loop `times` times in a row."""
        inside = list(range(self.loop_start, self.loop_stop))
        return list(range(self.loop_start)) + inside * self.loop_times + list(range(self.loop_stop, len(self.layers)))

    def to_dict(self) -> Dict[str, Any]:
        return dict(self.raw)


def build_plan(cfg: VebusunConfig) -> ModelPlan:
    E, eps, m = cfg.width, cfg.norm_eps, cfg.residual_mult
    norm = lambda name: PartSpec("dynamic_tanh", "", dict(width=E, tensor=name))
    layers: List[LayerPlan] = []
    for i, layer in enumerate(cfg.layers):
        base, x = f"l{i}", layer.mixer
        if layer.type == "channel_delta":
            mixer = PartSpec("channel_delta", f"{base}.mix", dict(
                width=E, heads=x["heads"], kv_heads=x["kv_heads"], dim=x["dim"], vdim=x["vdim"], taps=x["conv"], eps=eps,
                out_scale=m))
        else:
            a, b = x["left"], x["right"]
            rot = a["rot"] and PartSpec("rope_neox", "", dict(rotary_dim=a["rot"]["dims"], base=a["rot"]["base"], precise=True))
            left = PartSpec("attention", f"{base}.mix.left", dict(
                width=E, heads=a["heads"], kv_heads=a["kv_heads"], head_dim=a["dim"], value_dim=a["vdim"], scale=a["scale"],
                window=a["window"], keep_first=a["keep_first"], softcap=a["softcap"], sink="sink", weight_suffix="",
                qk_norm=PartSpec("rms_norm", "", dict(eps=eps)), exact_weights=True, out_scale=x["left_scale"] * m,
                names=dict(q="q", k="k", v="v", o="o", q_norm="q.norm", k_norm="k.norm"), position=rot))
            right = PartSpec("retention", f"{base}.mix.right", dict(
                width=E, heads=b["heads"], dim=b["dim"], vdim=b["vdim"], decay=b["decay"], eps=eps, silu_in=True,
                key_scale=1.0, norm="norm", gate="sigmoid", out_scale=x["right_scale"] * m))
            mixer = PartSpec("mixer_pair", f"{base}.mix", dict(width=E, eps=eps, left=left, right=right, normed=False))
        parts = dict(mixer_norm=("norm", norm(f"{base}.norm1")), mixer=("mixer", mixer))
        if layer.ff is not None:
            parts["ffn_norm"] = ("norm", norm(f"{base}.norm2"))
            parts["ffn"] = ("feed_forward", PartSpec("swiglu", f"{base}.mlp", dict(
                width=E, hidden=layer.ff, weight_suffix="", names=dict(gate="gate", up="up", down="down"), out_scale=m)))
        layers.append(LayerPlan(parts, "pre_norm"))
    plan = ModelPlan(
        architecture=ARCHITECTURE,
        vocab_size=cfg.vocab,
        hidden_size=E,
        max_position=MAX_POSITION,
        embedding=PartSpec("embedding", "embed", dict(vocab=cfg.vocab, width=E, tensor="embed", scale=cfg.embedding_scale)),
        layers=layers,
        order=[LayerCall(i) for i in cfg.order()],
        final_norm=norm("final.norm"),
        head=PartSpec("linear_head", "head", dict(vocab=cfg.vocab, width=E, tensor="head")),
    )
    plan.validate()
    return plan
