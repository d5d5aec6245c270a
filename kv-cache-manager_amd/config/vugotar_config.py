"""Typed configuration of the Vugotar decoder, read from the nested keys of its config.json.

  architecture    "Vugotar"
  vocab, width    sizes of the vocabulary and of the residual stream
  norm.eps        epsilon of every root-mean-square division
  layers[i]       type: "parallel" | "mamba2"; mixer: that mixer's sizes; mlp: null, {kind: "dense", ff} or
                  {kind: "moe", expert: {ff}, router: {experts, top, scale}, shared: {ff} or absent}
  loop            {start, stop, times} or absent: layers start .. stop-1 run ``times`` times in a row, each pass with
                  caches and states of its own; before each pass but the first the embedding's output is added again

Mixers.  parallel: left (attention: heads, kv_heads, dim, vdim, scale, mask {size} or absent: every earlier token, rot
{dims, base} or absent: no rotation), right (gated delta rule: heads, kv_heads, dim, vdim, conv taps), left_scale,
right_scale.  mamba2: heads, vdim, state, groups, norm_groups, conv taps.  kv_heads defaults to heads, vdim to dim,
rot.base to 10000, both scales, router.scale, groups and norm_groups to 1.
"""
from dataclasses import dataclass
from typing import Optional, Tuple

from .fisesun_config import _object
from .furapel_config import LoopConfig
from .kasuvik_config import _number, _pos_int
from .model_config import ConfigError

NAME = "Vugotar"
MIXERS = ("parallel", "mamba2")


@dataclass(frozen=True)
class ChunkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int = 0
    rot_dims: int = 0
    rot_base: float = 10000.0

    def to_dict(self):
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.chunk:
            d["mask"] = {"size": self.chunk}
        if self.rot_dims:
            d["rot"] = {"dims": self.rot_dims, "base": self.rot_base}
        return d


@dataclass(frozen=True)
class GatedDeltaConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int

    def to_dict(self):
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv}


@dataclass(frozen=True)
class ParallelConfig:
    left: ChunkAttentionConfig
    right: GatedDeltaConfig
    left_scale: float = 1.0
    right_scale: float = 1.0

    def to_dict(self):
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale, "right_scale": self.right_scale}


@dataclass(frozen=True)
class Mamba2Config:
    heads: int
    vdim: int
    state: int
    groups: int
    norm_groups: int
    conv: int

    def to_dict(self):
        return {"heads": self.heads, "vdim": self.vdim, "state": self.state, "groups": self.groups, "norm_groups": self.norm_groups,
                "conv": self.conv}


@dataclass(frozen=True)
class FeedForwardConfig:
    """kind "dense": one gated feed-forward of ``ff`` columns, with biases.  kind "moe": ``experts`` gated experts of ``ff``
    columns of which a token uses ``top``, their weights times ``scale``, and a shared expert of ``shared_ff`` columns with a
    gate of its own (0: none)."""
    kind: str
    ff: int
    experts: int = 0
    top: int = 0
    scale: float = 1.0
    shared_ff: int = 0

    def to_dict(self):
        if self.kind == "dense":
            return {"kind": "dense", "ff": self.ff}
        d = {"kind": "moe", "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top, "scale": self.scale}}
        if self.shared_ff:
            d["shared"] = {"ff": self.shared_ff}
        return d


@dataclass(frozen=True)
class VugotarLayer:
    type: str
    mixer: object
    mlp: Optional[FeedForwardConfig] = None

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None}


def _multiple(problems, where, what, n, of, m):
    if n % m:
        problems.append(f"{where}: {what} {n} is not a multiple of {of} {m}")


def _heads(problems, w, m):
    heads, dim = _pos_int(problems, w, m, "heads"), _pos_int(problems, w, m, "dim")
    kv = _pos_int(problems, w, m, "kv_heads") if "kv_heads" in m else heads
    _multiple(problems, w, "heads", heads, "kv_heads", kv)
    return heads, kv, dim, _pos_int(problems, w, m, "vdim") if "vdim" in m else dim


def _attention(problems, w, m):
    heads, kv, dim, vdim = _heads(problems, w, m)
    rot, dims, base = _object(problems, w, m, "rot"), 0, 10000.0
    if rot is not None:
        dims = _pos_int(problems, w + ".rot", rot, "dims", allow_zero=True)
        if dims and "base" in rot:
            base = _number(problems, w + ".rot", rot, "base")
    if dims % 2 or dims > dim:
        problems.append(f"{w}.rot.dims {dims} must be even and at most dim {dim}")
    mask = _object(problems, w, m, "mask")
    return ChunkAttentionConfig(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=_number(problems, w, m, "scale", positive=False),
                                chunk=_pos_int(problems, w + ".mask", mask, "size") if mask is not None else 0, rot_dims=dims, rot_base=base)


def _parallel(problems, w, m):
    left, right = _object(problems, w, m, "left"), _object(problems, w, m, "right")
    if left is None or right is None:
        problems.append(f"{w} needs 'left' and 'right'")
        return None
    heads, kv, dim, vdim = _heads(problems, w + ".right", right)
    delta = GatedDeltaConfig(heads, kv, dim, vdim, _pos_int(problems, w + ".right", right, "conv"))
    scale = lambda key: _number(problems, w, m, key, positive=False) if key in m else 1.0
    return ParallelConfig(_attention(problems, w + ".left", left), delta, scale("left_scale"), scale("right_scale"))


def _mamba2(problems, w, m):
    one = lambda key: _pos_int(problems, w, m, key) if key in m else 1
    cfg = Mamba2Config(heads=_pos_int(problems, w, m, "heads"), vdim=_pos_int(problems, w, m, "vdim"), state=_pos_int(problems, w, m, "state"),
                       groups=one("groups"), norm_groups=one("norm_groups"), conv=_pos_int(problems, w, m, "conv"))
    _multiple(problems, w, "heads", cfg.heads, "groups", cfg.groups)
    _multiple(problems, w, "heads x vdim", cfg.heads * cfg.vdim, "norm_groups", cfg.norm_groups)
    return cfg


def _feed_forward(problems, w, mlp):
    kind = mlp.get("kind")
    if kind == "dense":
        return FeedForwardConfig("dense", _pos_int(problems, w, mlp, "ff"))
    if kind == "moe":
        router, shared = _object(problems, w, mlp, "router") or {}, _object(problems, w, mlp, "shared")
        cfg = FeedForwardConfig("moe", _pos_int(problems, w + ".expert", mlp.get("expert"), "ff"),
                                experts=_pos_int(problems, w + ".router", router, "experts"), top=_pos_int(problems, w + ".router", router, "top"),
                                scale=_number(problems, w + ".router", router, "scale", positive=False) if "scale" in router else 1.0,
                                shared_ff=_pos_int(problems, w + ".shared", shared, "ff") if shared is not None else 0)
        if cfg.top > cfg.experts:
            problems.append(f"{w}.router.top {cfg.top} exceeds its {cfg.experts} experts")
        return cfg
    problems.append(f"{w}.kind {kind!r} is not supported (dense | moe, or a null mlp)")
    return None


@dataclass(frozen=True)
class VugotarConfig:
    vocab: int
    width: int
    eps: float
    layers: Tuple[VugotarLayer, ...]
    loop: Optional[LoopConfig] = None

    @classmethod
    def from_dict(cls, raw: dict) -> "VugotarConfig":
        problems = []
        vocab, width = _pos_int(problems, "config", raw, "vocab"), _pos_int(problems, "config", raw, "width")
        eps = _number(problems, "norm", raw.get("norm"), "eps")
        listed = raw.get("layers")
        if not isinstance(listed, list) or not listed:
            problems.append("'layers' must be a non-empty list")
            listed = []
        layers = []
        for i, entry in enumerate(listed):
            where = f"layers[{i}]"
            if not isinstance(entry, dict) or not isinstance(entry.get("mixer"), dict):
                problems.append(f"{where} must be an object with 'type' and 'mixer'")
                continue
            kind, mixer, mlp = entry.get("type"), entry["mixer"], entry.get("mlp")
            ff = None
            if mlp is not None:
                if not isinstance(mlp, dict):
                    problems.append(f"{where}.mlp must be an object or null")
                else:
                    ff = _feed_forward(problems, where + ".mlp", mlp)
            if kind == "parallel":
                layers.append(VugotarLayer(kind, _parallel(problems, where + ".mixer", mixer), ff))
            elif kind == "mamba2":
                layers.append(VugotarLayer(kind, _mamba2(problems, where + ".mixer", mixer), ff))
            else:
                problems.append(f"{where}.type {kind!r} is not supported ({' | '.join(MIXERS)})")
        loop, lp = None, _object(problems, "config", raw, "loop")
        if lp is not None:
            loop = LoopConfig(start=_pos_int(problems, "loop", lp, "start", allow_zero=True), stop=_pos_int(problems, "loop", lp, "stop"),
                              times=_pos_int(problems, "loop", lp, "times"))
            if not loop.start < loop.stop <= max(len(listed), 1):
                problems.append(f"loop: layers {loop.start} .. {loop.stop - 1} are not a stretch of the model's {len(listed)} layers")
        if problems:
            raise ConfigError("config.json: " + "; ".join(problems))
        return cls(vocab=vocab, width=width, eps=eps, layers=tuple(layers), loop=loop)

    def to_dict(self) -> dict:
        d = {"architecture": NAME, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "layers": [l.to_dict() for l in self.layers]}
        if self.loop:
            d["loop"] = self.loop.to_dict()
        return d
