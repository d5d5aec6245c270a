"""Typed configuration of the Zalunex decoder, read from the nested keys of its config.json.

  architecture    "Zalunex"
  vocab, width    sizes of the vocabulary and of the residual stream
  max_positions   how many positions have a learned vector: the longest sequence
  norm.eps        epsilon of every root-mean-square division
  residual_mult   a factor on what a sublayer adds to the stream
  logit_softcap   cap c on the logits, c tanh(logits / c) (absent or null: none)
  layers[i]       type: "parallel"; mixer: its sizes; mlp: null, {kind: "dense", ff, limit} or
                  {kind: "moe", expert: {ff}, router: {experts, top}}
  loop            {start, stop, times} or absent: layers start .. stop-1 run ``times`` times in a row, each pass with
                  caches and states of its own

The mixer: left (attention: heads, kv_heads, dim, vdim, scale, mask {size} or absent: every earlier token), right (lightning
attention: heads, dim, vdim, decay [one number per head]), left_scale, right_scale.  kv_heads defaults to heads, vdim to dim,
residual_mult and both scales to 1.
"""
from dataclasses import dataclass
from typing import Optional, Tuple

from .fisesun_config import _object
from .furapel_config import LoopConfig
from .kasuvik_config import _number, _pos_int
from .model_config import ConfigError

NAME = "Zalunex"
MIXERS = ("parallel",)


@dataclass(frozen=True)
class WindowAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: int = 0

    def to_dict(self):
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.window:
            d["mask"] = {"size": self.window}
        return d


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    def to_dict(self):
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}


@dataclass(frozen=True)
class ParallelConfig:
    left: WindowAttentionConfig
    right: LightningConfig
    left_scale: float = 1.0
    right_scale: float = 1.0

    def to_dict(self):
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale, "right_scale": self.right_scale}


@dataclass(frozen=True)
class FeedForwardConfig:
    """kind "dense": one feed-forward of ``ff`` columns whose gate and values are held within ``limit``.  kind "moe": ``experts``
    experts of ``ff`` columns without gates, of which a token uses ``top``."""
    kind: str
    ff: int
    limit: float = 0.0
    experts: int = 0
    top: int = 0

    def to_dict(self):
        if self.kind == "dense":
            return {"kind": "dense", "ff": self.ff, "limit": self.limit}
        return {"kind": "moe", "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top}}


@dataclass(frozen=True)
class ZalunexLayer:
    type: str
    mixer: ParallelConfig
    mlp: Optional[FeedForwardConfig] = None

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": self.mlp.to_dict() if self.mlp else None}


def _attention(problems, w, m):
    heads, dim = _pos_int(problems, w, m, "heads"), _pos_int(problems, w, m, "dim")
    kv = _pos_int(problems, w, m, "kv_heads") if "kv_heads" in m else heads
    if heads % kv:
        problems.append(f"{w}: heads {heads} is not a multiple of kv_heads {kv}")
    mask = _object(problems, w, m, "mask")
    return WindowAttentionConfig(heads=heads, kv_heads=kv, dim=dim, vdim=_pos_int(problems, w, m, "vdim") if "vdim" in m else dim,
                                 scale=_number(problems, w, m, "scale", positive=False),
                                 window=_pos_int(problems, w + ".mask", mask, "size") if mask is not None else 0)


def _lightning(problems, w, m):
    heads, dim, decay = _pos_int(problems, w, m, "heads"), _pos_int(problems, w, m, "dim"), m.get("decay")
    if not isinstance(decay, list) or not all(isinstance(x, (int, float)) and not isinstance(x, bool) for x in decay):
        problems.append(f"{w}.decay must be a list of numbers")
        decay = []
    elif len(decay) != heads:
        problems.append(f"{w}.decay has {len(decay)} numbers for {heads} heads")
    elif not all(0.0 <= x <= 1.0 for x in decay):
        problems.append(f"{w}.decay must lie between 0 and 1")
    return LightningConfig(heads=heads, dim=dim, vdim=_pos_int(problems, w, m, "vdim") if "vdim" in m else dim,
                           decay=tuple(float(x) for x in decay))


def _parallel(problems, w, m):
    left, right = _object(problems, w, m, "left"), _object(problems, w, m, "right")
    if left is None or right is None:
        problems.append(f"{w} needs 'left' and 'right'")
        return None
    scale = lambda key: _number(problems, w, m, key, positive=False) if key in m else 1.0
    return ParallelConfig(_attention(problems, w + ".left", left), _lightning(problems, w + ".right", right),
                          scale("left_scale"), scale("right_scale"))


def _feed_forward(problems, w, mlp):
    kind = mlp.get("kind")
    if kind == "dense":
        return FeedForwardConfig("dense", _pos_int(problems, w, mlp, "ff"), limit=_number(problems, w, mlp, "limit"))
    if kind == "moe":
        router = _object(problems, w, mlp, "router") or {}
        cfg = FeedForwardConfig("moe", _pos_int(problems, w + ".expert", mlp.get("expert"), "ff"),
                                experts=_pos_int(problems, w + ".router", router, "experts"), top=_pos_int(problems, w + ".router", router, "top"))
        if cfg.top > cfg.experts:
            problems.append(f"{w}.router.top {cfg.top} exceeds its {cfg.experts} experts")
        return cfg
    problems.append(f"{w}.kind {kind!r} is not supported (dense | moe, or a null mlp)")
    return None


@dataclass(frozen=True)
class ZalunexConfig:
    vocab: int
    width: int
    max_positions: int
    eps: float
    layers: Tuple[ZalunexLayer, ...]
    residual_mult: float = 1.0
    logit_softcap: float = 0.0
    loop: Optional[LoopConfig] = None

    @classmethod
    def from_dict(cls, raw: dict) -> "ZalunexConfig":
        problems = []
        vocab, width = _pos_int(problems, "config", raw, "vocab"), _pos_int(problems, "config", raw, "width")
        positions = _pos_int(problems, "config", raw, "max_positions")
        eps = _number(problems, "norm", raw.get("norm"), "eps")
        mult = _number(problems, "config", raw, "residual_mult", positive=False) if "residual_mult" in raw else 1.0
        cap = _number(problems, "config", raw, "logit_softcap") if raw.get("logit_softcap") is not None else 0.0
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
            if entry.get("type") not in MIXERS:
                problems.append(f"{where}.type {entry.get('type')!r} is not supported ({' | '.join(MIXERS)})")
                continue
            ff, mlp = None, entry.get("mlp")
            if mlp is not None:
                if not isinstance(mlp, dict):
                    problems.append(f"{where}.mlp must be an object or null")
                else:
                    ff = _feed_forward(problems, where + ".mlp", mlp)
            layers.append(ZalunexLayer(entry["type"], _parallel(problems, where + ".mixer", entry["mixer"]), ff))
        loop, lp = None, _object(problems, "config", raw, "loop")
        if lp is not None:
            loop = LoopConfig(start=_pos_int(problems, "loop", lp, "start", allow_zero=True), stop=_pos_int(problems, "loop", lp, "stop"),
                              times=_pos_int(problems, "loop", lp, "times"))
            if not loop.start < loop.stop <= max(len(listed), 1):
                problems.append(f"loop: layers {loop.start} .. {loop.stop - 1} are not a stretch of the model's {len(listed)} layers")
        if problems:
            raise ConfigError("config.json: " + "; ".join(problems))
        return cls(vocab=vocab, width=width, max_positions=positions, eps=eps, layers=tuple(layers), residual_mult=mult, logit_softcap=cap,
                   loop=loop)

    def to_dict(self) -> dict:
        d = {"architecture": NAME, "vocab": self.vocab, "width": self.width, "max_positions": self.max_positions, "norm": {"eps": self.eps},
             "residual_mult": self.residual_mult, "layers": [l.to_dict() for l in self.layers]}
        if self.logit_softcap:
            d["logit_softcap"] = self.logit_softcap
        if self.loop:
            d["loop"] = self.loop.to_dict()
        return d
