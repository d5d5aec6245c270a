"""The Zalunex decoder as data: x = embed[token] + pos[position], then layers that norm on both sides of every sublayer,
x <- x + m * n_b(s(n(x))), the norms' weights stored around zero.  One kind of mixer, ``parallel``: attention over a sliding
window (a norm per head with a weight, no rotation, a learned sink in the softmax, a gate per head) beside lightning attention
(linear attention with a constant decay per head), each with a factor; the two share one product at each end
(``joined_sublayers``).  The feed-forward is none, a gated one whose gate and values are held within a limit, or a mixture of
gelu experts chosen and weighted by sigmoid scores that act on the experts' input.  The logits are capped.  A stretch of layers
may run several times in a row with the same weights: every pass is a layer of its own in the description (caches and states
of its own, the tensors shared by name).
Tensor names: ``l<i>.`` + norm1 | norm1b | norm2 | norm2b | mix.left.* | mix.right.* | mlp.*; ``embed``, ``pos``,
``final.norm``, ``head``.
"""
from ..config.zalunex_config import NAME, ZalunexConfig
from .. import parts  # noqa: F401  (registers the built-in part kinds)
from ..parts.base import LayerSpec, ModelSpec, PartSpec
from ..registry import ARCHITECTURES, Architecture
from .furapel import layer_runs


def _norm(cfg, name, factor=1.0):
    return PartSpec("rmsnorm_chain", {"size": cfg.width, "eps": cfg.eps, "offset": 1.0, "factor": factor, "name": name})


def _mixer(cfg, m, prefix):
    a, r = m.left, m.right
    left = PartSpec("chunk_attention", {
        "heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale, "window": a.window, "sink": "learned",
        "norm_weights": True, "gate": True, "eps": cfg.eps, "out_factor": m.left_scale}, prefix + "left.")
    right = PartSpec("lightning_attention", {"heads": r.heads, "dim": r.dim, "vdim": r.vdim, "decay": r.decay, "eps": cfg.eps,
                                             "out_factor": m.right_scale}, prefix + "right.")
    return PartSpec("joined_sublayers", {"members": (("left", "mixer", left), ("right", "mixer", right))}, prefix)


def _feed_forward(ff, prefix):
    if ff.kind == "dense":
        return PartSpec("gated_mlp", {"intermediate_size": ff.ff, "activation": "clamped", "limit": ff.limit, "partial_out": True}, prefix)
    return PartSpec("routed_experts", {"experts": ff.experts, "top": ff.top, "ff": ff.ff, "routing": "sigmoid", "activation": "gelu",
                                       "weigh": "input"}, prefix)


def zalunex_spec(cfg: ZalunexConfig) -> ModelSpec:
    layers = []
    for i, t, _ in layer_runs(cfg):
        layer, p = cfg.layers[i], f"l{i}."
        parts_ = {"norm_mixer": _norm(cfg, p + "norm1"), "mixer": _mixer(cfg, layer.mixer, p + "mix."),
                  "norm_mixer_out": _norm(cfg, p + "norm1b", cfg.residual_mult)}
        if layer.mlp:
            parts_.update({"norm_ffn": _norm(cfg, p + "norm2"), "ffn": _feed_forward(layer.mlp, p + "mlp."),
                           "norm_ffn_out": _norm(cfg, p + "norm2b", cfg.residual_mult)})
        layers.append(LayerSpec(name=f"l{i}" if t == 0 else f"l{i}.pass{t}", block="sandwich_residual", parts=parts_))
    return ModelSpec(
        architecture=NAME, hidden_size=cfg.width, vocab_size=cfg.vocab,
        embedding=PartSpec("scaled_token_embedding", {"vocab_size": cfg.vocab, "scale": 1.0, "name": "embed",
                                                      "positions": cfg.max_positions, "position_name": "pos"}),
        layers=tuple(layers), schedule=tuple(range(len(layers))),
        final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "tied": False, "name": "head", "softcap": cfg.logit_softcap}),
        max_position=cfg.max_positions, max_position_fixed=True)


ARCHITECTURES.register(NAME, Architecture(NAME, ZalunexConfig, zalunex_spec))
