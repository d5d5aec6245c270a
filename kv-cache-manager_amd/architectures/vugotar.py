"""The Vugotar decoder as data: parallel layers, h = rms(x) * (1 + w), x <- x + (mixer(h) + ff(h)), one norm a layer.  Two
kinds of mixer: ``parallel`` (attention over chunks with an interleaved rotation, a norm per head and a sink in its softmax,
beside a gated delta rule, each with a factor) and ``mamba2`` (the state-space recurrence with one decay per head).  The
feed-forward is a dense gated one with biases, or a mixture of gated experts weighted over the chosen ones beside a shared
expert with a gate.  A layer's sublayers share one product at each end (``joined_sublayers``).  A stretch of layers may run
several times in a row with the same weights: every pass is a layer of its own in the description (caches and states of its
own, the tensors shared by name), and before each pass but the first the embedding's output is added to the stream again.
Tensor names: ``l<i>.`` + norm1 | mix.* (mix.left.*, mix.right.*) | mlp.*; ``embed``, ``final.norm``, ``head``.
"""
from ..config.vugotar_config import NAME, VugotarConfig
from .. import parts  # noqa: F401  (registers the built-in part kinds)
from ..parts.base import LayerSpec, ModelSpec, PartSpec
from ..registry import ARCHITECTURES, Architecture
from .furapel import layer_runs


def _norm(cfg, name):
    return PartSpec("offset_rmsnorm", {"size": cfg.width, "eps": cfg.eps, "offset": 1.0, "name": name})


def _mixers(cfg, layer, prefix):
    m = layer.mixer
    if layer.type == "mamba2":
        return [("mamba2", "mixer", PartSpec("state_space_duality", {
            "heads": m.heads, "vdim": m.vdim, "state": m.state, "groups": m.groups, "norm_groups": m.norm_groups, "conv": m.conv,
            "eps": cfg.eps}, prefix))]
    a, r = m.left, m.right
    position = PartSpec("rotary_pairs", {"dims": a.rot_dims, "base": a.rot_base}) if a.rot_dims else None
    return [("left", "mixer", PartSpec("chunk_attention", {
                "heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale, "chunk": a.chunk, "sink": True,
                "eps": cfg.eps, "position": position, "out_factor": m.left_scale}, prefix + "left.")),
            ("right", "mixer", PartSpec("gated_delta", {
                "heads": r.heads, "kv_heads": r.kv_heads, "dim": r.dim, "vdim": r.vdim, "conv": r.conv, "eps": cfg.eps,
                "out_factor": m.right_scale}, prefix + "right."))]


def _feed_forward(ff, prefix):
    if ff.kind == "dense":
        return PartSpec("gated_mlp", {"intermediate_size": ff.ff, "activation": "silu", "bias": True}, prefix)
    shared = PartSpec("gated_mlp", {"intermediate_size": ff.shared_ff, "activation": "silu"}, prefix + "shared.") if ff.shared_ff else None
    return PartSpec("routed_experts", {"experts": ff.experts, "top": ff.top, "ff": ff.ff, "routing": "softmax_chosen", "route_factor": ff.scale,
                                       "activation": "silu_gated", "shared": shared, "shared_gate": "shared.sg" if shared else None}, prefix)


def vugotar_spec(cfg: VugotarConfig) -> ModelSpec:
    layers = []
    for i, t, leads in layer_runs(cfg):
        layer, p = cfg.layers[i], f"l{i}."
        members = _mixers(cfg, layer, p + "mix.")
        if layer.mlp:
            members.append(("ffn", "ffn", _feed_forward(layer.mlp, p + "mlp.")))
        parts_ = {"norm": _norm(cfg, p + "norm1"), "mixer": PartSpec("joined_sublayers", {"members": tuple(members)}, p)}
        if leads and t > 0:
            parts_["again"] = PartSpec("embedding_again")
        layers.append(LayerSpec(name=f"l{i}" if t == 0 else f"l{i}.pass{t}", block="parallel_residual", parts=parts_))
    return ModelSpec(
        architecture=NAME, hidden_size=cfg.width, vocab_size=cfg.vocab,
        embedding=PartSpec("scaled_token_embedding", {"vocab_size": cfg.vocab, "scale": 1.0, "name": "embed"}),
        layers=tuple(layers), schedule=tuple(range(len(layers))),
        final_norm=_norm(cfg, "final.norm"),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "tied": False, "name": "head"}),
        max_position=0, keep_embedding=cfg.loop is not None and cfg.loop.times > 1)


ARCHITECTURES.register(NAME, Architecture(NAME, VugotarConfig, vugotar_spec))
