"""Grouped-query attention over chunks of positions or a sliding window: interleaved rotation, a norm per head after it, a
softmax with a sink, a gate per head.  Every size, constant and tensor name is a parameter."""
from ..registry import MIXERS, POSITIONS
from .base import KVCacheNeed, ParamSpec, PartSpec
from .ends import EndsMixer


@MIXERS.register("chunk_attention")
class ChunkAttention(EndsMixer):
    """q, k, v without biases; q and k are rotated (``position``: a PartSpec, default none), then each head of q and k is
    divided by its own root mean square (eps inside the root), with ``norm_weights`` times a weight of the head's size that all
    heads share; query head h reads KV head h / (heads / kv_heads); score = (q . k) * scale; position i sees j <= i with
    j // chunk == i // chunk, or with ``window`` those with i - j < window (both 0: every earlier token); softmax, with ``sink``
    over a denominator that has one more summand: exp(0) ("zero", or True), or exp(sink_h) with a learned number per head
    ("learned").  ``gate``: head h's output is multiplied by sigmoid(W_g h)_h, one number per head; output projection.
    params: heads, kv_heads, dim, vdim, scale, chunk, window, sink, norm_weights, gate, eps, position, out_factor (on the output,
    default 1).  Tensors under the prefix: q, k, v, o, and where asked for q.norm, k.norm, sink, g."""

    capturable = True
    sub_part_names = ("position",)
    ends_name = "chunk_attention"

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        p = params
        self.nh, self.nkv, self.d, self.dv = p["heads"], p["kv_heads"], p["dim"], p["vdim"]
        if self.nkv <= 0 or self.nh % self.nkv:
            raise ValueError(f"chunk_attention {prefix!r}: heads {self.nh} is not a multiple of kv_heads {self.nkv}")
        pos = p.get("position") or PartSpec("rotary_pairs", {"dims": 0, "base": 10000.0})
        self.position = POSITIONS.get(pos.kind)(pos.params, prefix, ctx)
        self.chunk, self.window, self.sink = p.get("chunk", 0), p.get("window", 0), p.get("sink")
        if self.chunk and self.window:
            raise ValueError(f"chunk_attention {prefix!r}: chunks beside a window are not supported")
        if self.sink not in (None, False, True, "zero", "learned"):
            raise ValueError(f"chunk_attention {prefix!r}: sink {self.sink!r} is not supported (zero | learned)")
        self.gate_at = (self.nh + self.nkv) * self.d + self.nkv * self.dv      # where the gates' columns start, after q, k and v

    def sub_parts(self):
        return (self.position,)

    def in_sources(self):
        H, pre = self.ctx.hidden_size, self.prefix
        sizes = (("q", self.nh * self.d), ("k", self.nkv * self.d), ("v", self.nkv * self.dv)) + ((("g", self.nh),) if self.params.get("gate") else ())
        return tuple((pre + n, (c, H)) for n, c in sizes)

    def out_source(self):
        return (self.prefix + "o", (self.ctx.hidden_size, self.nh * self.dv))

    def own_specs(self):
        specs = []
        if self.params.get("norm_weights"):
            specs += [ParamSpec("q_norm", ((self.prefix + "q.norm", (self.d,)),), role="vector"),
                      ParamSpec("k_norm", ((self.prefix + "k.norm", (self.d,)),), role="vector")]
        if self.sink == "learned":
            specs.append(ParamSpec("sink", ((self.prefix + "sink", (self.nh,)),), role="bias"))
        return specs

    def cache_need(self):
        return KVCacheNeed(self.nkv, self.d, self.window, value_dim=self.dv, chunk=self.chunk)

    def flops(self, rows, attended=0):
        seen = min(attended, rows * (self.chunk + 1) // 2) if self.chunk else min(attended, rows * self.window) if self.window else attended
        return super().flops(rows) + 2.0 * seen * (self.d + self.dv) * self.nh

    def between(self, step, h, proj, out):
        ops, p, w = self.ctx.ops, self.params, self.w
        g, T = self.cache.group, step.rows
        kc, vc = self.cache.k(self.cache_index), self.cache.v(self.cache_index)
        q = step.ws("ca_q", (T, self.nh * self.d))
        slots = step.slots(g) if self.cache_owner else None
        ops.head_norm_store(proj, q, self.nh, self.nkv, self.d, self.dv, p["eps"], q_weight=w.get("q_norm"), k_weight=w.get("k_norm"), plain_norm=True, cos_sin=self.position.pairs_table(step),
                            rot=self.position.params["dims"], slots=slots, kcache=kc, vcache=vc, rows=T)
        rule = dict(chunk=self.chunk, sink=w.get("sink", bool(self.sink)), out_scale=p.get("out_factor", 1.0))
        if p.get("gate"):
            rule.update(gate=proj[:, self.gate_at:], gate_heads=True)
        if step.max_run > 1 and ops.attention_window_pool_tiles_supported(self.d, self.dv, out.dtype, kc.shape[2]):
            ops.attention_window_pool_tiles(q, out, kc, vc, None, None, step.tables(g), step.table_stride(g), step.run_start,
                                            step.seq_start, step.seqs, step.max_run, self.nh, self.nkv, self.d, self.dv, p["scale"], self.window, 0, **rule)
        else:
            ops.attention_window_pool(q, out, kc, vc, None, None, step.tables(g), step.table_stride(g), step.row_seq, step.ctx_lens,
                                      self.nh, self.nkv, self.d, self.dv, p["scale"], self.window, 0, rows=T, **rule)
