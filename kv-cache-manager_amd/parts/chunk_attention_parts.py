"""Grouped-query attention over chunks of positions: interleaved rotation, a norm per head without a weight after it, a
softmax with a sink.  Every size, constant and tensor name is a parameter."""
from ..registry import MIXERS, POSITIONS
from .base import KVCacheNeed, ParamSpec, PartSpec
from .ends import EndsMixer


@MIXERS.register("chunk_attention")
class ChunkAttention(EndsMixer):
    """q, k, v without biases; q and k are rotated (``position``: a PartSpec, default none), then each head of q and k is
    divided by its own root mean square (eps inside the root, no weight); query head h reads KV head h / (heads / kv_heads);
    score = (q . k) * scale; position i sees j <= i with j // chunk == i // chunk (chunk 0: every earlier token); softmax,
    with ``sink`` over a denominator that has one more summand, exp(0); output projection.
    params: heads, kv_heads, dim, vdim, scale, chunk, sink, eps, position, out_factor (on the output, default 1).
    Tensors under the prefix: q, k, v, o."""

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
        self.chunk, self.sink = p.get("chunk", 0), bool(p.get("sink"))

    def sub_parts(self):
        return (self.position,)

    def in_sources(self):
        H, pre = self.ctx.hidden_size, self.prefix
        return tuple((pre + n, (c, H)) for n, c in (("q", self.nh * self.d), ("k", self.nkv * self.d), ("v", self.nkv * self.dv)))

    def out_source(self):
        return (self.prefix + "o", (self.ctx.hidden_size, self.nh * self.dv))

    def cache_need(self):
        return KVCacheNeed(self.nkv, self.d, value_dim=self.dv, chunk=self.chunk)

    def flops(self, rows, attended=0):
        seen = min(attended, rows * (self.chunk + 1) // 2) if self.chunk else attended
        return super().flops(rows) + 2.0 * seen * (self.d + self.dv) * self.nh

    def between(self, step, h, proj, out):
        ops, p = self.ctx.ops, self.params
        g, T = self.cache.group, step.rows
        kc, vc = self.cache.k(self.cache_index), self.cache.v(self.cache_index)
        q = step.ws("ca_q", (T, self.nh * self.d))
        slots = step.slots(g) if self.cache_owner else None
        ops.head_norm_store(proj, q, self.nh, self.nkv, self.d, self.dv, p["eps"], plain_norm=True, cos_sin=self.position.pairs_table(step),
                            rot=self.position.params["dims"], slots=slots, kcache=kc, vcache=vc, rows=T)
        rule = dict(chunk=self.chunk, sink=self.sink, out_scale=p.get("out_factor", 1.0))
        if step.max_run > 1 and ops.attention_window_pool_tiles_supported(self.d, self.dv, out.dtype, kc.shape[2]):
            ops.attention_window_pool_tiles(q, out, kc, vc, None, None, step.tables(g), step.table_stride(g), step.run_start,
                                            step.seq_start, step.seqs, step.max_run, self.nh, self.nkv, self.d, self.dv, p["scale"], 0, 0, **rule)
        else:
            ops.attention_window_pool(q, out, kc, vc, None, None, step.tables(g), step.table_stride(g), step.row_seq, step.ctx_lens,
                                      self.nh, self.nkv, self.d, self.dv, p["scale"], 0, 0, rows=T, **rule)
