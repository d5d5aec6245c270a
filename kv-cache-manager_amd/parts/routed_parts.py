"""A routed feed-forward (mixture of experts): for every row a few of many small feed-forward layers are picked, by a
router's scores or by a table per token id; the row's output is the sum of theirs, weighted.  A shared feed-forward
may run for every row beside them.  Every size, constant and tensor name is a parameter.
"""
import torch

from ..registry import FEED_FORWARDS
from .base import FeedForward, JoinableEnds, ParamSpec
from .chain_norm_parts import linear32, pad_rows


def interleave_gate_up(gate, up):
    """[E, F, K] gate and up matrices of gated experts as the one matrix [E, 2F, K] the routed kernels read: rows
    interleaved sixteen at a time (gate 0..15, up 0..15, gate 16..31, ...).  F must be a multiple of 16."""
    E, F, K = gate.shape
    if F % 16 or tuple(up.shape) != (E, F, K):
        raise ValueError("interleave_gate_up: [E, F, K] twice, F a multiple of 16")
    return torch.stack([gate.reshape(E, F // 16, 16, K), up.reshape(E, F // 16, 16, K)], dim=2).reshape(E, 2 * F, K).contiguous()


@FEED_FORWARDS.register("routed_experts")
class RoutedExperts(JoinableEnds, FeedForward):
    """Which experts a row uses (``routing``):
      "softmax" (default)  router logits z = W_router h in 32-bit, scores s = softmax(z) over all experts; the ``top``
                           experts with the largest scores, weighted by their scores as they are (not renormalized)
      "softmax_chosen"     the ``top`` experts with the largest logits, weighted by the softmax over those logits alone
      "sigmoid"            scores s = sigmoid(z), each of its own logit; the ``top`` largest, weighted by their scores as they are
      "table"              an integer table [vocabulary, top] names the experts of every token id; each weighs 1 / top
    What an expert computes (``activation``):
      "relu2" (default)    W_down act(W_up h), act = the square of relu
      "gelu"               W_down act(W_up h), act = the exact gelu (by the error function)
      "silu_gated"         W_down (silu(W_gate h) * (W_up h))
    ``weigh``: "output" (default): the row gets the sum of weight * expert(h); "input": the sum of expert(weight * h).
    Experts have no biases.  ``shared``: a PartSpec of a feed-forward that runs for every row and is added (default none).
    ``shared_gate``: the shared feed-forward's output is multiplied by sigmoid(W_sg h), one number per row (the tensor's name
    after the prefix; default none).  ``route_factor``: a constant on the experts' weights (default 1).
    Offers its ends (JoinableEnds): the router's product, the gate's and the shared feed-forward's first at one end, the shared
    feed-forward's last at the other; the experts' sum is the further output.  With ``shared_gate`` it runs that way on its own too.
    params: experts, top, ff, routing, activation, weigh, shared, shared_gate, route_factor, vocab_size (rows of the table; default: as stored); router / table (the checkpoint name after the prefix, defaults
    "router", "table"); expert (a pattern for an expert's prefix, default "e{}."), gate, up, down (names after it).
    The result is 32-bit."""

    capturable = True
    sub_part_names = ("shared",)
    # rows from which a bfloat16 step groups its (row, slot) pairs by expert; below, every pair streams its expert's rows itself
    GROUPED_MIN_ROWS = 16

    def __init__(self, params, prefix, ctx):
        super().__init__(params, prefix, ctx)
        self.routing, self.activation = params.get("routing", "softmax"), params.get("activation", "relu2")
        if self.routing not in ("softmax", "softmax_chosen", "sigmoid", "table"):
            raise ValueError(f"routed_experts {prefix!r}: routing {self.routing!r} is not supported (softmax | softmax_chosen | sigmoid | table)")
        if self.activation not in ("relu2", "gelu", "silu_gated"):
            raise ValueError(f"routed_experts {prefix!r}: activation {self.activation!r} is not supported (relu2 | gelu | silu_gated)")
        if params.get("weigh", "output") not in ("output", "input"):
            raise ValueError(f"routed_experts {prefix!r}: weigh {params['weigh']!r} is not supported (output | input)")
        self.gated = self.activation == "silu_gated"
        sh = params.get("shared")
        self.by_ends = bool(params.get("joined") or params.get("shared_gate"))
        if self.by_ends and self.routing == "table":
            raise ValueError(f"routed_experts {prefix!r}: a table's routing has no product to join")
        if params.get("shared_gate") and sh is None:
            raise ValueError(f"routed_experts {prefix!r}: a gate on a shared feed-forward needs one")
        self.shared = None
        if sh is not None:
            self.shared = FEED_FORWARDS.get(sh.kind)({**sh.params, "joined": True} if self.by_ends else sh.params, sh.prefix, ctx)
            if self.by_ends and not isinstance(self.shared, JoinableEnds):
                raise ValueError(f"routed_experts {prefix!r}: the shared {sh.kind!r} does not offer its ends")
        self.F = params["ff"]

    def sub_parts(self):
        return (self.shared,) if self.shared is not None else ()

    def in_sources(self):
        H, p, pre = self.ctx.hidden_size, self.params, self.prefix
        sources = self.shared.in_sources() if self.shared is not None else ()
        sources += ((pre + p.get("router", "router"), (p["experts"], H)),)
        if p.get("shared_gate"):
            sources += ((pre + p["shared_gate"], (1, H)),)
        return sources

    def out_source(self):
        return self.shared.out_source() if self.shared is not None else None

    def out_bias(self):
        return self.shared.out_bias() if self.shared is not None else None

    def param_specs(self):
        H, p, pre = self.ctx.hidden_size, self.params, self.prefix
        E, F = p["experts"], p["ff"]
        names = [pre + p.get("expert", "e{}.").format(e) for e in range(E)]
        specs = [ParamSpec("w_up", tuple((n + p.get("up", "up"), (F, H)) for n in names)),
                 ParamSpec("w_down", tuple((n + p.get("down", "down"), (H, F)) for n in names))]
        if self.gated:
            specs.append(ParamSpec("w_gate", tuple((n + p.get("gate", "gate"), (F, H)) for n in names)))
        if self.routing == "table":
            specs.append(ParamSpec("table", ((pre + p.get("table", "table"), (p.get("vocab_size", -1), p["top"])),), role="index", distinct_below=E))
        elif not self.by_ends:
            specs.append(ParamSpec("w_router", ((pre + p.get("router", "router"), (E, H)),)))
        elif not p.get("joined"):
            specs += [ParamSpec("w_in", self.in_sources()), ParamSpec("w_shared_out", (self.out_source(),))]
        return specs

    def bind(self, tensors):
        E, F, H = self.params["experts"], self.params["ff"], self.ctx.hidden_size
        bound = {}
        if self.routing == "table":
            bound["table"] = tensors["table"].contiguous()
        elif self.by_ends:
            if "w_in" in tensors:
                bound["w_in"] = self.ctx.derive(self, "w_in", lambda: pad_rows(tensors["w_in"]))
                bound["w_shared_out"] = tensors["w_shared_out"]
        else:
            bound["w_router"] = pad_rows(tensors["w_router"])      # the route reads the first E

        def gated_pair():
            up, down = tensors["w_up"].view(E, F, H), tensors["w_down"].view(E, H, F)
            # gate and up as one matrix, rows interleaved sixteen at a time; columns that bring F to a multiple of 16 are zero
            # (silu(0) * 0 = 0, and the down matrix has zero columns there)
            gate, pad = tensors["w_gate"].view(E, F, H), -F % 16
            if pad:
                zeros = torch.zeros(E, pad, H, dtype=up.dtype, device=up.device)
                gate, up = torch.cat([gate, zeros], 1), torch.cat([up, zeros], 1)
                down = torch.cat([down, torch.zeros(E, H, pad, dtype=down.dtype, device=down.device)], 2).contiguous()
            return interleave_gate_up(gate, up), down
        if self.gated:
            bound["w_up"], bound["w_down"] = self.ctx.derive(self, "gated_pair", gated_pair)
            self.F = F + -F % 16
        else:
            bound["w_up"], bound["w_down"] = tensors["w_up"].view(E, F, H), tensors["w_down"].view(E, H, F)
        super().bind(bound)

    def bytes_read(self, rows):
        """The router (or the rows' table entries), and the experts that ``rows`` rows can reach at most."""
        p, w = self.params, self.w
        reached = min(p["experts"], rows * p["top"])
        per_expert = (w["w_up"][0].numel() + w["w_down"][0].numel()) * w["w_up"].element_size()
        if self.routing == "table":
            routing = rows * p["top"] * 4
        else:      # (joined, the router is counted where its product is)
            routing = sum(w[n].numel() * w[n].element_size() for n in ("w_router", "w_in", "w_shared_out") if n in w)
        return routing + reached * per_expert

    def flops(self, rows, attended=0):
        p, H = self.params, self.ctx.hidden_size
        router = 0 if self.routing == "table" or p.get("joined") else p["experts"] * H
        if self.by_ends and not p.get("joined"):
            router = self.w["w_in"].shape[0] * H + self.w["w_shared_out"].numel()
        return 2.0 * rows * (router + p["top"] * (3 if self.gated else 2) * p["ff"] * H)

    def between(self, step, h, proj, out):
        p = self.params
        at = sum(shape[0] for _, shape in self.shared.in_sources()) if self.shared is not None else 0
        if self.shared is not None:
            if p.get("shared_gate"):
                self.shared.between(step, h, proj, out, row_gate=proj[:, at + p["experts"]:])
            else:
                self.shared.between(step, h, proj, out)
        return self._experts(step, h, proj[:, at:])

    def forward(self, step, h):
        if self.by_ends:
            proj = linear32(self.ctx, step, h, self.w["w_in"], "routed_in")
            values = step.ws("routed_values", (step.rows, self.w["w_shared_out"].shape[1]))
            experts = self.between(step, h, proj, values)
            ops = self.ctx.ops
            return ops.StreamTerms([(linear32(self.ctx, step, values, self.w["w_shared_out"], "routed_shared_out", keep_partial=True), 1.0),
                                    (experts, 1.0)], self.out_bias())
        return self._experts(step, h)

    def _experts(self, step, h, logits=None):
        """The experts' weighted sum, 32-bit [T, H]; ``logits``: the router's, where somebody else made them."""
        ops, p, w = self.ctx.ops, self.params, self.w
        E, top, F, T = p["experts"], p["top"], self.F, step.rows
        chosen = step.ws("routed_chosen", (T, top), torch.int32)
        weight = step.ws("routed_weight", (T, top), torch.float32)
        if self.routing == "table":
            ops.moe_table_route(step.tokens, w["table"], top, chosen, weight, rows=T)
        else:
            if logits is None:
                logits = linear32(self.ctx, step, h, w["w_router"], "routed_logits", keep_partial=True)      # the route adds the slices
            ops.moe_route(logits, E, top, chosen, weight, rows=T, over_chosen=self.routing == "softmax_chosen", sigmoid=self.routing == "sigmoid",
                          factor=p.get("route_factor", 1.0))
        add = self.shared.forward(step, h) if self.shared is not None and not self.by_ends else None      # 32-bit [T, H]: the experts' sum starts from it
        H = self.ctx.hidden_size
        how = dict(gated=self.gated, add=add, weigh_input=p.get("weigh") == "input", **({} if self.gated else {"activation": self.activation}))
        act = step.ws("routed_act", (T, top * F)).view(T * top, F)
        out = step.ws("routed_out", (T, H), torch.float32)
        if T >= self.GROUPED_MIN_ROWS and ops.moe_grouped_supported(H, F, E, act.dtype) and h.stride(0) % 8 == 0:
            # many rows: the pairs grouped by expert, tiles on the matrix cores, every expert's weights read once per tile
            order = step.ws("routed_order", (T, top), torch.int32)
            tiles = step.flat("routed_tiles", ops.moe_grouped_tiles(max(T, step.limits.max_tokens if step.limits else T) * top, E), torch.int32)
            y = step.ws("routed_y", (T, top * H), torch.float32).view(T * top, H)
            return ops.moe_grouped(h, w["w_up"], w["w_down"], chosen, weight, order, tiles, act, y, out, **how)
        return ops.moe_rows(h, w["w_up"], w["w_down"], chosen, weight, act, out, **how)
