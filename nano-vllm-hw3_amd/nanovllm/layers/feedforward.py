"""Feed-forward layers beyond the SiLU-gated MLP: a dense layer with the PolyNorm activation, the clamped GLU expert,
and a routed mixture of such experts with group-limited top-k routing and an optional shared expert."""
import torch
import torch.nn.functional as F
from torch import nn

from nanovllm import seq_ops


class PolyNormMLP(nn.Module):
    """down(PolyNorm(up(h))): PolyNorm(z) = a N(z) + b N(z^2) + c N(z^3) + e with N = division by the row's RMS."""

    def __init__(self, width: int, ff: int, eps: float):
        super().__init__()
        self.eps = eps
        self.up = nn.Parameter(torch.empty(ff, width), requires_grad=False)
        self.down = nn.Parameter(torch.empty(width, ff), requires_grad=False)
        self.coef = nn.Parameter(torch.zeros(4, dtype=torch.float32), requires_grad=False)     # a, b, c, e

    def forward(self, h):
        return F.linear(seq_ops.poly_norm(F.linear(h, self.up), self.coef, self.eps), self.down)


class ClampedGLU(nn.Module):
    """down(g * sigmoid(alpha g) * (u + 1)) with g = min(gate(h), limit), u = clamp(up(h), +-limit); no biases."""

    def __init__(self, width: int, ff: int, limit: float, alpha: float = 1.702):
        super().__init__()
        self.ff, self.limit, self.alpha = ff, float(limit), alpha
        self.gate_up = nn.Parameter(torch.empty(2 * ff, width), requires_grad=False)          # gate rows, then up rows
        self.down = nn.Parameter(torch.empty(width, ff), requires_grad=False)

    def forward(self, h):
        return F.linear(seq_ops.clamped_glu(F.linear(h, self.gate_up), self.limit, self.alpha), self.down)


class GatedMLP(nn.Module):
    """down(act(gate h) * up h) for the gated activations of seq_ops (``act`` = "silu_glu" | "gelu_tanh_glu")."""

    def __init__(self, width: int, ff: int, act: str):
        super().__init__()
        self.ff, self.act_kind = ff, RoutedExperts.ACTS[act]
        assert self.act_kind in seq_ops.GATED_ACTS
        self.gate_up = nn.Parameter(torch.empty(2 * ff, width), requires_grad=False)          # gate rows, then up rows
        self.down = nn.Parameter(torch.empty(width, ff), requires_grad=False)

    def forward(self, h):
        return F.linear(seq_ops.gated_act(F.linear(h, self.gate_up), self.act_kind), self.down)


class RoutedExperts(nn.Module):
    """Softmax router in float32; experts in ``groups`` equal groups of neighbours, only the ``keep`` groups with the
    largest member score are eligible; the ``top`` best eligible experts run, weighted by their renormalised scores.
    A shared expert (its own size and limit) runs for every token and is added.

    Variations: ``score`` = "sigmoid" (independent scores instead of a softmax); ``correction``: a learned per-expert
    number added to the scores for the CHOICE of groups and experts only (the weights stay the scores); ``group_top``: a
    group scores the sum of that many of its largest choice scores instead of the largest; ``renorm`` = False: the chosen
    scores weigh as they are; ``act`` = "gelu" / "gelu_tanh": an expert is down(gelu(up h)), no gate, no clamp;
    ``act`` = "silu_glu": an expert is down(silu(gate h) * up h), no clamp; ``bias``: a learned number per expert added to
    the router's logits (with softmax scores and ``renorm`` the weights are the softmax over the chosen logits);
    ``act`` = "gelu_tanh_glu": down(gelu_tanh(gate h) * up h), "relu_sq": down(max(up h, 0)^2); ``weight_in``: a weight
    multiplies what its expert reads instead of what it gives; ``shared_gate``: the shared expert's result is multiplied by
    sigmoid(shared_gate . h), one number per token from the router's pass over h.

    ``route`` and ``products`` are the two halves of the routed part (a block that sums up its results itself calls them)."""

    ACTS = {"clamped_glu": seq_ops.ACT_CLAMPED_GLU, "gelu": seq_ops.ACT_GELU, "gelu_tanh": seq_ops.ACT_GELU_TANH,
            "silu_glu": seq_ops.ACT_SILU_GLU, "relu_sq": seq_ops.ACT_RELU_SQ, "gelu_tanh_glu": seq_ops.ACT_GELU_TANH_GLU}

    def __init__(self, width: int, experts: int, top: int, ff: int, limit: float = 0.0, groups: int = 1, keep: int = 1,
                 shared: nn.Module = None, alpha: float = 1.702, score: str = "softmax", correction: bool = False,
                 group_top: int = 1, renorm: bool = True, act: str = "clamped_glu", bias: bool = False, weight_in: bool = False,
                 shared_gate: bool = False):
        super().__init__()
        assert shared is not None or not shared_gate
        self.weight_in = weight_in
        self.shared_gate = nn.Parameter(torch.zeros(width, dtype=torch.float32), requires_grad=False) if shared_gate else None
        if act == "silu_glu":                  # the gated form with nothing clamped and a plain sigmoid
            limit, alpha = float("inf"), 1.0
        self.experts, self.top, self.groups, self.keep, self.limit, self.alpha = experts, top, groups, keep, float(limit), alpha
        self.score = {"softmax": seq_ops.ROUTE_SOFTMAX, "sigmoid": seq_ops.ROUTE_SIGMOID}[score]
        self.group_top, self.renorm, self.act_kind = group_top, renorm, self.ACTS[act]
        self.parts = 2 if self.act_kind in seq_ops.GATED_ACTS else 1           # gate and up rows, or up rows alone
        self.bias = nn.Parameter(torch.zeros(experts, dtype=torch.float32), requires_grad=False) if bias else None
        self.correction = nn.Parameter(torch.zeros(experts, dtype=torch.float32), requires_grad=False) if correction else None
        self.router = nn.Parameter(torch.empty(experts, width, dtype=torch.float32), requires_grad=False)
        self.w_gu = nn.Parameter(torch.empty(experts, self.parts * ff, width), requires_grad=False)
        self.w_down = nn.Parameter(torch.empty(experts, width, ff), requires_grad=False)
        self.shared = shared
        self._tiled = None         # the expert weights in the layout the matrix-core kernels stream (made at the first step)

    def route(self, h):
        """(chosen experts [T, top], their weights f32 [T, top], the shared expert's gate f32 [T] or None)."""
        r = seq_ops.moe_route(h, self.router, self.top, self.groups, self.keep, self.score, self.correction, self.group_top,
                              self.renorm, self.bias, self.shared_gate)
        return r if self.shared_gate is not None else (*r, None)

    def products(self, h, idx, wts, **kw):
        """The chosen experts' products and their sum, or what is to be summed (see seq_ops.moe_experts)."""
        if self._tiled is None and h.is_cuda and h.dtype == torch.bfloat16:
            self._tiled = (seq_ops.tile_expert_weights(self.w_gu, self.parts), seq_ops.tile_expert_weights(self.w_down))
        return seq_ops.moe_experts(h, idx, wts, self.w_gu, self.w_down, self.limit, self.alpha, tiled=self._tiled,
                                   act_kind=self.act_kind, weight_in=self.weight_in, **kw)

    def forward(self, h):
        idx, wts, gate = self.route(h)
        shared = self.shared(h) if self.shared is not None else None
        if isinstance(shared, tuple):
            shared = shared[0]
        return self.products(h, idx, wts, shared=shared, shared_scale=gate)


class ReluSquaredMLP(nn.Module):
    """down(relu(up(h))^2).  ``extra_rows`` more rows of the up product belong to the caller (a gate that reads the same
    h): forward returns (result, those columns of the product)."""

    def __init__(self, width: int, ff: int, extra_rows: int = 0):
        super().__init__()
        self.ff = ff
        self.up = nn.Parameter(torch.empty(ff + extra_rows, width), requires_grad=False)
        self.down = nn.Parameter(torch.empty(width, ff), requires_grad=False)

    def forward(self, h):
        from nanovllm import hy_ops
        z = F.linear(h, self.up)
        return F.linear(hy_ops.relu_squared(z[:, :self.ff]), self.down), z[:, self.ff:]
