"""A block whose mixer and feed-forward read the same normed input and add into the same residual:
    h = norm(x),   x <- x + mixer(h) + feed_forward(h).
All weights that multiply h share ONE product (the mixer's first rows, then the dense feed-forward's or the shared expert's),
and all weights whose results are added share ONE product over the joined columns; the modules keep their parameters, as views
into the merged storage.  Routed experts leave their per-pair rows to whoever closes the block (hy_ops.layer_norm_residual).

A mixer offers (first weight, last weight, how to get from the first product's columns to the last one's); a feed-forward is
None, a GatedMLP, or RoutedExperts with or without a squared-ReLU shared expert."""
import torch
import torch.nn.functional as F
from torch import nn

from nanovllm import hy_ops, seq_ops
from nanovllm.layers.feedforward import GatedMLP, ReluSquaredMLP, RoutedExperts
from nanovllm.layers.latent_attention import LatentAttention
from nanovllm.layers.selective_scan import SelectiveScan


def merge_storage(params, dim):
    """One tensor that holds the given parameters side by side along ``dim``; they become views into it."""
    if len(params) == 1:
        return params[0].data
    merged = torch.cat([p.data for p in params], dim)
    at = 0
    for p in params:
        p.data = merged.narrow(dim, at, p.shape[dim])
        at += p.shape[dim]
    return merged


class ParallelBlock(nn.Module):
    def __init__(self, mixer, mlp=None):
        super().__init__()
        self.mixer, self.mlp = mixer, mlp
        if isinstance(mixer, LatentAttention):
            first, self._mix = mixer.qc_proj, lambda p, out: mixer.attend(p, out=out)
        elif isinstance(mixer, SelectiveScan):
            first, self._mix = mixer.in_proj, lambda p, out: mixer.scan(p, out=out)
        else:
            raise TypeError(f"no parallel form of {type(mixer).__name__}")
        self.routed = mlp if isinstance(mlp, RoutedExperts) else None
        side = mlp.shared if self.routed is not None else mlp          # what rides on the two shared products
        assert side is None or isinstance(side, (GatedMLP, ReluSquaredMLP))
        self.gated = isinstance(side, GatedMLP)
        assert not (self.routed is not None and self.gated), "a shared expert beside routed ones is a squared-ReLU layer here"
        self.act_kind = side.act_kind if self.gated else None
        self.rows, self.cols = first.shape[0], mixer.o_proj.shape[1]
        self.side = side is not None
        firsts, lasts = [first], [mixer.o_proj]
        if side is not None:
            firsts.append(side.gate_up if self.gated else side.up)
            lasts.append(side.down)
        self._firsts, self._lasts = firsts, lasts
        self.w_first, self.w_last = merge_storage(firsts, 0), merge_storage(lasts, 1)

    def forward(self, h):
        """h [T, width] -> (what the dense parts add to the residual [T, width], the routed experts' rows or None; see
        hy_ops.layer_norm_residual)."""
        p = F.linear(h, self.w_first)
        a = torch.empty((h.shape[0], self.w_last.shape[1]), dtype=h.dtype, device=h.device)
        self._mix(p[:, :self.rows], a[:, :self.cols])
        gate = rows = None
        if self.routed is not None:
            idx, wts, gate = self.routed.route(h)
            rows = self.routed.products(h, idx, wts, combine=False)
        if self.side:
            if self.gated:
                seq_ops.gated_act(p[:, self.rows:], self.act_kind, out=a[:, self.cols:])
            else:                              # a shared expert's gate scales what its last product reads
                hy_ops.relu_squared(p[:, self.rows:], row_scale=gate, out=a[:, self.cols:])
        return F.linear(a, self.w_last), rows
