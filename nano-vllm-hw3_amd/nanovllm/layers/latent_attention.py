"""Latent attention: keys and values are up-projections of one small per-token latent, and only the latent is cached.
The key up-projection is folded into the query ("absorbed": q'_h = W_uk,h^T q_h, so that
q_h . k_h = q'_h . c) and the value up-projection is applied after the attention sum, which makes the cached latent
both key and value of a multi-query attention with ``heads`` query heads of size ``kv_rank``.

Without further arguments positions do not enter.  ``rot_dim`` > 0 adds a rotated part: every query head carries
``rot_dim`` more channels, the down-projection ``rot_dim`` more rows that form ONE key part shared by all heads; the
first ``rot_dims`` channels of both turn with the position (channel 2i pairs with 2i + 1, angle = position *
rot_base^(-2i/rot_dims)) and their product joins the score.  The cache row is then [latent | rotated key part], the
absorbed query [W_uk^T q | rotated q part], and only the latent columns are values.  ``window`` > 0: a query sees itself
and the window - 1 tokens before it.  ``q_rank`` > 0: the queries come through a latent of their own,
q = W_uq rms_norm(W_dq h) with a weight on the norm (the down-projection shares its product with the key/value latent's).
``rot_scaling``: a frequency table stretched for longer contexts, with its factor on cosines and sines
(hy_ops.rotary_table).  ``sink``: a learned number per head whose exponential joins the softmax denominator.  ``kv_source``:
another LatentAttention whose cached rows this layer reads with its own queries and up-projections; it has no
down-projection and no cache of its own.

``attend`` is the mixer between its first product and its last one (a block that merges those with others' calls it)."""
import torch
import torch.nn.functional as F
from torch import nn

from nanovllm import hy_ops, seq_ops


class LatentAttention(nn.Module):
    def __init__(self, width: int, heads: int, dim: int, vdim: int, kv_rank: int, scale: float, eps: float,
                 rot_dim: int = 0, rot_dims: int = 0, rot_base: float = 10000.0, window: int = 0, q_rank: int = 0,
                 rot_scaling=None, sink: bool = False, kv_source=None):
        super().__init__()
        assert kv_source is None or (kv_source.kv_source is None and (kv_source.kv_rank, kv_source.rot_dim, kv_source.rot_dims) ==
                                     (kv_rank, rot_dim, rot_dims)), "a reader's row layout is its source's"
        self.__dict__["kv_source"] = kv_source             # (not a submodule of this layer)
        self.rot_scaling, self.rot_mag = rot_scaling, 1.0
        assert rot_dims % 2 == 0 and rot_dims <= rot_dim
        self.heads, self.dim, self.vdim, self.kv_rank, self.scale, self.eps = heads, dim, vdim, kv_rank, float(scale), eps
        self.rot_dim, self.rot_dims, self.rot_base, self.window = rot_dim, rot_dims, rot_base, int(window)
        self.row = kv_rank + rot_dim           # columns of a cache row
        self.inv_freq = None                   # f32 [rot_dims / 2], made with the cache
        # query and latent down-projection share one product: rows [0, heads*(dim+rot_dim)) = W_q (per head [dim | rot_dim]),
        # then kv_rank rows of W_dkv and its rot_dim rows of the shared key part
        # with a query latent: rows [0, q_rank) = W_dq instead, and W_uq [heads*(dim+rot_dim), q_rank] follows its norm
        self.q_rank = int(q_rank)
        self.q_rows = self.q_rank or heads * (dim + rot_dim)
        self.qc_proj = nn.Parameter(torch.empty(self.q_rows + (kv_rank + rot_dim if kv_source is None else 0), width), requires_grad=False)
        self.q_latent_norm = nn.Parameter(torch.ones(q_rank), requires_grad=False) if q_rank else None
        self.uq = nn.Parameter(torch.empty(heads * (dim + rot_dim), q_rank), requires_grad=False) if q_rank else None
        self.latent_norm = nn.Parameter(torch.ones(kv_rank), requires_grad=False) if kv_source is None else None
        self.sink = nn.Parameter(torch.zeros(heads, dtype=torch.float32), requires_grad=False) if sink else None
        self.uk = nn.Parameter(torch.empty(heads, dim, kv_rank), requires_grad=False)      # per head [dim, kv_rank]
        self.uv = nn.Parameter(torch.empty(heads, kv_rank, vdim), requires_grad=False)     # per head W_uv^T [kv_rank, vdim]
        self.o_proj = nn.Parameter(torch.empty(width, heads * vdim), requires_grad=False)
        self.cache = {}            # layer run -> [blocks, block_size, kv_rank + rot_dim]

    def allocate(self, run, num_blocks, block_size, dtype, device):
        """The cache of one layer run (a reader takes its source's: allocate it after the source)."""
        if self.kv_source is None:
            self.cache[run] = torch.zeros(num_blocks, block_size, self.row, dtype=dtype, device=device)
        else:
            self.cache[run] = self.kv_source.cache[run]
        if self.rot_dims and self.inv_freq is None:
            self.inv_freq, self.rot_mag = hy_ops.rotary_table(self.rot_dims, self.rot_base, device, self.rot_scaling)

    def cache_bytes_per_token(self, itemsize):
        return self.row * itemsize if self.kv_source is None else 0

    def forward(self, h, run: int = 0):
        return F.linear(self.attend(F.linear(h, self.qc_proj), run), self.o_proj)

    def attend(self, qc, run: int = 0, out=None):
        """qc [T, rows of qc_proj] (may be a column slice of a wider product) -> the heads' outputs [T, heads * vdim], in
        ``out`` if given (may be a column slice)."""
        ctx = seq_ops.get_step()
        T = qc.shape[0]
        H, D, Rd, R = self.heads, self.dim, self.rot_dim, self.kv_rank
        nq = self.q_rows
        cache = self.cache[run]
        if self.rot_dim or self.window or self.q_rank or self.kv_source is not None:
            qa = torch.empty((T, H, self.row), dtype=qc.dtype, device=qc.device)      # absorbed queries [T, H, R | Rd]
            if self.q_rank:
                q2 = F.linear(seq_ops.rms_norm_rows(qc[:, :nq], self.q_latent_norm, self.eps), self.uq)
            else:
                q2 = qc[:, :nq]
            q = q2.view(T, H, D + Rd)
            # q'_h = W_uk,h^T q_h straight into the first R columns of every head's row
            torch.bmm(q[..., :D].transpose(0, 1), self.uk, out=qa.transpose(0, 1)[..., :R])
            seq_ops.latent_rope_store(qc[:, nq:] if self.kv_source is None else None, self.latent_norm, self.eps, q2, qa,
                                      self.inv_freq, self.rot_dims, H, D, R, Rd, cache, ctx, self.rot_mag)
        else:
            seq_ops.latent_norm_store(qc[:, nq:], self.latent_norm, self.eps, cache, ctx.slot_mapping)
            q = qc[:, :nq].view(T, H, D).transpose(0, 1)                              # [H, T, D]
            qa = torch.bmm(q, self.uk).transpose(0, 1).contiguous()                   # absorbed queries [T, H, R]
        ol = seq_ops.latent_attention(qa, cache, ctx, self.scale, value_cols=R, window=self.window, sink=self.sink)     # [T, H, R]
        if out is None:
            out = torch.empty((T, H * self.vdim), dtype=qc.dtype, device=qc.device)
        torch.bmm(ol.transpose(0, 1), self.uv, out=out.view(T, H, self.vdim).transpose(0, 1))
        return out
