"""Selective scan (Mamba): a recurrent mixer whose per-channel state S [states] decays, learns and is read by what the token
itself says,
    S <- exp(dt A) S + dt x B,   y = S . C + D x,   result = W_o (y * silu(z)),
with [x | z] = W_in h, x behind a short causal convolution with bias and SiLU, [d | B | C] = W_x x, dt = softplus(W_dt d + b)
one step size per channel, A = -exp(A_log) and D learned.  The state is float32, one [channels, states] block per state slot,
the convolution's last inputs beside it; dt's product leaves the matrix unit in float32, and everything of the recurrence
is float32.

``scan`` is the mixer between its first product and its last one (a block that merges those with others' calls it)."""
import torch
import torch.nn.functional as F
from torch import nn

from nanovllm import hy_ops, seq_ops
from nanovllm.layers.canon import CausalTaps
from nanovllm.layers.f32_product import F32Product


class SelectiveScan(nn.Module):
    def __init__(self, width, inner, states, taps, dt_rank):
        super().__init__()
        self.inner, self.states, self.taps, self.dt_rank = inner, states, taps, dt_rank
        f32 = dict(dtype=torch.float32)
        self.in_proj = nn.Parameter(torch.empty(2 * inner, width), requires_grad=False)                   # rows: x | z
        self.conv = CausalTaps(inner, taps, bias=True, silu=True, add_input=False)
        self.x_proj = nn.Parameter(torch.empty(dt_rank + 2 * states, inner), requires_grad=False)         # rows: d | B | C
        self.dt_proj = nn.Parameter(torch.empty(inner, dt_rank), requires_grad=False)
        self.dt_bias = nn.Parameter(torch.zeros(inner, **f32), requires_grad=False)
        self.A = nn.Parameter(torch.zeros(inner, states, **f32), requires_grad=False)                     # -exp(A_log)
        self.D = nn.Parameter(torch.zeros(inner, **f32), requires_grad=False)
        self.o_proj = nn.Parameter(torch.empty(width, inner), requires_grad=False)
        self.dt_product = F32Product()
        self.state = None          # f32 [slots, inner, states]

    def allocate(self, num_slots, dtype, device):
        self.state = torch.zeros(num_slots, self.inner, self.states, dtype=torch.float32, device=device)
        self.conv.state = torch.zeros(num_slots, 1, max(self.taps - 1, 1), self.inner, dtype=dtype, device=device)

    def state_bytes_per_slot(self, itemsize):
        return self.inner * self.states * 4 + max(self.taps - 1, 1) * self.inner * itemsize

    def forward(self, h):
        return F.linear(self.scan(F.linear(h, self.in_proj)), self.o_proj)

    def scan(self, xz, out=None):
        """xz [T, 2 * inner] (may be a column slice of a wider product) -> gated channels [T, inner], in ``out`` if given (may
        be a column slice)."""
        C, N, R = self.inner, self.states, self.dt_rank
        x = self.conv(xz[:, :C])
        d = F.linear(x, self.x_proj)
        dt = self.dt_product(d[:, :R], self.dt_proj)
        return hy_ops.selective_scan(x, dt, self.dt_bias, d, R, R + N, self.A, self.D, xz[:, C:2 * C], self.state, seq_ops.get_step(),
                                     out=out)
