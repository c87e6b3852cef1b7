"""A matrix product whose result is float32 whatever the storage type: float32 accumulation AND output."""
import torch
import torch.nn.functional as F


class F32Product:
    """x [T, K] times w [N, K]^T -> float32 [T, N].  16-bit operands stay 16-bit where the vendor GEMM can write float32 for the
    shape; otherwise the same sums come from widened operands (which of the two is settled at the first call)."""

    def __init__(self):
        self.native = None

    def __call__(self, x, w):
        if x.dtype == torch.float32:
            return F.linear(x, w)
        if x.is_cuda and self.native is not False:
            try:
                out = torch.mm(x, w.t(), out_dtype=torch.float32)
                self.native = True
                return out
            except RuntimeError:
                if self.native:            # it has worked before: this is another fault
                    raise
                self.native = False
        return F.linear(x.float(), w.float())
