"""What joins the residual stream where a pass over a stretch of the schedule starts.

A model may run a stretch of its layers several times over with the same weights (every run with a cache of its own:
the schedule names a layer once a run). "step_and_embedding": before pass t, the vector t of a stored table joins
x, and from the second pass on, before that, the embedding's output once more. "joined_projection": before every pass
x becomes W [x | x0], x0 the embedding's output.

A part of this category either says what joins x (`rows`), which a block may take on, or makes x anew itself
(`replaces`, with `begin` once a step and `forward` at every pass).
"""
import torch

from ..kernels import ops
from ..weights import TensorNeed
from .base import Part
from .linear import Linear
from .registry import register


def _step_init(shape, gen, device, std, norm_std):
    """A random model's vectors: of a size that a pass with another's vector, or with none, shows."""
    return 0.5 * torch.randn(shape, generator=gen, device=device, dtype=torch.float32)


@register("pass_input", "step_and_embedding")
class StepAndEmbedding(Part):
    graph_safe = True

    def __init__(self, hidden_size, passes, weight):
        self.hidden_size, self.passes, self.weight_name = int(hidden_size), int(passes), weight
        self.steps = None

    def tensor_needs(self):
        return {self.weight_name: TensorNeed((self.passes, self.hidden_size), "bias", _step_init)}

    def load(self, tensors, rt):
        self.steps = rt.weight(tensors[self.weight_name], matrix=False)

    @property
    def reads_embedding(self):
        """True if a later pass needs the embedding's output, which the model then keeps."""
        return self.passes > 1

    def rows(self, pass_number, embedded):
        """(rows [T, hidden] or None, vector [hidden]) that join x before this pass, in this order."""
        return (embedded if pass_number > 0 else None), self.steps[pass_number]


@register("pass_input", "joined_projection")
class JoinedProjection(Part):
    """x <- W [x | x0] with W [hidden, 2 hidden]. Its second half times x0 is the same in every pass: it is worked out once a
    step, and a pass adds the first half's product to a copy of it, as any part adds its last product to the
    stream (the norm that follows prepared with it)."""
    graph_safe = True
    replaces = True
    reads_embedding = False

    def __init__(self, hidden_size, weight):
        self.hidden_size, self.weight_name = int(hidden_size), weight
        self.w_stream = self.w_embedding = None

    def tensor_needs(self):
        return {self.weight_name: TensorNeed((self.hidden_size, 2 * self.hidden_size))}

    def load(self, tensors, rt):
        w = rt.weight(tensors[self.weight_name])
        H = self.hidden_size
        self.w_stream = Linear(w[:, :H].contiguous(), scratch=rt.scratch)
        self.w_embedding = Linear(w[:, H:].contiguous(), scratch=rt.scratch)

    def begin(self, ctx, x):
        """x is the embedding's output. Returns what `forward` needs of it."""
        rt = ctx.rt
        rows = rt.buffer("pass_rows", tuple(x.shape))
        ops.rows_and_base(x, rows)
        base = rt.buffer("pass_base", tuple(x.shape), torch.float32)
        self.w_embedding.forward(rows, base)
        return base

    def forward(self, ctx, x, base):
        rows = ctx.rt.buffer("pass_rows", tuple(x.shape))
        ops.rows_and_base(x, rows, base)
        ctx.project_out(self.w_stream, rows, x)
