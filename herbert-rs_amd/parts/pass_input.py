"""What joins the residual stream where a pass over a stretch of the schedule starts.

A model may run a stretch of its layers several times over with the same weights (every run with a cache of its own:
the schedule names a layer once a run). "step_and_embedding": before pass t, the vector t of a stored table joins
x, and from the second pass on, before that, the embedding's output once more.
"""
import torch

from ..weights import TensorNeed
from .base import Part
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
