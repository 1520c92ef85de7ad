"""What stands between a norm and its sublayer."""
import torch

from .. import memory
from ..registry import register_part
from ..status import EINVAL, fail
from .base import FixedState, ParamSpec, Part


@register_part("input", "causal_conv")
class InputConv(Part):
    """``h_t = n_t + sum_j w[:, j] n_(t - taps + 1 + j)``: a causal convolution over time on each channel (tensor ``prefix + weight``,
    [width, taps], the last column the current token's; no bias; zeros before a sequence's start), added to its own input. The last
    ``taps - 1`` inputs are part of a request's state, fp32. ``n`` is fp32, ``h`` the activations' dtype, the sum fp32."""
    graph_safe = True
    shares_cache = False          # the state is this entry's own, whoever's keys its mixer reads

    def __init__(self, size, taps, prefix="", weight="conv.weight"):
        super().__init__(prefix)
        if not 1 <= taps <= 8:
            fail(EINVAL, f"causal_conv: a convolution over {taps} tokens (1 to 8)")
        self.E, self.K = size, int(taps)
        self.name = prefix + weight
        self.taps = self.taps_by_age = self.no_state = None

    def param_specs(self):
        return [ParamSpec(self.name, (self.E, self.K), "vector", ("normal", 0.3))]

    def cache_need(self):
        return FixedState((self.K - 1) * self.E) if self.K > 1 else None       # one tap is a factor a channel

    def bind(self, params, ops):
        # the input itself joins the current token's tap: h = sum_j w'[:, j] n_(..) with w'[:, last] = 1 + w[:, last]
        memory.note(f"{self.name}, its input added")
        self.taps = params[self.name].clone().contiguous()
        self.taps[:, -1] += 1.0
        self.taps_by_age = self.taps.t().contiguous()          # the order in which single tokens read them
        self.no_state = ops.shared("a convolution's state that is never read",
                                   lambda: memory.zeros((1, 1), torch.float32, ops.device, "a convolution's state that is never read"))

    def single_token(self, step, cache):
        """Keywords of ``Ops.stream_input`` for a step in which every request brings one token."""
        return dict(taps=self.taps_by_age) if self.K == 1 else dict(taps=self.taps_by_age, state=cache.state, slots=step.token_slot)

    def forward(self, ops, step, n, cache, out):
        ops.causal_conv(n, self.taps, None, self.no_state if self.K == 1 else cache.state, step, out)
