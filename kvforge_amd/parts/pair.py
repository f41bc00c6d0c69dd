"""Two mixers side by side: both read the same input, and their outputs add into the stream, each
scaled by its own constant, which the mixers apply themselves, or each through an RMS norm of its
own over the stream's width."""

from __future__ import annotations

import torch

from kvforge_amd.kernels import ops
from kvforge_amd.parts.base import CacheSpec, LayerState, Mixer, Norm, Part, StateSpec, WeightSpec
from kvforge_amd.registry import register_mixer


def _floats(spec: StateSpec | None) -> int:
    if spec is None:
        return 0
    if len(spec.shape) != 1 or spec.dtype != torch.float32:
        raise ValueError(f"mixers side by side keep their state as one row of fp32 numbers each, got {spec}")
    return int(spec.shape[0])


@register_mixer("pair")
class MixerPair(Mixer):
    """``left`` and ``right`` are whole mixers with prefixes of their own.  A call has one set of
    pages, so at most one of the two may keep pages (``cache_spec``): attention beside a
    recurrence, say.  Where both keep a state, a request's slot holds the left one's numbers and
    behind them the right one's.  Each is handed what it declared of the call's ``LayerState``.
    ``norms``: two RMS norms of one eps that the outputs pass, ``out_scale (norm_l(left) + norm_r(right))``;
    the constant goes into their fp32 weights, and both norms and the sum into the stream are one kernel."""

    def __init__(self, left: Mixer, right: Mixer, norms: tuple[Norm, Norm] | None = None, out_scale: float = 1.0) -> None:
        self.left, self.right, self.norms = left, right, norms
        self.out_scale = float(out_scale)
        if left.cache_spec is not None and right.cache_spec is not None:
            raise ValueError("two mixers side by side: only one of them may keep pages")
        if norms is None and self.out_scale != 1.0:
            raise ValueError("a constant on mixers side by side goes with norms on their outputs")
        if norms is not None and norms[0].eps != norms[1].eps:
            raise ValueError("the norms of mixers side by side share one eps")
        self.weights: tuple[torch.Tensor, torch.Tensor] | None = None
        # where the right one's numbers begin in a slot that both use (on 16 bytes)
        self.right_off = 0
        if left.state_spec is not None and right.state_spec is not None:
            if not (left.shares_slot and right.shares_slot):
                raise ValueError("two mixers side by side that both keep a state must take a block of columns of a slot")
            self.right_off = -(-_floats(left.state_spec) // 4) * 4

    @property
    def cache_spec(self) -> CacheSpec | None:
        return self.left.cache_spec if self.left.cache_spec is not None else self.right.cache_spec

    @property
    def state_spec(self) -> StateSpec | None:
        if self.right_off:
            return StateSpec((-(-(self.right_off + _floats(self.right.state_spec)) // 4) * 4,), torch.float32)
        return self.left.state_spec if self.left.state_spec is not None else self.right.state_spec

    @property
    def replayable(self) -> bool:
        return self.left.replayable and self.right.replayable

    def _both(self) -> tuple[Part, ...]:
        return (self.left, self.right, *(self.norms or ()))

    def weight_specs(self) -> dict[str, WeightSpec]:
        out: dict[str, WeightSpec] = {}
        for m in self._both():
            out.update(m.weight_specs())
        return out

    def load(self, tensors: dict[str, torch.Tensor]) -> None:
        for m in self._both():
            m.load(tensors)
        if self.norms is not None:
            self.weights = tuple((n.weight.float() * self.out_scale).contiguous() for n in self.norms)

    def seal(self) -> None:
        for m in self._both():
            m.seal()

    def kernel_modules(self, dtype: torch.dtype) -> set[str]:
        return set().union(*(m.kernel_modules(dtype) for m in self._both()))

    def num_bytes(self) -> int:
        return sum(m.num_bytes() for m in self._both())

    def held_tensors(self) -> list[torch.Tensor]:
        return [t for m in self._both() for t in m.held_tensors()] + list(self.weights or ())

    def launch_key(self, shape):
        return self.left.launch_key(shape), self.right.launch_key(shape)

    def _layers(self, layer: LayerState) -> tuple[LayerState, LayerState]:
        if not self.right_off or layer.state is None:
            return layer, layer
        n = _floats(self.left.state_spec)
        halves = (layer.state[:, :n], layer.state[:, self.right_off:self.right_off + _floats(self.right.state_spec)])
        return tuple(LayerState(layer.group, layer.pages, layer.owns_cache, s) for s in halves)

    def forward(self, x, step, layer: LayerState, residual) -> None:
        """``x``: normalised activations.  Without norms, what the first leaves owed to the stream the
        second settles (or takes along) as any part does; with norms, each writes rows of its own."""
        ll, rl = self._layers(layer)
        if self.norms is None:
            self.left.forward(x, step, ll, residual)
            self.right.forward(x, step, rl, residual)
            return
        step.settle()
        rows = []
        for m, state, name in ((self.left, ll, "pair_left_out"), (self.right, rl, "pair_right_out")):
            out = step.ws.buf(name, tuple(residual.shape), torch.float32)
            step.fresh = out
            m.forward(x, step, state, out)
            if step.fresh is out:
                raise RuntimeError("a mixer whose output passes a norm must write its fresh rows (end in "
                                   "parts.base.add_product)")
            rows.append(out)
        ops.rms_add_two(residual, rows[0], self.weights[0], rows[1], self.weights[1], self.norms[0].eps)
