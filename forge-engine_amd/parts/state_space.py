"""A state-space mixer with one decay per head and token (Mamba-2, state-space duality).

In order: one product gives ``[z | x | B | C | dt]`` (``inner = heads * value_dim``, inner, groups *
state, groups * state, heads wide); x, B and C pass a short causal convolution per channel with a
bias and SiLU; per head h, which reads the B and C of its group (heads / groups neighbours share
one), with ``dt = softplus(dt + dt_bias_h)``,

    S <- exp(-exp(A_log_h) dt) S + dt B x^T,      y = S^T C + D_h x        (S: [state, value_dim]);

then the heads side by side times silu(z), divided by the root mean square of each of
``norm_groups`` equal parts, times a weight, and the output product.  Per request the state S
(float32) and the last taps - 1 rows ahead of the convolution are kept in a state slot, so a
request may be cut into steps anywhere.  Step sizes, decays, the state, the read-out, the gate's
activation and the norm are float32 in both compute modes.  ``output_scale``: a factor on the mixer's
output (it joins the norm's weight).
"""

from __future__ import annotations

import torch
from torch import Tensor

from ..cache.spec import CacheNeeds, CacheView, FixedState
from ..kernels import ops
from ..registry import register_part
from .base import BuildContext, JointEnds, Mixer, ParamSpec


class StateSpaceMixer(Mixer):
    DEFAULT_NAMES = {"in": "in", "conv": "conv", "conv_bias": "conv.b", "dt_bias": "dt_bias", "a_log": "A_log", "d": "D",
                     "norm": "norm", "o": "o"}
    STATE, CONV_STATE = "matrix", "conv"

    def __init__(self, ctx: BuildContext, prefix: str, *, hidden_size: int, heads: int, value_dim: int, state: int, groups: int,
                 conv_taps: int, norm_groups: int, eps: float, output_scale: float = 1.0,
                 names: dict[str, str] | None = None) -> None:
        super().__init__(ctx, prefix)
        if heads % groups:
            raise ValueError(f"{heads} heads do not form {groups} equal groups")
        if not 1 <= state <= 256:
            raise ValueError(f"between 1 and 256 states, not {state}")
        if not 1 <= conv_taps <= 8:
            raise ValueError(f"a short convolution has 1 to 8 taps, not {conv_taps}")
        if (heads * value_dim) % norm_groups:
            raise ValueError(f"{heads * value_dim} channels do not form {norm_groups} equal parts")
        self.hidden_size, self.heads, self.value_dim, self.state, self.groups = hidden_size, heads, value_dim, state, groups
        self.conv_taps, self.norm_groups, self.eps, self.output_scale = conv_taps, norm_groups, float(eps), float(output_scale)
        self.inner = heads * value_dim
        self.channels = self.inner + 2 * groups * state        # what passes the convolution
        self.names = dict(self.DEFAULT_NAMES, **(names or {}))
        self.tensors: dict[str, Tensor] = {}

    def shapes(self) -> dict[str, tuple[tuple[int, ...], str, str]]:
        width, per_head = self.hidden_size, (self.heads,)
        return {"in": ((self.inner + self.channels + self.heads, width), "matrix", "normal"),
                "conv": ((self.channels, self.conv_taps), "vector", "taps"), "conv_bias": ((self.channels,), "vector", "small"),
                "dt_bias": (per_head, "vector", "unit"), "a_log": (per_head, "vector", "unit"), "d": (per_head, "vector", "norm"),
                "norm": ((self.inner,), "vector", "norm"), "o": ((width, self.inner), "matrix", "normal")}

    def param_specs(self):
        return {self.name(self.names[key]): ParamSpec(shape, kind=kind, init=init)
                for key, (shape, kind, init) in self.shapes().items()}

    def set_param(self, name: str, tensor: Tensor) -> None:
        local = name[len(self.prefix) + 1:] if self.prefix else name
        key = next((k for k, leaf in self.names.items() if leaf == local), None)
        if key is None:
            raise KeyError(name)
        self.tensors[key] = tensor

    def finalize(self) -> None:
        t = self.tensors
        t["rate"] = (-torch.exp(t.pop("a_log").to(torch.float32))).contiguous()
        t["norm"] = t["norm"].to(torch.float32) * self.output_scale
        for key in ("conv", "conv_bias", "dt_bias", "d", "norm"):
            t[key] = t[key].to(torch.float32).contiguous()

    def cache_needs(self) -> CacheNeeds:
        states = {self.STATE: FixedState((self.heads, self.value_dim, self.state), torch.float32)}    # value-major
        if self.conv_taps > 1:
            states[self.CONV_STATE] = FixedState((self.conv_taps - 1, self.channels), torch.float32)
        return CacheNeeds(state=states)

    takes_stream = True

    def forward(self, x: Tensor, batch, cache: CacheView, writes_cache: bool = True, stream: Tensor | None = None) -> Tensor | None:
        out = torch.empty((x.shape[0], self.inner), dtype=x.dtype, device=x.device)
        self.forward_joint(ops.linear(x, self.tensors["in"]), out, batch, cache, writes_cache)
        return ops.linear_update(out, self.tensors["o"], stream=stream)

    def joint_ends(self) -> JointEnds:
        return JointEnds(self.tensors["in"], self.tensors["o"])

    def release_ends(self) -> None:
        self.tensors["in"] = self.tensors["o"] = None

    def forward_joint(self, z: Tensor, out: Tensor, batch, cache: CacheView, writes_cache: bool = True) -> None:
        t, inner, shared = self.tensors, self.inner, self.groups * self.state
        single = batch.num_decode is not None and batch.num_decode == batch.num_seqs == z.shape[0]
        u = ops.causal_conv_act(z[:, inner:inner + self.channels], t["conv"], t["conv_bias"],
                                cache.states[self.CONV_STATE] if self.conv_taps > 1 else None, batch.token_seq, batch.cu_q,
                                batch.state_slots, num_seqs=batch.num_seqs, act="silu", single_tokens=single)
        y = ops.head_recurrence(u[:, inner + shared:], u[:, inner:inner + shared], u[:, :inner], cache.states[self.STATE],
                                batch.cu_q, batch.state_slots, num_seqs=batch.num_seqs, heads=self.heads, key_dim=self.state,
                                value_dim=self.value_dim, rate=t["rate"], share=self.heads // self.groups,
                                dt=z[:, inner + self.channels:], dt_bias=t["dt_bias"], skip=t["d"], single_tokens=single)
        ops.gated_group_norm(y.view(-1, inner), z[:, :inner], t["norm"], out, groups=self.norm_groups, eps=self.eps)

    def kernel_libraries(self):
        return {"head_recurrence", "selective_scan", "conv_rope", "stream_ops", "gemm_f32", "gemm_skinny", "gemm_mid", "gemm_wide"}


register_part("mixer", "state_space_duality", StateSpaceMixer)
