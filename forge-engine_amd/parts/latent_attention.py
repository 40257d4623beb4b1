"""Causal attention whose keys and values are made from one small cached vector per token.

With x the mixer's input, H heads, per head ``head_dim`` plain and ``rot_dim`` rotated query/key
dims and ``value_dim`` value dims:

* queries through a bottleneck: ``a = rmsnorm(W_dq x)`` (weighted, ``q_rank`` wide), ``q = W_uq a``,
  laid out head by head as [plain | rotated]; without one (``q_rank`` None) ``q = W_q x``;
* what a token leaves in the cache: ``c = rmsnorm(first kv_rank rows of W_dkv x)`` (weighted) and
  ``r = rotate(last rot_dim rows of W_dkv x)``, one key part shared by all heads;
* head h's key of token j is ``[W_uk[h] c_j | r_j]`` and its value ``W_uv[h] c_j``; scores are
  ``(q_plain . W_uk[h] c_j + q_rot . r_j) * scale``, softmax over j <= i, output ``W_o`` on the
  concatenated heads.

Keys and values are never made.  ``q_plain . W_uk[h] c = (W_uk[h]^T q_plain) . c``, so every head's
query is taken through its key up-projection once and attention then runs over the cached rows
``[c | r]`` themselves, all heads sharing them like the query heads of one key/value head; the values
are the first ``kv_rank`` dims of those rows, and ``W_uv[h]`` is applied once to the attention's
result.  The cache holds one row ``[c | r]`` a token as its key pages and ``c`` a second time in
transposed value pages (the layout the matrix-core kernel reads its second operand in):
``2 kv_rank + rot_dim`` numbers a token, whatever the number of heads.

A layer with ``own_kv`` False has no ``W_dkv``: it is scheduled to read the pages of an earlier layer
of the same geometry, with its own queries, ``W_uk``, ``W_uv`` and ``W_o``.

Options: ``window`` (token i sees keys i - window + 1 .. i only, and pages that the window has passed go back),
``sink`` (a learned number per head whose exponential joins the softmax's denominator, without key or value, after the
scale), ``output_gate`` (the concatenated heads times ``sigmoid(W_g x)``).  Without a query bottleneck everything that
reads x (queries, gate, down-projection) is one product.  ``fill_rows`` (bfloat16): cache rows of sizes that the
matrix-core kernel is not compiled for lie in rows of the next sizes it is, filled up with zeros, and the
up-projections with them.

The rotation is the position part's (over its first ``rotary_dim`` dims of the ``rot_dim`` wide part; either pairing, and
a factor on cosines and sines).  Norms, angles, scores and softmax are float32; behind a query bottleneck the
down-projections are stored float32 for the norms.
"""

from __future__ import annotations

import torch
from torch import Tensor

from ..cache.spec import CacheNeeds, CacheView, PagedKV
from ..kernels import ops
from ..registry import register_part
from .base import BuildContext, Mixer, ParamSpec, build_part
from .plan import PartSpec


class LatentAttention(Mixer):
    DEFAULT_NAMES = {"dq": "q_down.weight", "dq_norm": "q_down.norm", "uq": "q_up.weight", "dkv": "kv_down.weight",
                     "dkv_norm": "kv_down.norm", "uk": "k_up.weight", "uv": "v_up.weight", "o": "o_proj.weight",
                     "q": "q_proj.weight", "gate": "gate_proj.weight", "sink": "sink"}

    def __init__(self, ctx: BuildContext, prefix: str, *, hidden_size: int, num_heads: int, head_dim: int, rot_dim: int,
                 value_dim: int, q_rank: int | None, kv_rank: int, eps: float, position: PartSpec, scale: float | None = None,
                 own_kv: bool = True, window: int | None = None, sink: bool = False, output_gate: bool = False,
                 fill_rows: bool = False, names: dict[str, str] | None = None) -> None:
        super().__init__(ctx, prefix)
        if min(num_heads, head_dim, value_dim, 1 if q_rank is None else q_rank, kv_rank) < 1 or rot_dim < 0:
            raise ValueError("heads, head sizes and ranks must be positive")
        if kv_rank + rot_dim > ops.MASKED_MAX_KEY_DIM or kv_rank > ops.MASKED_MAX_VALUE_DIM:
            raise ValueError(f"cached rows of up to {ops.MASKED_MAX_KEY_DIM} numbers with a latent of up to "
                             f"{ops.MASKED_MAX_VALUE_DIM}, not {kv_rank} + {rot_dim}")
        self.hidden_size, self.num_heads = hidden_size, num_heads
        self.head_dim, self.rot_dim, self.value_dim = head_dim, rot_dim, value_dim
        self.q_rank, self.kv_rank = q_rank, kv_rank
        if window is not None and window < 1:
            raise ValueError("a window has at least one key")
        if q_rank is None and not own_kv:
            raise ValueError("a layer without a down-projection of its own has a query bottleneck")
        self.window, self.sink, self.output_gate = window, sink, output_gate
        # what a token leaves in the cache, and how wide its latent part is there
        self.row_dim, self.latent_row = ops.latent_row_sizes(ctx.dtype, kv_rank, rot_dim) if fill_rows else (kv_rank + rot_dim, kv_rank)
        self.q_head = head_dim + rot_dim
        self.eps = float(eps)
        self.scale = (head_dim + rot_dim) ** -0.5 if scale is None else float(scale)
        self.own_kv = own_kv
        self.names = dict(self.DEFAULT_NAMES, **(names or {}))
        self.position = build_part("position", position, ctx)
        rotary = self.position.rotary()
        if rotary is not None and rotary[1] > rot_dim:
            raise ValueError(f"{rotary[1]} rotated dims do not fit a rotated part of {rot_dim}")
        # one product for what reads x: both bottlenecks [dq | dkv], or without one for the queries [q | gate | dkv]
        blocks = [("dq", q_rank)] if q_rank is not None else [("q", num_heads * self.q_head), ("gate", self.gate_size)]
        if own_kv:
            blocks.append(("dkv", kv_rank + rot_dim))
        self._rows, self.down_rows = {}, 0
        for key, rows in blocks:
            if rows:
                self._rows[key] = (self.down_rows, rows)
                self.down_rows += rows
        self.down_weight: Tensor | None = None      # [down_rows, hidden]
        self.gate_weight: Tensor | None = None      # beside a query bottleneck, whose product is stored float32
        self.sink_weight: Tensor | None = None
        self.q_norm: Tensor | None = None
        self.kv_norm: Tensor | None = None
        self.uq_weight: Tensor | None = None
        self.uk: Tensor | None = None               # [heads, head_dim, latent_row]
        self.uv_t: Tensor | None = None             # [heads, latent_row, value_dim]
        self.uk_t: Tensor | None = None             # the same two with the summed dim last, for steps of a few tokens
        self.uv: Tensor | None = None
        self.o_weight: Tensor | None = None

    @property
    def gate_size(self) -> int:
        return self.num_heads * self.value_dim if self.output_gate else 0

    def param_specs(self):
        n = {key: self.name(leaf) for key, leaf in self.names.items()}
        heads, hidden = self.num_heads, self.hidden_size
        if self.q_rank is None:
            specs = {n["q"]: ParamSpec((heads * self.q_head, hidden))}
        else:
            specs = {n["dq"]: ParamSpec((self.q_rank, hidden)), n["dq_norm"]: ParamSpec((self.q_rank,), kind="vector", init="norm"),
                     n["uq"]: ParamSpec((heads * self.q_head, self.q_rank))}
        specs.update({
            n["uk"]: ParamSpec((heads * self.head_dim, self.kv_rank)),
            n["uv"]: ParamSpec((heads * self.value_dim, self.kv_rank)),
            n["o"]: ParamSpec((hidden, heads * self.value_dim)),
        })
        if self.output_gate:
            specs[n["gate"]] = ParamSpec((self.gate_size, hidden))
        if self.sink:
            specs[n["sink"]] = ParamSpec((heads,), kind="vector", init="unit")
        if self.own_kv:
            specs[n["dkv"]] = ParamSpec((self.kv_rank + self.rot_dim, hidden))
            specs[n["dkv_norm"]] = ParamSpec((self.kv_rank,), kind="vector", init="norm")
        return specs

    def set_param(self, name: str, tensor: Tensor) -> None:
        local = name[len(self.prefix) + 1:] if self.prefix else name
        key = next((k for k, leaf in self.names.items() if leaf == local), None)
        if key in self._rows:
            if self.down_weight is None:
                self.down_weight = torch.empty((self.down_rows, self.hidden_size), dtype=tensor.dtype, device=tensor.device)
            if tensor.dtype != self.down_weight.dtype:
                raise ValueError(f"{name}: the down-projections of one input must be stored in one dtype")
            start, rows = self._rows[key]
            self.down_weight[start:start + rows].copy_(tensor)
        elif key == "gate" and self.output_gate:
            self.gate_weight = tensor
        elif key == "sink" and self.sink:
            self.sink_weight = tensor
        elif key == "dq_norm" and self.q_rank is not None:
            self.q_norm = tensor
        elif key == "dkv_norm" and self.own_kv:
            self.kv_norm = tensor
        elif key == "uq" and self.q_rank is not None:
            self.uq_weight = tensor
        elif key == "uk":
            self.uk = self._filled(tensor.view(self.num_heads, self.head_dim, self.kv_rank))
            self.uk_t = self.uk.transpose(1, 2).contiguous() if self._steps(1) else None
        elif key == "uv":
            uv = self._filled(tensor.view(self.num_heads, self.value_dim, self.kv_rank))
            self.uv_t, self.uv = uv.transpose(1, 2).contiguous(), uv if self._steps(1) else None
        elif key == "o":
            self.o_weight = tensor
        else:
            raise KeyError(name)

    def _filled(self, tensor: Tensor) -> Tensor:
        """The last dim filled up from the latent's size to its width in a cache row."""
        return tensor if self.latent_row == self.kv_rank else torch.nn.functional.pad(tensor, (0, self.latent_row - self.kv_rank))

    def _steps(self, tokens: int) -> bool:
        """Whether a step of so few tokens takes the products per head with their endings in one launch each."""
        return ops.latent_step_fits(tokens, self.ctx.dtype, self.head_dim, self.rot_dim, self.latent_row)

    def cache_needs(self) -> CacheNeeds:
        return CacheNeeds(paged=PagedKV(1, self.row_dim, self.window, self.latent_row))

    takes_stream = True

    def forward(self, x: Tensor, batch, cache: CacheView, writes_cache: bool = True, stream: Tensor | None = None) -> Tensor | None:
        if writes_cache != self.own_kv:
            raise ValueError(f"{self.prefix}: a layer with a down-projection of its own writes its cache, one without reads another's")
        tokens, heads = x.shape[0], self.num_heads
        rotary = self.position.rotary()
        inv_freq, rotary_dim = rotary if rotary is not None else (None, 0)
        turning = {"rot_dim": self.rot_dim, "rotary_dim": rotary_dim, "interleaved": self.position.interleaved,
                   "magnitude": self.position.magnitude()}
        gate = latent_q = None
        if self.q_rank is None:
            product = ops.linear(x, self.down_weight)
            q = product[:, :heads * self.q_head]
            if self.output_gate:
                start, rows = self._rows["gate"]
                gate = product[:, start:start + rows]
            down = product[:, self._rows["dkv"][0]:]
        else:
            down = ops.linear(x, self.down_weight, out_dtype=torch.float32)
            latent_q = torch.empty((tokens, self.q_rank), dtype=x.dtype, device=x.device)
        if self.q_rank is not None or writes_cache:
            ops.latent_norm_rope_write(down, self.q_norm, self.kv_norm, inv_freq, batch.positions, batch.token_seq,
                                       cache.block_table, cache.key_pages, cache.value_pages, latent_q, q_rank=self.q_rank or 0,
                                       kv_rank=self.kv_rank, eps=self.eps, write_kv=writes_cache, latent_row=self.latent_row, **turning)
        if self.q_rank is not None:
            q = ops.linear(latent_q, self.uq_weight)                                   # [T, H * (plain | rotated)]
            if self.output_gate:
                gate = ops.linear(x, self.gate_weight)
        few = self._steps(tokens) and q.stride(0) % 8 == 0
        rows = torch.empty((tokens, heads, self.row_dim), dtype=x.dtype, device=x.device)
        if few:
            ops.latent_query_step(q, self.uk_t, inv_freq, batch.positions, rows, heads=heads, dim=self.head_dim, **turning)
        else:
            plain = q.unflatten(1, (heads, self.q_head))[:, :, :self.head_dim]
            through_keys = ops.heads_product(plain, self.uk)                           # [H, T, latent_row]
            ops.latent_query_pack(q, through_keys, inv_freq, batch.positions, rows, heads=heads, dim=self.head_dim,
                                  kv_rank=self.latent_row, **turning)
        read = torch.empty((tokens, heads * self.latent_row), dtype=x.dtype, device=x.device)
        ops.latent_attention(rows.view(tokens, heads * self.row_dim), cache.key_pages, cache.value_pages, read, batch.cu_q, batch.ctx_len,
                             cache.block_table, num_seqs=batch.num_seqs, max_q_len=batch.max_q_len, heads=heads,
                             row_dim=self.row_dim, value_dim=self.latent_row, scale=self.scale, num_decode=batch.num_decode,
                             max_ctx=batch.max_ctx, window=self.window, sink=self.sink_weight)
        attn = torch.empty((tokens, heads * self.value_dim), dtype=x.dtype, device=x.device)
        read = read.view(tokens, heads, self.latent_row)
        if few:
            ops.latent_value_step(read, self.uv, gate, attn)
        else:
            ops.gate_heads(ops.heads_product(read, self.uv_t), gate, attn)             # values [H, T, value_dim]
        return ops.linear_update(attn, self.o_weight, stream=stream)

    def token_inputs(self):
        return self.position.token_inputs()

    def kernel_libraries(self):
        return {"latent", "attention_latent", "attention_masked", "stream_ops", "gemm_f32", "gemm_skinny", "gemm_mid", "gemm_wide"}


register_part("mixer", "latent_attention", LatentAttention)
