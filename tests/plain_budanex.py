"""A plain, slow implementation of the Budanex decoder, one function per mechanism, in float64 on the
CPU.  It shares no code with the package: the tests compare the engine with it.  What another design's
plain implementation already spells out (the Mamba-2 recurrence, the rotate-half layout) is taken from there.

Budanex: an embedding with a norm behind it; pre-norm layers; a run of layers that is passed through
several times, the embedding's output being added to the stream ahead of every pass but the first and
the pass's own learned vector ahead of every pass; three mixers (softcapped attention with biases and a
norm over the whole projection of q and of k; a Mamba-2 recurrence; attention through a latent over a
sliding window with a sink and an output gate, interleaved rotary positions with YaRN frequencies);
gated feed-forwards with the tanh form of gelu; a last norm, a head of its own and a cap on the logits.

A model is (config dict, {tensor name: float64 tensor}).  ``forward`` runs whole sequences;
``Stepper`` runs a request in portions from explicit state.
"""

from __future__ import annotations

import math

import torch

from plain_talapel import load_weights, rms_unit, rotate_half_layout, run_order, state_space_branch  # noqa: F401

F64 = torch.float64


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return rms_unit(x, eps) * weight


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def capped(x: torch.Tensor, cap: float | None) -> torch.Tensor:
    return x if cap is None else cap * torch.tanh(x / cap)


def join(state: dict | None, **rows) -> list[torch.Tensor]:
    """Every named tensor behind what the state already holds of it, which the state then keeps."""
    if state is None:
        return list(rows.values())
    for name, new in rows.items():
        state[name] = torch.cat([state[name], new]) if name in state else new
    return [state[name] for name in rows]


def attention_mixer(h, w, p, sizes, positions, eps: float, state: dict | None = None) -> torch.Tensor:
    """Grouped-query attention; q and k are normed over all their heads at once before they are turned."""
    heads, groups, dim, vdim, rot = sizes["heads"], sizes["kv_heads"], sizes["dim"], sizes["vdim"], sizes["rot"]
    count = h.shape[0]
    q, k, v = (h @ w[f"{p}.{n}"].T + w[f"{p}.{n}.b"] for n in "qkv")
    q, k = rms_norm(q, w[p + ".q.norm"], eps), rms_norm(k, w[p + ".k.norm"], eps)
    q = rotate_half_layout(q.view(count, heads, dim), positions, rot["dims"], rot["base"])
    k = rotate_half_layout(k.view(count, groups, dim), positions, rot["dims"], rot["base"])
    k, v, k_positions = join(state, k=k, v=v.view(count, groups, vdim), pos=positions)
    out = torch.zeros((count, heads, vdim), dtype=h.dtype)
    unseen = k_positions[None, :] > positions[:, None]
    for head in range(heads):
        g = head // (heads // groups)
        score = capped((q[:, head] @ k[:, g].T) * sizes["scale"], sizes.get("softcap"))
        out[:, head] = torch.softmax(score.masked_fill(unseen, -math.inf), dim=1) @ v[:, g]
    return out.reshape(count, heads * vdim) @ w[p + ".o"].T


def yarn_frequencies(dims: int, base: float, scaling: dict | None) -> tuple[torch.Tensor, float]:
    """(frequency of every pair, factor on cosines and sines)."""
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if scaling is None:
        return torch.tensor(plain, dtype=F64), 1.0
    factor, original = scaling["factor"], scaling["original"]

    def turning(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(turning(scaling["fast"])), 0), min(math.ceil(turning(scaling["slow"])), dims - 1)
    found = []
    for i, f in enumerate(plain):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        found.append(f / factor * ramp + f * (1.0 - ramp))
    return torch.tensor(found, dtype=F64), 0.1 * math.log(factor) + 1.0


def rotate_interleaved(x: torch.Tensor, positions: torch.Tensor, rot: dict) -> torch.Tensor:
    """x [T, ..., D]: the first ``rot.dims`` dims turned, dims 2i and 2i + 1 forming a pair."""
    dims = rot["dims"]
    frequencies, magnitude = yarn_frequencies(dims, rot["base"], rot.get("scaling"))
    angle = positions.to(F64)[:, None] * frequencies[None, :]
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (dims // 2,)
    cos, sin = (magnitude * torch.cos(angle)).view(shape), (magnitude * torch.sin(angle)).view(shape)
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2], out[..., 1:dims:2] = u * cos - v * sin, v * cos + u * sin
    return out


def sink_softmax(score: torch.Tensor, sink: torch.Tensor | float) -> torch.Tensor:
    """Softmax over the last dim whose denominator also holds exp(sink)."""
    top = torch.clamp(score.max(dim=-1, keepdim=True).values, min=float(sink))
    weights = torch.exp(score - top)
    return weights / (weights.sum(dim=-1, keepdim=True) + torch.exp(torch.as_tensor(sink, dtype=score.dtype) - top))


def latent_attention_mixer(h, w, p, sizes, positions, eps: float, state: dict | None = None) -> torch.Tensor:
    heads, dim, turned, vdim, rank, rot = (sizes[n] for n in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "rot"))
    window, count = (sizes.get("mask") or {}).get("size"), h.shape[0]
    q = (h @ w[p + ".q"].T).view(count, heads, dim + turned)
    q_plain, q_turned = q[..., :dim], rotate_interleaved(q[..., dim:], positions, rot)
    down = h @ w[p + ".dkv"].T
    latent, part, k_positions = join(state, latent=rms_norm(down[:, :rank], w[p + ".dkv.norm"], eps),
                                     part=rotate_interleaved(down[:, rank:], positions, rot), pos=positions)
    k = (latent @ w[p + ".uk"].T).view(-1, heads, dim)
    v = (latent @ w[p + ".uv"].T).view(-1, heads, vdim)
    distance = positions[:, None] - k_positions[None, :]
    unseen = distance < 0
    if window is not None:
        unseen |= distance >= window
    out = torch.zeros((count, heads, vdim), dtype=h.dtype)
    for head in range(heads):
        score = (q_plain[:, head] @ k[:, head].T + q_turned[:, head] @ part.T) * sizes["scale"]
        out[:, head] = sink_softmax(score.masked_fill(unseen, -math.inf), float(w[p + ".sink"][head])) @ v[:, head]
    return (out.reshape(count, heads * vdim) * torch.sigmoid(h @ w[p + ".g"].T)) @ w[p + ".o"].T


def state_space_mixer(h, w, p, sizes, positions, eps: float, state: dict | None = None) -> torch.Tensor:
    return state_space_branch(h, w, p, sizes, eps, state)


MIXERS = {"attention": attention_mixer, "mamba2": state_space_mixer, "latent_attention": latent_attention_mixer}


def dense_feed_forward(h, w, p) -> torch.Tensor:
    return (gelu_tanh(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T)) @ w[p + ".down"].T


def enter_pass(x, first, steps, number: int) -> torch.Tensor:
    """The stream right ahead of pass ``number``: the embedding's output comes in again from the second pass on, and
    every pass has a vector of its own."""
    return (x if number == 0 else x + first) + steps[number]


def run_layers(config: dict, w: dict, tokens, positions, states: list | None = None, trail: list | None = None):
    """The residual stream after the last layer; ``states``: one dict per layer run for a request that
    is run in steps; ``trail`` collects the stream after every layer run."""
    eps = config["norm"]["eps"]
    first = rms_norm(w["embed"][torch.as_tensor(tokens, dtype=torch.long)], w["embed.norm"], eps)
    x, number = first, 0
    for index, (layer_number, begins) in enumerate(run_order(config)):
        if begins:
            x = enter_pass(x, first, w["loop.step"], number)
            number += 1
        layer, p = config["layers"][layer_number], f"l{layer_number}"
        state = None if states is None else states[index]
        x = x + MIXERS[layer["type"]](rms_norm(x, w[p + ".norm1"], eps), w, p + ".mix", layer["mixer"], positions, eps, state)
        if layer.get("mlp") is not None:
            x = x + dense_feed_forward(rms_norm(x, w[p + ".norm2"], eps), w, p + ".mlp")
        if trail is not None:
            trail.append(x.clone())
    return x


def logits_of(config: dict, w: dict, x: torch.Tensor) -> torch.Tensor:
    return capped(rms_norm(x, w["final.norm"], config["norm"]["eps"]) @ w["head"].T, config.get("logit_softcap"))


def forward(config: dict, w: dict, tokens, trail=None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence from position 0."""
    return logits_of(config, w, run_layers(config, w, tokens, torch.arange(len(tokens)), None, trail))


class Stepper:
    """One request run in portions of any size from explicit state."""

    def __init__(self, config: dict, w: dict) -> None:
        self.config, self.w = config, w
        self.states = [{} for _ in run_order(config)]
        self.length = 0

    def step(self, tokens) -> torch.Tensor:
        positions = torch.arange(self.length, self.length + len(tokens))
        self.length += len(tokens)
        return logits_of(self.config, self.w, run_layers(self.config, self.w, tokens, positions, self.states))
