"""A plain, slow implementation of the Talapel decoder, one function per mechanism, in float64 on the
CPU.  It shares no code with the package: the tests compare the engine with it.

Talapel: an embedding times a constant; a run of layers that is passed through several times, the
stream being blended with the embedding's output by one matrix ahead of each pass; layers with one
layer norm that both sublayers read, ``x += mixer(h) + ff(h)``; two mixers (capped attention with a
query temperature and an output gate beside a Mamba-2 recurrence; retention with rotary positions);
feed-forwards that are gated or a mixture of experts that a table of token ids chooses; a last layer
norm and a head of its own.

A model is (config dict, {tensor name: float64 tensor}).  ``forward`` runs whole sequences;
``Stepper`` runs a request in portions from explicit state.
"""

from __future__ import annotations

import math

import torch

F64 = torch.float64


def layer_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    centred = x - x.mean(dim=-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(dim=-1, keepdim=True) + eps) * weight


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.where(z > 30.0, z, torch.log1p(torch.exp(torch.clamp(z, max=30.0))))


def query_temperature(positions: torch.Tensor, coef: float, every: float) -> torch.Tensor:
    """One factor a position: 1 in the first run of ``every`` positions (less one), growing with the
    logarithm of the run's number."""
    return torch.tensor([1.0 + coef * math.log(math.floor((int(p) + 1) / every) + 1.0) for p in positions], dtype=F64)


def capped_attention(q, k, v, q_positions, k_positions, *, scale: float, softcap: float) -> torch.Tensor:
    """q [Tq, H, D], k [Tk, G, D], v [Tk, G, Dv]; every key at or before the query is seen."""
    heads, groups = q.shape[1], k.shape[1]
    out = torch.zeros((q.shape[0], heads, v.shape[2]), dtype=q.dtype)
    unseen = k_positions[None, :] > q_positions[:, None]
    for h in range(heads):
        g = h // (heads // groups)
        score = softcap * torch.tanh((q[:, h] @ k[:, g].T) * scale / softcap)
        score = score.masked_fill(unseen, -math.inf)
        out[:, h] = torch.softmax(score, dim=1) @ v[:, g]
    return out


def attention_branch(h, w, p, sizes, positions, state: dict | None = None) -> torch.Tensor:
    heads, groups, dim, vdim = sizes["heads"], sizes["kv_heads"], sizes["dim"], sizes["vdim"]
    count = h.shape[0]
    q, k, v = (h @ w[f"{p}.{n}"].T + w[f"{p}.{n}.b"] for n in "qkv")
    q, k, v = q.view(count, heads, dim), k.view(count, groups, dim), v.view(count, groups, vdim)
    q = q * query_temperature(positions, sizes["q_temp"]["coef"], sizes["q_temp"]["every"])[:, None, None]
    k_positions = positions
    if state is not None:
        if "k" in state:
            k, v = torch.cat([state["k"], k]), torch.cat([state["v"], v])
            k_positions = torch.cat([state["pos"], positions])
        state["k"], state["v"], state["pos"] = k, v, k_positions
    out = capped_attention(q, k, v, positions, k_positions, scale=sizes["scale"], softcap=sizes["softcap"])
    gated = out.reshape(count, heads * vdim) * torch.sigmoid(h @ w[p + ".g"].T)
    return gated @ w[p + ".o"].T + w[p + ".o.b"]


def causal_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor, before: torch.Tensor | None = None) -> torch.Tensor:
    """x [T, C], taps [C, K] (the last column weighs the token itself); ``before`` [K - 1, C]: the rows
    ahead of x (zeros at a sequence's start)."""
    count = taps.shape[1]
    if before is None:
        before = torch.zeros((count - 1, x.shape[1]), dtype=x.dtype)
    padded = torch.cat([before, x], dim=0)
    return sum(taps[:, j] * padded[j:j + x.shape[0]] for j in range(count)) + bias


def group_norm(y: torch.Tensor, weight: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """RMS norm in equal parts of the row, each by its own root mean square."""
    return rms_unit(y.view(y.shape[0], groups, -1), eps).reshape(y.shape) * weight


def state_space_branch(h, w, p, sizes, eps: float, state: dict | None = None) -> torch.Tensor:
    """Mamba-2: one decay a head and token, B and C shared by the heads of a group."""
    heads, vdim, n, groups, taps = sizes["heads"], sizes["vdim"], sizes["state"], sizes["groups"], sizes["conv"]
    inner, count = heads * vdim, h.shape[0]
    z, raw, dt = (h @ w[p + ".in"].T).split([inner, inner + 2 * groups * n, heads], dim=1)
    before = None if state is None else state.get("conv")
    u = silu(causal_conv(raw, w[p + ".conv"], w[p + ".conv.b"], before))
    if state is not None and taps > 1:
        rows = torch.cat([before if before is not None else torch.zeros((taps - 1, raw.shape[1]), dtype=h.dtype), raw])
        state["conv"] = rows[-(taps - 1):].clone()
    x = u[:, :inner].view(count, heads, vdim)
    b = u[:, inner:inner + groups * n].view(count, groups, n).repeat_interleave(heads // groups, dim=1)
    c = u[:, inner + groups * n:].view(count, groups, n).repeat_interleave(heads // groups, dim=1)
    dt = softplus(dt + w[p + ".dt_bias"])
    decay = torch.exp(-torch.exp(w[p + ".A_log"]) * dt)
    s = torch.zeros((heads, n, vdim), dtype=h.dtype) if state is None or "S" not in state else state["S"]
    ys = []
    for t in range(count):
        s = decay[t][:, None, None] * s + dt[t][:, None, None] * b[t][:, :, None] * x[t][:, None, :]
        ys.append((s * c[t][:, :, None]).sum(1) + w[p + ".D"][:, None] * x[t])
    if state is not None:
        state["S"] = s
    y = torch.stack(ys).reshape(count, inner) * silu(z)
    return group_norm(y, w[p + ".norm"], sizes["norm_groups"], eps) @ w[p + ".o"].T


def parallel_mixer(h, w, p, sizes, positions, eps: float, state: dict | None = None) -> torch.Tensor:
    left_state = right_state = None
    if state is not None:
        left_state, right_state = state.setdefault("left", {}), state.setdefault("right", {})
    left = attention_branch(h, w, p + ".left", sizes["left"], positions, left_state)
    right = state_space_branch(h, w, p + ".right", sizes["right"], eps, right_state)
    return sizes["left_scale"] * left + sizes["right_scale"] * right


def rotate_half_layout(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, heads, D]: the first ``dims`` dims of every head turned, dim i paired with i + dims/2."""
    half = dims // 2
    freq = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=F64)
    angle = positions.to(F64)[:, None] * freq[None, :]
    cos, sin = torch.cos(angle)[:, None, :], torch.sin(angle)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


def retention_mixer(h, w, p, sizes, positions, eps: float, state: dict | None = None) -> torch.Tensor:
    heads, dim, vdim, count = sizes["heads"], sizes["dim"], sizes["vdim"], h.shape[0]
    rot = sizes["rot"]
    q = rotate_half_layout((h @ w[p + ".q"].T).view(count, heads, dim), positions, rot["dims"], rot["base"])
    k = rotate_half_layout((h @ w[p + ".k"].T).view(count, heads, dim), positions, rot["dims"], rot["base"]) * dim ** -0.5
    v = (h @ w[p + ".v"].T).view(count, heads, vdim)
    decay = torch.tensor(sizes["decay"], dtype=F64)[:, None, None]
    s = torch.zeros((heads, dim, vdim), dtype=h.dtype) if state is None or "S" not in state else state["S"]
    outs = []
    for t in range(count):
        s = decay * s + k[t][:, :, None] * v[t][:, None, :]
        outs.append((s * q[t][:, :, None]).sum(1))
    if state is not None:
        state["S"] = s
    o = rms_unit(torch.stack(outs), eps).reshape(count, heads * vdim)
    return (o * silu(h @ w[p + ".g"].T)) @ w[p + ".o"].T


def dense_feed_forward(h, w, p) -> torch.Tensor:
    return (silu(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T)) @ w[p + ".down"].T


def expert(h, w, p) -> torch.Tensor:
    return torch.relu(h @ w[p + ".up"].T) ** 2 @ w[p + ".down"].T


def table_experts(h, tokens, w, p, mlp: dict) -> torch.Tensor:
    """A token id's row of the table names its experts; each counts alike."""
    top, out = mlp["router"]["top"], torch.zeros_like(h)
    for t, token in enumerate(tokens):
        for e in w[p + ".table"][token].tolist():
            out[t] += expert(h[t:t + 1], w, f"{p}.e{e}")[0] / top
    return out


def run_order(config: dict) -> list[tuple[int, bool]]:
    """(layer, whether a pass begins right before it), in the order the layers run."""
    count, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, False) for i in range(count)]
    order = [(i, False) for i in range(loop["start"])]
    for _ in range(loop["times"]):
        order += [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return order + [(i, False) for i in range(loop["stop"], count)]


def run_layers(config: dict, w: dict, tokens, positions, states: list | None = None, trail: list | None = None):
    """The residual stream after the last layer; ``states``: one dict per layer run for a request that
    is run in steps; ``trail`` collects the stream after every layer run."""
    eps = config["norm"]["eps"]
    first = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * config["embedding"]["scale"]
    x = first
    for index, (number, begins) in enumerate(run_order(config)):
        if begins:
            x = torch.cat([x, first], dim=1) @ w["loop.in"].T
        layer, p = config["layers"][number], f"l{number}"
        state = None if states is None else states[index]
        h = layer_norm(x, w[p + ".norm1"], eps)
        mixer = parallel_mixer if layer["type"] == "parallel" else retention_mixer
        y = mixer(h, w, p + ".mix", layer["mixer"], positions, eps, state)
        mlp = layer.get("mlp")
        if mlp is not None:
            y = y + (dense_feed_forward(h, w, p + ".mlp") if mlp["kind"] == "dense" else table_experts(h, tokens, w, p + ".mlp", mlp))
        x = x + y
        if trail is not None:
            trail.append(x.clone())
    return x


def logits_of(config: dict, w: dict, x: torch.Tensor) -> torch.Tensor:
    return layer_norm(x, w["final.norm"], config["norm"]["eps"]) @ w["head"].T


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


def load_weights(folder) -> dict:
    """Every tensor of a model folder as float64 (integers stay integers)."""
    from pathlib import Path

    from safetensors.torch import load_file

    return {name: (t.to(F64) if t.is_floating_point() else t) for name, t in load_file(str(Path(folder) / "model.safetensors")).items()}
