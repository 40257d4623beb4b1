"""Talapel as a plan over the generic parts.

Embedding ``embed`` times ``embedding.scale``; layers ``l<i>`` in the order config.json lists them, of which the run
``loop`` is passed through several times with the same weights, each pass with a cache and state of its own
and entered through ``loop.in`` (the stream beside the embedding's output); every layer has one layer norm
``l<i>.norm1`` (a weight, no bias) that the mixer under ``l<i>.mix`` and the feed-forward under ``l<i>.mlp`` (or none)
both read, and adds the sum of what they put out; last layer norm ``final.norm``; head ``head``.

Mixers by layer type.  ``parallel``: grouped-query attention with biases on all four projections, a query temperature,
a soft cap and an output gate under ``.left``, a state-space recurrence (Mamba-2) under ``.right``, each times a
factor, summed.  ``retention``: a matrix state per head with a fixed decay and rotary positions.

Feed-forwards: ``dense`` is ``down(silu(gate x) * (up x))``; ``moe`` takes the experts that the table
``l<i>.mlp.table`` names for the token's id, ``down(relu(up x)^2)`` each, and averages them.
"""

from __future__ import annotations

from ..config.talapel import TalapelConfig
from ..parts.plan import LayerCall, LayerSpec, ModelPlan, PartSpec
from ..registry import register_architecture

ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b", "o_bias": "o.b",
                   "gate": "g"}
DENSE_NAMES = {"gate": "gate", "up": "up", "down": "down"}
EXPERT_NAMES = {"expert": "e{e}", "up": "up", "down": "down", "table": "table"}


def _mixer(config: TalapelConfig, kind: str, sizes: dict, prefix: str) -> PartSpec:
    width, eps = config.width, config.norm_eps
    if kind == "retention":
        rot = sizes["rot"]
        return PartSpec("retention", {
            "hidden_size": width, "heads": sizes["heads"], "dim": sizes["dim"], "value_dim": sizes["vdim"], "eps": eps,
            "decay": sizes["decay"],
            "position": PartSpec("rotary", {"head_dim": sizes["dim"], "theta": rot["base"], "rotary_dim": rot["dims"], "precise": True}),
        }, prefix)
    left, right = sizes["left"], sizes["right"]
    attention = PartSpec("gqa_attention", {
        "hidden_size": width, "num_heads": left["heads"], "num_kv_heads": left["kv_heads"], "head_dim": left["dim"],
        "value_dim": left["vdim"], "scale": left["scale"], "softcap": left.get("softcap"), "query_temperature": left.get("q_temp"),
        "bias": True, "bias_init": "small", "output_bias_init": "small", "output_gate": True, "output_scale": sizes["left_scale"], "fill_rows": True,
        "position": PartSpec("none"),
        "names": ATTENTION_NAMES,
    }, f"{prefix}.left")
    recurrence = PartSpec("state_space_duality", {
        "hidden_size": width, "heads": right["heads"], "value_dim": right["vdim"], "state": right["state"],
        "groups": right["groups"], "conv_taps": right["conv"], "norm_groups": right["norm_groups"], "eps": eps,
        "output_scale": sizes["right_scale"],
    }, f"{prefix}.right")
    return PartSpec("parallel_mixers", {"hidden_size": width, "combine": "sum", "branches": {"left": attention, "right": recurrence}},
                    prefix)


def _feed_forward(config: TalapelConfig, mlp: dict | None, prefix: str) -> PartSpec | None:
    if mlp is None:
        return None
    if mlp["kind"] == "dense":
        return PartSpec("swiglu", {"hidden_size": config.width, "intermediate_size": mlp["ff"], "names": DENSE_NAMES}, prefix)
    return PartSpec("routed_experts", {
        "hidden_size": config.width, "experts": mlp["router"]["experts"], "top": mlp["router"]["top"],
        "intermediate_size": mlp["expert"]["ff"], "scoring": "table", "form": "relu_squared", "router_bias": False,
        "vocab_size": config.vocab, "names": EXPERT_NAMES,
    }, prefix)


def run_order(count: int, loop: tuple[int, int, int] | None) -> tuple[LayerCall, ...]:
    """The calls of ``count`` layers of which the run ``loop`` (start, stop, times) is passed through several times."""
    if loop is None:
        return tuple(LayerCall(index) for index in range(count))
    start, stop, times = loop
    calls = [LayerCall(index) for index in range(start)]
    for _ in range(times):
        calls += [LayerCall(index, enters=index == start) for index in range(start, stop)]
    return tuple(calls + [LayerCall(index) for index in range(stop, count)])


def talapel_plan(config: TalapelConfig) -> ModelPlan:
    width = config.width

    def norm(name: str) -> PartSpec:
        return PartSpec("layer_norm", {"size": width, "eps": config.norm_eps, "leaf": "", "bias_leaf": None}, name)

    layers = tuple(
        LayerSpec("parallel", _mixer(config, layer["type"], layer["mixer"], f"l{index}.mix"),
                  _feed_forward(config, layer.get("mlp"), f"l{index}.mlp"), {"input": norm(f"l{index}.norm1")})
        for index, layer in enumerate(config.layers))
    sizes = {"vocab_size": config.vocab, "hidden_size": width, "leaf": ""}
    return ModelPlan(
        hidden_size=width,
        vocab_size=config.vocab,
        embedding=PartSpec("token_embedding", dict(sizes, scale=config.embedding_scale), "embed"),
        layers=layers,
        schedule=run_order(len(layers), config.loop),
        final_norm=norm("final.norm"),
        head=PartSpec("lm_head", dict(sizes), "head"),
        entry=None if config.loop is None else PartSpec("concat_projection", {"hidden_size": width, "leaf": ""}, "loop.in"),
        eos_token_ids=frozenset() if config.eos_token_id is None else frozenset({config.eos_token_id}),
        max_positions=None,
    )


register_architecture(TalapelConfig.architecture, TalapelConfig, talapel_plan)
