"""Budanex as a plan over the generic parts.

Embedding ``embed`` with an RMS norm ``embed.norm`` behind it; layers ``l<i>`` in the order config.json lists them, of
which the run ``loop`` is passed through several times with the same weights, each pass with a cache and state of its
own; ahead of every pass but the first the embedding's (normed) output is added to the stream, and ahead of every pass a
row of ``loop.step``; pre-norm layers (``l<i>.norm1``, ``l<i>.norm2``, RMS norms) with the mixer under ``l<i>.mix`` and
the feed-forward under ``l<i>.mlp`` (or none); last norm ``final.norm``; head ``head`` with a soft cap on the logits.

Mixers by layer type.  ``attention``: grouped-query attention with biases on q, k and v, a weighted RMS norm over the
whole projection of q and of k, rotary positions on the first dims of every head, a soft cap on the scores.
``mamba2``: the state-space recurrence with one decay a head and token.  ``latent_attention``: attention through a
cached latent over a sliding window, queries straight from the input, interleaved rotary positions with YaRN
frequencies, a sink per head, an output gate.

Feed-forward: ``down(gelu(gate x) * (up x))`` with the tanh form of gelu.
"""

from __future__ import annotations

from ..config.budanex import BudanexConfig
from ..parts.plan import LayerSpec, ModelPlan, PartSpec
from ..registry import register_architecture
from .talapel import DENSE_NAMES, run_order

ATTENTION_NAMES = {"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b", "q_norm": "q.norm",
                   "k_norm": "k.norm"}
LATENT_NAMES = {"q": "q", "dkv": "dkv", "dkv_norm": "dkv.norm", "uk": "uk", "uv": "uv", "o": "o", "gate": "g", "sink": "sink"}


def _position(rot: dict, head_dim: int, interleaved: bool = False) -> PartSpec:
    params = {"head_dim": head_dim, "theta": rot["base"], "rotary_dim": rot["dims"], "interleaved": interleaved}
    scaling = rot.get("scaling")
    if scaling is None:
        return PartSpec("rotary", dict(params, precise=True))
    return PartSpec("yarn_rotary", dict(params, **{key: scaling[key] for key in ("factor", "original", "fast", "slow")}))


def _mixer(config: BudanexConfig, kind: str, sizes: dict, prefix: str) -> PartSpec:
    width, eps = config.width, config.norm_eps
    if kind == "attention":
        return PartSpec("gqa_attention", {
            "hidden_size": width, "num_heads": sizes["heads"], "num_kv_heads": sizes["kv_heads"], "head_dim": sizes["dim"],
            "value_dim": sizes["vdim"], "scale": sizes["scale"], "softcap": sizes.get("softcap"), "whole_norm_eps": eps,
            "bias": True, "bias_init": "small", "output_bias": False, "fill_rows": True,
            "position": _position(sizes["rot"], sizes["dim"]), "names": ATTENTION_NAMES,
        }, prefix)
    if kind == "mamba2":
        return PartSpec("state_space_duality", {
            "hidden_size": width, "heads": sizes["heads"], "value_dim": sizes["vdim"], "state": sizes["state"],
            "groups": sizes["groups"], "conv_taps": sizes["conv"], "norm_groups": sizes["norm_groups"], "eps": eps,
        }, prefix)
    return PartSpec("latent_attention", {
        "hidden_size": width, "num_heads": sizes["heads"], "head_dim": sizes["dim"], "rot_dim": sizes["rot_dim"],
        "value_dim": sizes["vdim"], "q_rank": None, "kv_rank": sizes["kv_rank"], "scale": sizes["scale"], "eps": eps,
        "window": (sizes.get("mask") or {}).get("size"), "sink": True, "output_gate": True, "fill_rows": True,
        "position": _position(sizes["rot"], sizes["rot_dim"], interleaved=True), "names": LATENT_NAMES,
    }, prefix)


def budanex_plan(config: BudanexConfig) -> ModelPlan:
    width, eps = config.width, config.norm_eps

    def norm(name: str) -> PartSpec:
        return PartSpec("rms_norm", {"size": width, "eps": eps, "leaf": ""}, name)

    layers, unread = [], set()
    for index, layer in enumerate(config.layers):
        prefix, mlp = f"l{index}", layer.get("mlp")
        norms, feed_forward = {"input": norm(f"{prefix}.norm1")}, None
        if mlp is not None:
            norms["post_mixer"] = norm(f"{prefix}.norm2")
            feed_forward = PartSpec("swiglu", {"hidden_size": width, "intermediate_size": mlp["ff"], "activation": "gelu_tanh",
                                               "names": DENSE_NAMES}, f"{prefix}.mlp")
        else:       # a checkpoint may still hold the norm of a feed-forward that is not there
            unread.add(f"{prefix}.norm2")
        layers.append(LayerSpec("pre_norm", _mixer(config, layer["type"], layer["mixer"], f"{prefix}.mix"), feed_forward, norms))
    sizes = {"vocab_size": config.vocab, "hidden_size": width, "leaf": ""}
    entry = None
    if config.loop is not None:
        entry = PartSpec("pass_vectors", {"hidden_size": width, "passes": config.loop[2]}, "loop")
    return ModelPlan(
        hidden_size=width,
        vocab_size=config.vocab,
        embedding=PartSpec("token_embedding", dict(sizes, norm_leaf="norm", norm_eps=eps), "embed"),
        layers=tuple(layers),
        schedule=run_order(len(layers), config.loop),
        final_norm=norm("final.norm"),
        head=PartSpec("lm_head", dict(sizes, softcap=config.logit_softcap), "head"),
        entry=entry,
        eos_token_ids=frozenset() if config.eos_token_id is None else frozenset({config.eos_token_id}),
        max_positions=None,
        ignorable_names=frozenset(unread),
    )


register_architecture(BudanexConfig.architecture, BudanexConfig, budanex_plan)
