"""Budanex through the engine on the CPU, with the kernels' plain references patched in, against the
plain implementation (tests/plain_budanex.py): configuration and tensor names, each mechanism alone,
and that logits do not depend on how requests are cut into steps, batched, or placed in pages and
state slots.  The kernels themselves run in the GPU tests."""

from __future__ import annotations

import copy
import math
from types import SimpleNamespace

import pytest
import torch

import budanex_util as bu
import kernel_refs
import replay_util as ru
from forge_engine_amd.config import ConfigError, SchedulerConfig, load_model_config
from forge_engine_amd.engine import build_engine, load_model
from forge_engine_amd.engine.loading import build_model
from forge_engine_amd.sampling import SamplingParams
from forge_engine_amd.weights.random_init import declared_tensors

plain = bu.plain
LENGTHS = {"A": (5, 1, 14, 31), "B": (2, 9, 47, 23), "C": (7, 18, 3, 40), "D": (12, 1, 45, 6)}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: bu.write_model(raw, 7, tmp_path_factory.mktemp(f"budanex_{name}"), change=bu.enlarge) for name, raw in bu.CONFIGS.items()}


def requests_of(name, seed, lengths):
    return ru.make_requests({"vocab_size": bu.CONFIGS[name]["vocab"]}, seed, lengths)


def test_configuration_names_and_shapes():
    config = load_model_config(bu.SMALL_A)
    assert config.architecture == "Budanex" and load_model_config(config.to_dict()) == config
    tensors = declared_tensors(config)
    for name, shape in {"embed": (90, 40), "embed.norm": (40,), "head": (90, 40), "final.norm": (40,), "loop.step": (3, 40), "l0.norm1": (40,),
                        "l0.norm2": (40,), "l0.mix.q": (48, 40), "l0.mix.q.b": (48,), "l0.mix.k": (24, 40), "l0.mix.k.b": (24,),
                        "l0.mix.v": (16, 40), "l0.mix.v.b": (16,), "l0.mix.q.norm": (48,), "l0.mix.k.norm": (24,), "l0.mix.o": (40, 32),
                        "l0.mlp.gate": (28, 40), "l0.mlp.up": (28, 40), "l0.mlp.down": (40, 28), "l1.mix.q": (48, 40), "l1.mix.dkv": (20, 40),
                        "l1.mix.dkv.norm": (14,), "l1.mix.uk": (30, 14), "l1.mix.uv": (36, 14), "l1.mix.sink": (3,), "l1.mix.g": (36, 40),
                        "l1.mix.o": (40, 36), "l2.mix.in": (40 + 64 + 4, 40), "l2.mix.conv": (64, 4), "l2.mix.conv.b": (64,),
                        "l2.mix.dt_bias": (4,), "l2.mix.A_log": (4,), "l2.mix.D": (4,), "l2.mix.norm": (40,), "l2.mix.o": (40, 40)}.items():
        assert tuple(tensors[name].shape) == shape, name
    # no bias on the output projection, no second norm without a feed-forward, no query bottleneck
    assert not any(n in tensors for n in ("l0.mix.o.b", "l1.norm2", "l1.mlp.gate", "l1.mix.dq", "l1.mix.uq", "l0.mix.g"))
    assert "loop.step" not in declared_tensors(load_model_config(bu.SMALL_C))
    a = bu.SMALL_A
    only = lambda mixer: {**a, "layers": [bu.layer(mixer, None)], "loop": None}      # noqa: E731
    for broken in ({**a, "layers": []}, {**a, "layers": [{**a["layers"][0], "type": "retention"}]}, only(bu.attention(3, 2, 8, 8, 4)),
                   only(bu.attention(2, 2, 8, 8, 10)), only(bu.attention(2, 1, 8, 8, 4, scale=0.0)), only(bu.latent(2, 8, 4, 8, 600, 5)),
                   only(bu.latent(2, 8, 4, 8, 6, 0)), only(bu.latent(2, 8, 4, 8, 6, 5, rot_dims=6)), only(bu.mamba(3, 4, 4, 2, 2, 1)),
                   only(bu.latent(2, 8, 4, 8, 6, 5, scaling=(4.0, 64, 8.0))), {**a, "logit_softcap": -1.0},
                   {**a, "layers": [{**a["layers"][0], "mlp": {"kind": "moe", "ff": 8}}]},
                   {**a, "loop": {"start": 2, "stop": 2, "times": 2}}, {**a, "loop": {"start": 0, "stop": 6, "times": 2}},
                   {**a, "loop": {"start": 0, "stop": 2, "times": 0}}, {k: v for k, v in a.items() if k != "norm"}):
        with pytest.raises(ConfigError):
            load_model_config(broken)


def test_run_order_and_caches_of_the_passes():
    """Every pass has a cache slot and a state of its own; windows of layers are their cache groups' windows."""
    model = build_model(load_model_config(bu.SMALL_A), dtype="float32", device="cpu")
    calls = model.schedule
    assert [(c.layer, c.enters) for c in calls] == plain.run_order(bu.SMALL_A)
    assert [c.layer for c in calls] == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4] and [c.cache for c in calls] == list(range(11))
    needs = model.cache_needs()
    assert [n.paged is not None for n in needs] == [i not in (2, 5, 8, 10) for i in range(11)]
    assert needs[1].paged.window == 9 and needs[0].paged.window is None and (needs[1].paged.head_dim, needs[1].paged.value_dim) == (20, 14)
    assert set(needs[2].states()) == {"matrix", "conv"}


def test_plain_in_steps_equals_plain_whole(folders):
    """The plain implementation's own pin: a request run from explicit state, token by token and in
    portions, gives the logits of the whole-sequence functions."""
    for name in bu.CONFIGS:
        cfg, weights = bu.folder_weights(folders[name])
        tokens = requests_of(name, 5, (29,))["r0"]
        whole = plain.forward(cfg, weights, tokens)
        for cuts in ([1] * 29, [7, 2, 13, 1, 6]):
            stepper, at = plain.Stepper(cfg, weights), 0
            for size in cuts:
                got = stepper.step(tokens[at:at + size])
                assert torch.allclose(got, whole[at:at + size], atol=1e-9), (name, at)
                at += size


@pytest.mark.parametrize("name", sorted(bu.CONFIGS))
@pytest.mark.parametrize("mode", ["whole", "tail", "portions", "mixed"])
def test_replay_matches_plain(name, mode, folders, tmp_path, monkeypatch):
    """Whole prompts; a prompt and then token by token; portions down to two tokens; up to three
    live requests, portions beside single tokens."""
    kernel_refs.install(monkeypatch)
    requests = requests_of(name, 3, LENGTHS[name])
    trace = {"whole": ru.trace_whole, "tail": lambda r: ru.trace_tail(r, 16), "portions": ru.trace_portions,
             "mixed": lambda r: ru.trace_mixed(r, 5, max_live=3)}[mode](requests)
    got = ru.run_trace(folders[name], "float32", trace, tmp_path, block_size=bu.BLOCK_SIZE[name], device="cpu", on_cpu=True)
    bu.compare(got, bu.plain_logits(folders[name], requests), "float32")


@pytest.mark.parametrize("name", ["A", "D"])
def test_decoding_from_the_first_token(name, folders, tmp_path, monkeypatch):
    """One token a step from position 0 on, 75 steps, across many windows and pages that are given back."""
    kernel_refs.install(monkeypatch)
    requests = requests_of(name, 8, (75,))
    got = ru.run_trace(folders[name], "float32", ru.trace_tail(requests, 75), tmp_path, block_size=bu.BLOCK_SIZE[name], device="cpu", on_cpu=True)
    bu.compare(got, bu.plain_logits(folders[name], requests), "float32")


def test_pages_and_state_slots_are_used_again(folders, tmp_path, monkeypatch):
    """Seven requests through four state slots and a pool smaller than their sum: every pass's recurrence and
    convolution start from nothing, whoever held the slot before."""
    kernel_refs.install(monkeypatch)
    for name in ("A", "B", "D"):
        requests = requests_of(name, 4, (12, 20, 7, 16, 9, 3, 11))
        trace = ru.trace_mixed(requests, 9, max_live=4)
        assert sum(ru.round64(len(t)) for t in requests.values()) > trace.peak_tokens
        got = ru.run_trace(folders[name], "float32", trace, tmp_path / name, block_size=bu.BLOCK_SIZE[name], device="cpu", on_cpu=True)
        bu.compare(got, bu.plain_logits(folders[name], requests), "float32")


def test_rows_filled_up_in_bfloat16(tmp_path, monkeypatch):
    """Cache rows, queries and matrices that are wider than what they hold: the references fill latents up by a few
    numbers in bfloat16, attention heads lie in rows of 64."""
    kernel_refs.install(monkeypatch)
    folder = bu.write_model(bu.SMALL_A, 7, tmp_path / "model", change=lambda t: bu.enlarge(t, 2.0))
    _, model = load_model(folder, dtype="bfloat16", device="cpu")
    mixers = [block.mixer for block in model.layers]
    assert (mixers[1].row_dim, mixers[1].latent_row) == (14 + 3 + 6 + 2, 17) and mixers[1].uk.shape == (3, 10, 17) and mixers[1].uv_t.shape == (3, 17, 12)
    assert (mixers[0].key_row, mixers[0].value_row) == (64, 64) and mixers[0].o_weight.shape == (40, 4 * 64)
    requests = requests_of("A", 3, (9, 31, 14))
    want = bu.plain_logits(folder, requests)
    for mode, trace in (("portions", ru.trace_portions(requests)), ("mixed", ru.trace_mixed(requests, 5, max_live=3))):
        got = ru.run_trace(folder, "bfloat16", trace, tmp_path / mode, block_size=4, device="cpu", on_cpu=True)
        bu.compare(got, want, "bfloat16", fraction=0.05)


def test_greedy_generation_through_the_scheduler(folders, monkeypatch):
    kernel_refs.install(monkeypatch)
    _, model = load_model(folders["A"], dtype="float32", device="cpu")
    engine = build_engine(model, scheduler_config=SchedulerConfig(block_size=4, block_capacity=64, token_budget=8, max_batch_size=3),
                          eos_token_ids=())
    prompts = list(requests_of("A", 6, (11, 4, 17)).values())
    ids = [engine.submit(prompt, sampling_params=SamplingParams(max_new_tokens=6)) for prompt in prompts]
    engine.run_until_idle()
    cfg, weights = bu.folder_weights(folders["A"])
    for request_id, prompt in zip(ids, prompts):
        tokens = list(prompt)
        for _ in range(6):
            tokens.append(int(plain.forward(cfg, weights, tokens)[-1].argmax()))
        assert list(engine.request(request_id).output_token_ids) == tokens[len(prompt):]


# ------------------------------------------------------------------ faults that random weights would hide, made to show

WINDOW = 13
SHARP = bu.config(80, 32, [
    bu.layer(bu.attention(2, 1, 8, 12, 4, scale=1.0, softcap=8.0, base=50.0), None),
    bu.layer(bu.latent(2, 8, 4, 10, 12, WINDOW, scale=1.0, base=50.0), None),
    bu.layer(bu.mamba(2, 8, 6, 1, 3, 2), 20),
], (0, 2, 2))


def sharpen(tensors):
    """Queries and keys several times as large: the softmax sits on a few keys, so one key that is wrongly seen or left
    out moves the result; sinks of the scores' size; a recurrence that remembers hundreds of tokens."""
    bu.enlarge(tensors)
    for name in tensors:
        if name.endswith((".mix.q.norm", ".mix.k.norm")):
            tensors[name] = (tensors[name].float() * 1.5).to(tensors[name].dtype)
        if name.endswith(".uk"):
            tensors[name] = (tensors[name].float() * 2.0).to(tensors[name].dtype)
        if name.endswith(".sink"):
            tensors[name] = torch.full_like(tensors[name], 1.5)
        if name.endswith(".A_log"):
            tensors[name] = torch.full_like(tensors[name], -4.0)
        if name.endswith(".dt_bias"):
            tensors[name] = torch.full_like(tensors[name], -2.0)


def test_what_would_show(tmp_path, monkeypatch):
    """Sharp attention and a long memory, in portions and single tokens, against the plain implementation; and the control:
    the plain implementation with one mechanism changed lands far outside the bound."""
    kernel_refs.install(monkeypatch)
    folder = bu.write_model(SHARP, 21, tmp_path / "model", change=sharpen)
    requests = ru.make_requests({"vocab_size": 80}, 12, (61, 38))
    want = bu.plain_logits(folder, requests)
    for mode, trace in (("portions", ru.trace_portions(requests)), ("tail", ru.trace_tail(requests, 30)),
                        ("mixed", ru.trace_mixed(requests, 3, max_live=2))):
        got = ru.run_trace(folder, "float32", trace, tmp_path / mode, block_size=4, device="cpu", on_cpu=True)
        bu.compare(got, want, "float32", float32_factor=2.0)
    cfg, weights = bu.folder_weights(folder)
    tokens = requests["r0"]
    right = plain.forward(cfg, weights, tokens)
    bound = 2e-5 + 2e-4 * float(right.abs().max())

    def moved(change_cfg=None, change_weights=None, other_tokens=None):
        c, w = copy.deepcopy(cfg), dict(weights)
        if change_cfg:
            change_cfg(c)
        if change_weights:
            change_weights(w)
        apart = (plain.forward(c, w, other_tokens or tokens) - right).abs()
        return float(apart[-1].max() if other_tokens else apart.max())

    mixer = lambda c, i: c["layers"][i]["mixer"]      # noqa: E731
    assert moved(lambda c: mixer(c, 1)["mask"].update(size=WINDOW + 1)) > 50 * bound
    assert moved(lambda c: mixer(c, 1)["mask"].update(size=WINDOW - 1)) > 50 * bound
    assert moved(lambda c: mixer(c, 1)["rot"]["scaling"].update(factor=8.0)) > 10 * bound
    assert moved(lambda c: mixer(c, 1)["rot"].pop("scaling")) > 10 * bound
    assert moved(lambda c: mixer(c, 0).update(softcap=30.0)) > 50 * bound
    assert moved(lambda c: mixer(c, 0)["rot"].update(base=51.0)) > 5 * bound
    assert moved(lambda c: mixer(c, 0)["rot"].update(dims=8)) > 10 * bound
    assert moved(lambda c: c["loop"].update(times=1)) > 50 * bound
    assert moved(lambda c: c.update(logit_softcap=6.2)) > 10 * bound
    assert moved(other_tokens=[(tokens[0] + 1) % 80] + tokens[1:]) > 5 * bound         # the first token reaches the last

    def zero(name, index=slice(None)):
        def change(w):
            w[name] = w[name].clone()
            w[name][index] = 0.0
        return change
    assert moved(change_weights=lambda w: w.update({"l1.mix.sink": torch.full_like(w["l1.mix.sink"], -50.0)})) > 50 * bound
    for name in ("l0.mix.q.b", "l0.mix.k.b", "l0.mix.v.b"):
        assert moved(change_weights=zero(name)) > 5 * bound, name
    assert moved(change_weights=zero("loop.step", 0)) > 50 * bound and moved(change_weights=zero("loop.step", 1)) > 50 * bound
    assert moved(change_weights=zero("l2.mix.conv", (slice(None), 0))) > 10 * bound
    assert moved(change_weights=zero("l1.mix.g")) > 50 * bound                          # a gate of one half everywhere


def test_recalled_embedding_and_pass_vectors_show(folders):
    """Controls on the plain implementation: without the embedding's output in the later passes, with it in the first one
    too, or with the vectors of two passes exchanged, the logits are others."""
    cfg, weights = bu.folder_weights(folders["A"])
    tokens = requests_of("A", 2, (12,))["r0"]
    right, enter = plain.forward(cfg, weights, tokens), plain.enter_pass
    changed = {"never": lambda x, first, steps, n: x + steps[n], "always": lambda x, first, steps, n: x + first + steps[n],
               "exchanged": lambda x, first, steps, n: enter(x, first, steps.flip(0), n),
               "last": lambda x, first, steps, n: enter(x, first, steps[-1:].expand_as(steps), n)}
    try:
        for name, other in changed.items():
            plain.enter_pass = other
            assert float((plain.forward(cfg, weights, tokens) - right).abs().max()) > 1e-2 * float(right.abs().max()), name
    finally:
        plain.enter_pass = enter


# ------------------------------------------------------------------ each mechanism alone

def _ctx(dtype=torch.float32):
    from forge_engine_amd.parts.base import BuildContext
    return BuildContext(torch.device("cpu"), dtype)


def _batch(q_lens, before, slots):
    """The metadata of a step: sequence i brings q_lens[i] tokens behind before[i] cached ones."""
    positions, token_seq, cu_q = [], [], [0]
    for i, (n, b) in enumerate(zip(q_lens, before)):
        positions += list(range(b, b + n))
        token_seq += [i] * n
        cu_q.append(cu_q[-1] + n)
    ints = lambda values: torch.tensor(values, dtype=torch.int32)      # noqa: E731
    return SimpleNamespace(num_tokens=cu_q[-1], num_seqs=len(q_lens), positions=ints(positions), token_seq=ints(token_seq), cu_q=ints(cu_q),
                           state_slots=ints(slots), ctx_len=ints([n + b for n, b in zip(q_lens, before)]), max_q_len=max(q_lens),
                           max_ctx=64, num_decode=sum(n == 1 for n in q_lens), carry={})


def _fill(part, generator, scale=0.3):
    weights = {}
    for name, spec in part.param_specs().items():
        weights[name] = torch.randn(spec.shape, generator=generator) * scale
        part.set_param(name, weights[name].clone())
    part.finalize()
    return {name: t.double() for name, t in weights.items()}


STEPS = ([(0, 5), (0, 1)], [(5, 6), (1, 2)], [(6, 11), (2, 6)], [(11, 12), (6, 7)])


def _in_steps(part, inputs, want, cache):
    """Two sequences fed in pieces of unequal size through one part (among them steps of single tokens)."""
    for step in STEPS:
        batch = _batch([b - a for a, b in step], [a for a, _ in step], [2, 0])
        x = torch.cat([rows[a:b] for (a, b), rows in zip(step, inputs)])
        got = part.forward(x, batch, cache)
        at = 0
        for (a, b), expected in zip(step, want):
            assert torch.allclose(got[at:at + b - a].double(), expected[a:b], atol=3e-5), step
            at += b - a


def _view(part, block=4):
    from forge_engine_amd.cache.spec import CacheView
    paged = part.cache_needs().paged
    return CacheView(torch.zeros(7, paged.kv_heads, block, paged.head_dim), torch.zeros(7, paged.kv_heads, paged.value_width, block),
                     torch.tensor([[3, 1, 6], [0, 5, -1]], dtype=torch.int32), block, paged.window, {})


@pytest.mark.parametrize("sizes", [(4, 2, 8, 12, 4), (3, 3, 6, 5, 6), (10, 1, 16, 4, 2)])
def test_attention_with_biases_and_whole_norms(sizes, monkeypatch):
    """Biases come ahead of the norm over all heads at once, the norm ahead of the rotation."""
    from forge_engine_amd.models.budanex import _mixer
    from forge_engine_amd.parts.base import build_part
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(sizes[2])
    kind, mixer = bu.attention(*sizes, base=30.0, scale=0.9, softcap=1.5)
    part = build_part("mixer", _mixer(SimpleNamespace(width=10, norm_eps=1e-4), kind, mixer, "m"), _ctx())
    w = _fill(part, g, 0.6)
    inputs = [torch.randn(12, 10, generator=g), torch.randn(7, 10, generator=g)]
    want = [plain.attention_mixer(x.double(), w, "m", mixer, torch.arange(len(x)), 1e-4) for x in inputs]
    _in_steps(part, inputs, want, _view(part))


@pytest.mark.parametrize("sizes,more", [((3, 6, 4, 5, 9, 4), {}), ((2, 8, 8, 8, 6, None), {"scaling": None}), ((4, 5, 6, 3, 7, 1), {"rot_dims": 4}),
                                        ((1, 1, 2, 1, 1, 7), {"scaling": (1.5, 10, 2.0, 0.5)})])
def test_latent_attention_with_window_sink_and_gate(sizes, more, monkeypatch):
    from forge_engine_amd.models.budanex import _mixer
    from forge_engine_amd.parts.base import build_part
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(sizes[1])
    kind, mixer = bu.latent(*sizes, base=30.0, scale=0.7, **more)
    part = build_part("mixer", _mixer(SimpleNamespace(width=10, norm_eps=1e-4), kind, mixer, "m"), _ctx())
    w = _fill(part, g, 0.6)
    inputs = [torch.randn(12, 10, generator=g), torch.randn(7, 10, generator=g)]
    want = [plain.latent_attention_mixer(x.double(), w, "m", mixer, torch.arange(len(x)), 1e-4) for x in inputs]
    _in_steps(part, inputs, want, _view(part))


@pytest.mark.parametrize("bottleneck", [True, False])
def test_gate_and_window_beside_a_query_bottleneck(bottleneck, monkeypatch):
    """The options do not depend on where the queries come from: through a bottleneck the same mixer is the one with
    ``W_q = W_uq diag(w) W_dq`` normed in between."""
    from forge_engine_amd.parts.latent_attention import LatentAttention
    from forge_engine_amd.parts.plan import PartSpec
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(3)
    heads, dim, turned, vdim, rank, window, q_rank = 2, 6, 4, 5, 7, 3, 8 if bottleneck else None
    names = {"dq": "dq", "dq_norm": "dq.norm", "uq": "uq", "q": "q", "dkv": "dkv", "dkv_norm": "dkv.norm", "uk": "uk", "uv": "uv", "o": "o", "gate": "g"}
    part = LatentAttention(_ctx(), "m", hidden_size=10, num_heads=heads, head_dim=dim, rot_dim=turned, value_dim=vdim, q_rank=q_rank,
                           kv_rank=rank, eps=1e-4, scale=0.5, window=window, sink=True, output_gate=True, names=names,
                           position=PartSpec("rotary", {"head_dim": turned, "theta": 30.0, "precise": True, "interleaved": True}))
    w = _fill(part, g, 0.6)
    _, sizes = bu.latent(heads, dim, turned, vdim, rank, window, base=30.0, scale=0.5, scaling=None)
    inputs = [torch.randn(12, 10, generator=g), torch.randn(7, 10, generator=g)]
    want = []
    for x in inputs:
        h, weights = x.double(), dict(w)
        if bottleneck:      # the queries as columns that the input is extended by
            q = plain.rms_norm(h @ w["m.dq"].T, w["m.dq.norm"], 1e-4) @ w["m.uq"].T
            h = torch.cat([h, q], dim=1)
            wider = q.shape[1]
            for name in ("m.dkv", "m.g"):
                weights[name] = torch.cat([w[name], torch.zeros(w[name].shape[0], wider, dtype=torch.float64)], dim=1)
            weights["m.q"] = torch.cat([torch.zeros(wider, 10, dtype=torch.float64), torch.eye(wider, dtype=torch.float64)], dim=1)
        want.append(plain.latent_attention_mixer(h, weights, "m", sizes, torch.arange(len(x)), 1e-4))
    _in_steps(part, inputs, want, _view(part))


@pytest.mark.parametrize("sizes", [(4, 10, 6, 2, 4, 4), (2, 16, 17, 1, 1, 1), (6, 4, 1, 6, 2, 3)])
def test_state_space_mixer(sizes, monkeypatch):
    from forge_engine_amd.cache.spec import CacheView
    from forge_engine_amd.models.budanex import _mixer
    from forge_engine_amd.parts.base import build_part
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(sizes[0])
    kind, mixer = bu.mamba(*sizes)
    part = build_part("mixer", _mixer(SimpleNamespace(width=10, norm_eps=1e-4), kind, mixer, "m"), _ctx())
    w = _fill(part, g, 0.5)
    inputs = [torch.randn(12, 10, generator=g), torch.randn(7, 10, generator=g)]
    states = {name: torch.full((4, *spec.shape), 3.0) for name, spec in part.cache_needs().states().items()}
    for tensor in states.values():
        tensor[[2, 0]] = 0.0
    _in_steps(part, inputs, [plain.state_space_mixer(x.double(), w, "m", mixer, None, 1e-4) for x in inputs], CacheView(states=states))
    assert all(float(t[1].min()) == 3.0 for t in states.values())         # nobody else's slot was touched


def test_yarn_frequencies_and_interleaved_pairs():
    """The position part's frequencies against the plain ones; a rotation keeps its pairs' lengths times the magnitude, and
    scores depend on distances alone."""
    from forge_engine_amd.parts.rotary import RotaryPosition, YarnRotaryPosition
    for dims, base, scaling in ((16, 250.0, (8.0, 2048, 32.0, 1.0)), (8, 1e4, (2.0, 16, 4.0, 1.0)), (4, 50.0, (40.0, 4096, 1.0, 0.5)), (32, 1e6, (1.0, 100, 8.0, 2.0))):
        values = dict(zip(("factor", "original", "fast", "slow"), scaling))
        part = YarnRotaryPosition(_ctx(), head_dim=dims, theta=base, interleaved=True, **values)
        want, magnitude = plain.yarn_frequencies(dims, base, values)
        assert torch.allclose(part.inv_freq.double(), want, rtol=1e-6) and abs(part.magnitude() - magnitude) < 1e-12 and part.interleaved
        rot = {"dims": dims, "base": base, "scaling": values}
        g = torch.Generator().manual_seed(dims)
        x, y = torch.randn(1, dims, dtype=torch.float64, generator=g), torch.randn(1, dims, dtype=torch.float64, generator=g)
        turned = [plain.rotate_interleaved(t.expand(40, dims), torch.arange(40), rot) for t in (x, y)]
        pairs = turned[0].view(40, dims // 2, 2).norm(dim=-1) / x.view(1, dims // 2, 2).norm(dim=-1)
        assert torch.allclose(pairs, torch.full_like(pairs, magnitude))
        scores = turned[0] @ turned[1].T
        assert torch.allclose(scores[7:], torch.stack([scores[i, :].roll(7) for i in range(33)])[:, :].where(torch.arange(40) >= 7, scores[7:]))
        assert torch.allclose(kernel_refs._turn(x.float().expand(40, dims), torch.arange(40), part.inv_freq, dims, True, magnitude).double(),
                              turned[0], atol=1e-4)
    assert not RotaryPosition(_ctx(), head_dim=8, theta=10.0).interleaved
    with pytest.raises(ValueError):
        RotaryPosition(_ctx(), head_dim=8, theta=10.0, interleaved=True).table(None)


def test_sink_softmax_is_a_softmax_with_one_more_score():
    score = torch.tensor([[1.0, -2.0, 3.0], [-40.0, -50.0, -60.0]], dtype=torch.float64)
    for sink in (-100.0, 0.0, 2.0, 90.0):
        want = torch.softmax(torch.cat([score, torch.full((2, 1), sink, dtype=torch.float64)], dim=1), dim=1)[:, :3]
        assert torch.allclose(plain.sink_softmax(score, sink), want)


def test_pass_vectors_join_what_is_pending(monkeypatch):
    """The entry leaves its additions on top of a pending update (whole, in parts, normed, or none); a norm adds all of it
    up, for whole steps and chosen rows; other readers get a plain stream."""
    from forge_engine_amd.parts.base import Residual
    from forge_engine_amd.parts.entry import PassVectors
    from forge_engine_amd.parts.norm import LayerNorm, RMSNorm
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(2)
    part = PassVectors(_ctx(), "loop", hidden_size=6, passes=3)
    steps = _fill(part, g, 0.5)["loop.step"]
    x0 = torch.randn(5, 6, generator=g)
    for pending in ("none", "whole", "parts", "normed", "biased"):
        for reader in ("rms", "rows", "layer", "flush", "add", "biased"):
            batch, residual = SimpleNamespace(carry={}), Residual(x0.clone())
            part.begin(residual, batch)
            want = x0.double()
            for number in range(3):
                part.forward(residual, batch, number)
                want = (want if number == 0 else want + x0) + steps[number]
                if number == 2:
                    break
                update = torch.randn(*((2,) if pending == "parts" else ()), 5, 6, generator=g)
                residual.flush()
                if pending == "normed":
                    weight = torch.randn(6, generator=g)
                    residual.add_normed(update, weight, 1e-3)
                    want = want + plain.rms_norm(update.double(), weight.double(), 1e-3)
                elif pending == "biased":
                    bias = torch.randn(6, generator=g)
                    residual.add(update, bias)
                    want = want + update.double() + bias
                elif pending != "none":
                    residual.add(update)
                    want = want + (update.double().sum(0) if pending == "parts" else update.double())
            w = torch.randn(6, generator=g)
            norm = (LayerNorm(_ctx(), "n", size=6, eps=1e-3, leaf="", bias_leaf=None) if reader == "layer" else RMSNorm(_ctx(), "n", size=6, eps=1e-3, leaf=""))
            norm.set_param("n", w)
            if reader == "rows":
                rows = torch.tensor([4, 0], dtype=torch.int32)
                got, expected = norm.forward(residual, rows=rows), plain.rms_norm(want, w.double(), 1e-3)[rows.long()]
            elif reader == "rms":
                got, expected = norm.forward(residual), plain.rms_norm(want, w.double(), 1e-3)
            elif reader == "layer":
                centred = want - want.mean(1, keepdim=True)
                got, expected = norm.forward(residual), plain.rms_norm(centred, w.double(), 1e-3)
            elif reader == "flush":
                got, expected = residual.flush(), want
            elif reader == "add":
                residual.add(x0)
                got, expected = residual.flush(), want + x0
            else:
                update, shift = residual.take_biased()
                assert update is None and shift is None
                got, expected = residual.h, want
            assert torch.allclose(got.double(), expected, atol=2e-5), (pending, reader)
            if reader != "add":
                assert torch.allclose(residual.flush().double(), want, atol=2e-5), (pending, reader)
    with pytest.raises(ValueError):
        part.forward(Residual(x0.clone()), SimpleNamespace(carry={}), 3)


def test_embedding_norm_feed_forward_and_logit_cap(monkeypatch):
    from forge_engine_amd.models.talapel import DENSE_NAMES
    from forge_engine_amd.parts.embedding import LMHead, TokenEmbedding
    from forge_engine_amd.parts.mlp import SwiGLU
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(9)
    part = SwiGLU(_ctx(), "f", hidden_size=10, intermediate_size=16, activation="gelu_tanh", names=DENSE_NAMES)
    w = _fill(part, g, 1.0)
    x = torch.randn(6, 10, generator=g)
    assert torch.allclose(part.forward(x).double(), plain.dense_feed_forward(x.double(), w, "f"), atol=1e-4)
    assert abs(float(plain.gelu_tanh(torch.tensor(1.0))) - 0.841192) < 1e-6 and plain.gelu_tanh(torch.tensor(-9.0)).abs() < 1e-6
    with pytest.raises(ValueError):
        SwiGLU(_ctx(), "f", hidden_size=10, intermediate_size=16, activation="relu")
    embedding = TokenEmbedding(_ctx(), "embed", vocab_size=7, hidden_size=10, leaf="", norm_leaf="norm", norm_eps=1e-2)
    w = _fill(embedding, g, 0.5)
    ids = torch.tensor([3, 0, 6, 3], dtype=torch.int32)
    got = embedding.forward(SimpleNamespace(token_ids=ids, num_tokens=4)).h
    assert torch.allclose(got.double(), plain.rms_norm(w["embed"][ids.long()], w["embed.norm"], 1e-2), atol=1e-5)
    for cap, scale in ((3.0, 1.0), (None, 1.0), (2.0, 0.5)):
        head = LMHead(_ctx(), "head", vocab_size=7, hidden_size=10, leaf="", softcap=cap, scale=scale)
        w = _fill(head, g, 1.0)["head"]
        logits = x.double() @ w.T * scale
        assert torch.allclose(head.forward(x).double(), plain.capped(logits, cap), atol=1e-5)
    assert math.isclose(float(plain.capped(torch.tensor(1e6, dtype=torch.float64), 3.0)), 3.0)
