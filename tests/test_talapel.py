"""Talapel through the engine on the CPU, with the kernels' plain references patched in, against the
plain implementation (tests/plain_talapel.py): configuration and tensor names, each mechanism alone,
and that logits do not depend on how requests are cut into steps, batched, or placed in pages and
state slots.  The kernels themselves run in the GPU tests."""

from __future__ import annotations

import copy
from types import SimpleNamespace

import pytest
import torch

import kernel_refs
import replay_util as ru
import talapel_util as tu
from forge_engine_amd.config import ConfigError, SchedulerConfig, load_model_config
from forge_engine_amd.engine import build_engine, load_model
from forge_engine_amd.engine.loading import build_model
from forge_engine_amd.sampling import SamplingParams
from forge_engine_amd.weights.random_init import declared_tensors, random_tensors

plain = tu.plain
LENGTHS = {"A": (5, 1, 14, 31), "B": (2, 9, 47, 23), "C": (7, 18, 3, 1), "D": (12, 1, 25, 6)}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: tu.write_model(raw, 7, tmp_path_factory.mktemp(f"talapel_{name}"), change=tu.enlarge) for name, raw in tu.CONFIGS.items()}


def requests_of(name, seed, lengths):
    return ru.make_requests({"vocab_size": tu.CONFIGS[name]["vocab"]}, seed, lengths)


def test_configuration_names_and_shapes():
    config = load_model_config(tu.SMALL_A)
    assert config.architecture == "Talapel" and load_model_config(config.to_dict()) == config
    tensors = declared_tensors(config)
    for name, shape in {"embed": (90, 40), "head": (90, 40), "final.norm": (40,), "loop.in": (40, 80), "l0.norm1": (40,),
                        "l0.mix.q": (36, 40), "l0.mix.v": (24, 40), "l0.mix.g": (24, 40), "l0.mix.o": (40, 24), "l0.mlp.gate": (28, 40),
                        "l0.mlp.down": (40, 28), "l1.mix.left.q": (32, 40), "l1.mix.left.q.b": (32,), "l1.mix.left.k": (16, 40),
                        "l1.mix.left.v": (24, 40), "l1.mix.left.v.b": (24,), "l1.mix.left.g": (48, 40), "l1.mix.left.o": (40, 48),
                        "l1.mix.left.o.b": (40,), "l1.mix.right.in": (40 + 40 + 24 + 4, 40), "l1.mix.right.conv": (64, 4),
                        "l1.mix.right.conv.b": (64,), "l1.mix.right.dt_bias": (4,), "l1.mix.right.A_log": (4,), "l1.mix.right.D": (4,),
                        "l1.mix.right.norm": (40,), "l1.mix.right.o": (40, 40), "l1.mlp.table": (90, 2), "l1.mlp.e4.up": (20, 40),
                        "l1.mlp.e0.down": (40, 20)}.items():
        assert tuple(tensors[name].shape) == shape, name
    # retention has no biases, experts no gate and no router, a layer one norm; a layer without a feed-forward has none
    assert not any(n in tensors for n in ("l0.mix.q.b", "l1.mlp.e0.gate", "l1.mlp.router", "l0.norm2", "final.norm.b", "l0.norm1.b"))
    assert not any(n.startswith(("l3.mlp", "l4.mlp")) for n in tensors)
    assert "loop.in" not in declared_tensors(load_model_config(tu.SMALL_C))
    table = random_tensors(config, 3)["l2.mlp.table"]
    assert table.dtype == torch.int32 and all(sorted(row) == [0, 1, 2] for row in table.tolist())     # rows of different experts
    a, left = tu.SMALL_A, tu.side(3, 2, 8, 8, (2, 4, 4, 1, 2, 1))
    right = {n: tu.side(2, 2, 8, 8, sizes) for n, sizes in {"groups": (3, 4, 4, 2, 2, 1), "parts": (3, 4, 4, 1, 2, 5), "states": (2, 4, 300, 1, 2, 1),
                                                            "taps": (2, 4, 4, 1, 9, 1)}.items()}
    for broken in ({**a, "layers": []}, {**a, "layers": [{**a["layers"][0], "type": "attention"}]},
                   *({**a, "layers": [tu.layer(mixer, None)], "loop": None} for mixer in (left, *right.values())),
                   {**a, "layers": [tu.layer(tu.retention(2, 8, 8, 10), None)], "loop": None},                    # more turned dims than dims
                   {**a, "layers": [tu.layer(tu.retention(2, 8, 8, 4, decay=[0.5]), None)], "loop": None},        # a decay too few
                   {**a, "layers": [tu.layer(tu.retention(1, 8, 8, 4, decay=[0.0]), None)], "loop": None},
                   {**a, "layers": [tu.layer(tu.retention(1, 8, 8, 4), tu.moe(2, 3, 8))], "loop": None},          # more chosen than there are
                   {**a, "loop": {"start": 2, "stop": 2, "times": 2}}, {**a, "loop": {"start": 0, "stop": 6, "times": 2}},
                   {**a, "loop": {"start": 0, "stop": 2, "times": 0}}, {k: v for k, v in a.items() if k != "norm"}):
        with pytest.raises(ConfigError):
            load_model_config(broken)


def test_run_order_and_caches_of_the_passes():
    """Every pass has a cache slot and a state of its own; the stream is replaced ahead of each pass's first layer."""
    plan = build_model(load_model_config(tu.SMALL_A), dtype="float32", device="cpu").plan
    calls = plan.resolved_schedule()
    assert [(c.layer, c.enters) for c in calls] == plain.run_order(tu.SMALL_A)
    assert [c.layer for c in calls] == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4] and [c.cache for c in calls] == list(range(11))
    assert [c.enters for c in calls] == [i in (1, 4, 7) for i in range(11)]
    model = build_model(load_model_config(tu.SMALL_A), dtype="float32", device="cpu")
    needs = model.cache_needs()
    assert [n.paged is not None for n in needs] == [i in (1, 3, 4, 6, 7, 9) for i in range(11)]
    assert set(needs[1].states()) == {"right.matrix", "right.conv"} and needs[1].states()["right.conv"].shape == (3, 64)
    assert set(build_model(load_model_config(tu.SMALL_B), dtype="float32", device="cpu").cache_needs()[0].states()) == {"right.matrix"}


def test_plain_in_steps_equals_plain_whole(folders):
    """The plain implementation's own pin: a request run from explicit state, token by token and in
    portions, gives the logits of the whole-sequence functions."""
    for name in tu.CONFIGS:
        cfg, weights = tu.folder_weights(folders[name])
        tokens = requests_of(name, 5, (29,))["r0"]
        whole = plain.forward(cfg, weights, tokens)
        for cuts in ([1] * 29, [7, 2, 13, 1, 6]):
            stepper, at = plain.Stepper(cfg, weights), 0
            for size in cuts:
                got = stepper.step(tokens[at:at + size])
                assert torch.allclose(got, whole[at:at + size], atol=1e-9), (name, at)
                at += size


@pytest.mark.parametrize("name", sorted(tu.CONFIGS))
@pytest.mark.parametrize("mode", ["whole", "tail", "portions", "mixed"])
def test_replay_matches_plain(name, mode, folders, tmp_path, monkeypatch):
    """Whole prompts; a prompt and then token by token; portions down to two tokens; up to three
    live requests, portions beside single tokens."""
    kernel_refs.install(monkeypatch)
    requests = requests_of(name, 3, LENGTHS[name])
    trace = {"whole": ru.trace_whole, "tail": lambda r: ru.trace_tail(r, 16), "portions": ru.trace_portions,
             "mixed": lambda r: ru.trace_mixed(r, 5, max_live=3)}[mode](requests)
    got = ru.run_trace(folders[name], "float32", trace, tmp_path, block_size=tu.BLOCK_SIZE[name], device="cpu", on_cpu=True)
    tu.compare(got, tu.plain_logits(folders[name], requests), "float32")


def test_decoding_from_the_first_token(folders, tmp_path, monkeypatch):
    """One token a step from position 0 on, 75 steps, over many runs of the query temperature."""
    kernel_refs.install(monkeypatch)
    requests = requests_of("A", 8, (75,))
    got = ru.run_trace(folders["A"], "float32", ru.trace_tail(requests, 75), tmp_path, block_size=4, device="cpu", on_cpu=True)
    tu.compare(got, tu.plain_logits(folders["A"], requests), "float32")


def test_pages_and_state_slots_are_used_again(folders, tmp_path, monkeypatch):
    """Seven requests through four state slots and a pool smaller than their sum: every pass's recurrence and
    convolution start from nothing, whoever held the slot before."""
    kernel_refs.install(monkeypatch)
    for name in ("A", "B"):
        requests = requests_of(name, 4, (12, 20, 7, 16, 9, 3, 11))
        trace = ru.trace_mixed(requests, 9, max_live=4)
        assert sum(ru.round64(len(t)) for t in requests.values()) > trace.peak_tokens
        got = ru.run_trace(folders[name], "float32", trace, tmp_path / name, block_size=tu.BLOCK_SIZE[name], device="cpu", on_cpu=True)
        tu.compare(got, tu.plain_logits(folders[name], requests), "float32")


def test_greedy_generation_through_the_scheduler(folders, monkeypatch):
    kernel_refs.install(monkeypatch)
    _, model = load_model(folders["A"], dtype="float32", device="cpu")
    engine = build_engine(model, scheduler_config=SchedulerConfig(block_size=4, block_capacity=64, token_budget=8, max_batch_size=3),
                          eos_token_ids=())
    prompts = list(requests_of("A", 6, (11, 4, 17)).values())
    ids = [engine.submit(prompt, sampling_params=SamplingParams(max_new_tokens=6)) for prompt in prompts]
    engine.run_until_idle()
    cfg, weights = tu.folder_weights(folders["A"])
    for request_id, prompt in zip(ids, prompts):
        tokens = list(prompt)
        for _ in range(6):
            tokens.append(int(plain.forward(cfg, weights, tokens)[-1].argmax()))
        assert list(engine.request(request_id).output_token_ids) == tokens[len(prompt):]


# ------------------------------------------------------------------ faults that random weights would hide, made to show

SHARP = tu.config(80, 32, [
    tu.layer(tu.side(2, 1, 8, 12, (2, 8, 6, 1, 3, 2), scale=1.0, softcap=8.0, every=7, coef=0.6), tu.moe(4, 2, 16)),
    tu.layer(tu.retention(2, 8, 8, 4, base=50.0, decay=[0.999, 0.97]), None),
], (0, 2, 2), scale=3.0)


def sharpen(tensors):
    """Queries and keys several times as large: the softmax sits on a few keys, so one key that is wrongly left out, or a
    query temperature that is one position off, moves the result; decays near one, so the recurrence remembers
    hundreds of tokens."""
    tu.enlarge(tensors)
    for name in tensors:
        if name.endswith((".left.q", ".left.k")):
            tensors[name] = (tensors[name].float() * 3.0).to(tensors[name].dtype)
        if name.endswith(".A_log"):
            tensors[name] = torch.full_like(tensors[name], -4.0)
        if name.endswith(".dt_bias"):
            tensors[name] = torch.full_like(tensors[name], -2.0)


def test_what_would_show(tmp_path, monkeypatch):
    """Sharp attention and a long memory, in portions and single tokens, against the plain implementation; and the control:
    the plain implementation with one mechanism changed lands far outside the bound."""
    kernel_refs.install(monkeypatch)
    folder = tu.write_model(SHARP, 21, tmp_path / "model", change=sharpen)
    requests = ru.make_requests({"vocab_size": 80}, 12, (61, 38))
    want = tu.plain_logits(folder, requests)
    for mode, trace in (("portions", ru.trace_portions(requests)), ("tail", ru.trace_tail(requests, 30)),
                        ("mixed", ru.trace_mixed(requests, 3, max_live=2))):
        got = ru.run_trace(folder, "float32", trace, tmp_path / mode, block_size=4, device="cpu", on_cpu=True)
        tu.compare(got, want, "float32", float32_factor=2.0)
    cfg, weights = tu.folder_weights(folder)
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

    left = lambda c: c["layers"][0]["mixer"]["left"]      # noqa: E731
    assert moved(lambda c: left(c)["q_temp"].update(every=7.2)) > 10 * bound          # some runs of positions begin elsewhere
    assert moved(lambda c: left(c).update(softcap=30.0)) > 100 * bound
    assert moved(lambda c: c["loop"].update(times=1)) > 100 * bound
    assert moved(lambda c: c["layers"][1]["mixer"].update(decay=[0.998, 0.97])) > 10 * bound
    assert moved(lambda c: c["layers"][1]["mixer"]["rot"].update(base=51.0)) > 10 * bound
    assert moved(lambda c: c["layers"][0]["mixer"].update(right_scale=1.31)) > 10 * bound
    assert moved(other_tokens=[(tokens[0] + 1) % 80] + tokens[1:]) > 5 * bound         # the first token reaches the last

    def swap_experts(w):
        row = w["l0.mlp.table"].clone()
        row[tokens[-1]] = torch.tensor([e for e in range(4) if e not in row[tokens[-1]].tolist()], dtype=row.dtype)
        w["l0.mlp.table"] = row
    assert moved(change_weights=swap_experts) > 100 * bound

    def lose_oldest_tap(w):
        w["l0.mix.right.conv"] = w["l0.mix.right.conv"].clone()
        w["l0.mix.right.conv"][:, 0] = 0.0
    assert moved(change_weights=lose_oldest_tap) > 10 * bound


# ------------------------------------------------------------------ each mechanism alone

def _ctx():
    from forge_engine_amd.parts.base import BuildContext
    return BuildContext(torch.device("cpu"), torch.float32)


def _batch(q_lens, before, slots, tables=None, block_size=4):
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


def _in_steps(part, inputs, want, cache, states=True):
    """Two sequences fed in pieces of unequal size through one part (among them steps of single tokens)."""
    for step in STEPS:
        batch = _batch([b - a for a, b in step], [a for a, _ in step], [2, 0])
        x = torch.cat([rows[a:b] for (a, b), rows in zip(step, inputs)])
        got = part.forward(x, batch, cache)
        got = got.sum(0) if got.dim() == 3 else got
        at = 0
        for (a, b), expected in zip(step, want):
            assert torch.allclose(got[at:at + b - a].double(), expected[a:b], atol=2e-5), step
            at += b - a


def _states(part):
    states = {name: torch.full((4, *spec.shape), 3.0) for name, spec in part.cache_needs().states().items()}
    for tensor in states.values():
        tensor[[2, 0]] = 0.0
    return states


@pytest.mark.parametrize("sizes", [(4, 10, 6, 2, 4, 4), (2, 16, 17, 1, 1, 1), (6, 4, 1, 6, 2, 3), (3, 5, 9, 3, 8, 1)])
def test_state_space_across_steps(sizes, monkeypatch):
    from forge_engine_amd.cache.spec import CacheView
    from forge_engine_amd.parts.state_space import StateSpaceMixer
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(sizes[0])
    heads, vdim, state, groups, taps, parts = sizes
    part = StateSpaceMixer(_ctx(), "m", hidden_size=10, heads=heads, value_dim=vdim, state=state, groups=groups, conv_taps=taps,
                           norm_groups=parts, eps=1e-4, output_scale=-1.5)
    w = _fill(part, g, 0.5)
    inputs = [torch.randn(12, 10, generator=g), torch.randn(7, 10, generator=g)]
    right = dict(zip(("heads", "vdim", "state", "groups", "conv", "norm_groups"), sizes))
    states = _states(part)
    _in_steps(part, inputs, [-1.5 * plain.state_space_branch(x.double(), w, "m", right, 1e-4) for x in inputs], CacheView(states=states))
    assert float(states[part.STATE][1].min()) == 3.0         # nobody else's slot was touched


@pytest.mark.parametrize("heads,dim,vdim,turned,decay", [(3, 12, 8, 6, [0.5, 0.9, 0.999]), (1, 6, 11, 6, [1.0]), (2, 8, 4, 2, [0.25, 1.01])])
def test_retention_across_steps(heads, dim, vdim, turned, decay, monkeypatch):
    from forge_engine_amd.cache.spec import CacheView
    from forge_engine_amd.parts.plan import PartSpec
    from forge_engine_amd.parts.recurrent import Retention
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(dim)
    part = Retention(_ctx(), "m", hidden_size=10, heads=heads, dim=dim, value_dim=vdim, eps=1e-4, decay=decay,
                     position=PartSpec("rotary", {"head_dim": dim, "theta": 30.0, "rotary_dim": turned, "precise": True}))
    w = _fill(part, g, 0.5)
    inputs = [torch.randn(12, 10, generator=g), torch.randn(7, 10, generator=g)]
    sizes = {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"dims": turned, "base": 30.0}, "decay": decay}
    want = [plain.retention_mixer(x.double(), w, "m", sizes, torch.arange(len(x)), 1e-4) for x in inputs]
    _in_steps(part, inputs, want, CacheView(states=_states(part)))


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,every", [(4, 2, 8, 12, 3), (3, 3, 7, 5, 1), (6, 1, 16, 4, 4)])
def test_attention_with_temperature_cap_gate_and_factor(heads, kv_heads, dim, vdim, every, monkeypatch):
    """Biases everywhere, an odd head size, queries whose temperature changes inside a portion, across steps and pages."""
    from forge_engine_amd.cache.spec import CacheView
    from forge_engine_amd.models.talapel import ATTENTION_NAMES
    from forge_engine_amd.parts.attention import GroupedQueryAttention
    from forge_engine_amd.parts.plan import PartSpec
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(dim)
    part = GroupedQueryAttention(_ctx(), "m", hidden_size=10, num_heads=heads, num_kv_heads=kv_heads, head_dim=dim, value_dim=vdim, scale=0.9,
                                 softcap=1.5, query_temperature={"coef": 0.8, "every": every}, bias=True, output_gate=True, output_scale=0.6,
                                 position=PartSpec("none"), names=ATTENTION_NAMES, fill_rows=True)
    w = _fill(part, g, 0.6)
    inputs = [torch.randn(12, 10, generator=g), torch.randn(7, 10, generator=g)]
    sizes = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 0.9, "softcap": 1.5, "q_temp": {"coef": 0.8, "every": every}}
    want = [0.6 * plain.attention_branch(x.double(), w, "m", sizes, torch.arange(len(x))) for x in inputs]
    view = CacheView(torch.zeros(7, kv_heads, 4, dim), torch.zeros(7, kv_heads, vdim, 4),
                     torch.tensor([[3, 1, 6], [0, 5, -1]], dtype=torch.int32), 4, None, {})
    _in_steps(part, inputs, want, view)


def test_query_temperature_at_the_edges_of_its_runs():
    """The run begins one position before a multiple: p + 1 counts."""
    for every, first in ((4, 3), (1, 0), (10, 9), (2.5, 2)):
        t = plain.query_temperature(torch.arange(40), 0.5, every)
        assert float(t[0]) == (1.0 if first > 0 else 1.0 + 0.5 * torch.log(torch.tensor(2.0, dtype=torch.float64)))
        change = (t[1:] != t[:-1]).nonzero().flatten() + 1
        if first > 0:
            assert int(change[0]) == first and float(t[first - 1]) == 1.0
        q_out = torch.zeros(40, 2)
        kernel_refs.conv_rope_norm_write(
            torch.ones(40, 6), None, None, None, None, torch.arange(40, dtype=torch.int32), torch.zeros(40, dtype=torch.int32), torch.tensor([0, 40]),
            torch.zeros(1, dtype=torch.int32), torch.zeros(1, 1, dtype=torch.int32), torch.zeros(1, 1, 40, 2), torch.zeros(1, 1, 2, 40), q_out,
            num_seqs=1, q_heads=1, kv_heads=1, head_dim=2, value_dim=2, rotary_dim=0, unit_norm_eps=None, taps=0, q_temp=(0.5, every))
        assert torch.allclose(q_out[:, 0].double(), t, atol=1e-6)


@pytest.mark.parametrize("experts,top", [(5, 2), (3, 3), (4, 1), (1, 1)])
def test_experts_by_table_alone(experts, top, monkeypatch):
    from forge_engine_amd.models.talapel import EXPERT_NAMES
    from forge_engine_amd.parts.moe import RoutedExperts
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(experts * 10 + top)
    width, ff, vocab = 14, 9, 21
    part = RoutedExperts(_ctx(), "f", hidden_size=width, experts=experts, top=top, intermediate_size=ff, scoring="table", form="relu_squared",
                         router_bias=False, vocab_size=vocab, names=EXPERT_NAMES)
    w = {}
    for name, spec in part.param_specs().items():
        w[name] = (torch.rand(vocab, experts, generator=g).argsort(1)[:, :top].to(torch.int32) if spec.kind == "int_table"
                   else torch.randn(spec.shape, generator=g) * 0.5)
        part.set_param(name, w[name].clone())
    part.finalize()
    ids = torch.randint(0, vocab, (13,), generator=g, dtype=torch.int32)
    x, extra = torch.randn(13, width, generator=g), torch.randn(2, 13, width, generator=g)
    want = plain.table_experts(x.double(), ids.tolist(), {n: t if n.endswith("table") else t.double() for n, t in w.items()}, "f",
                               tu.moe(experts, top, ff))
    batch = SimpleNamespace(token_ids=ids, carry={})
    got = part.forward(x, batch)
    assert got.shape == (top, 13, width) and torch.allclose(got.sum(0).double(), want, atol=1e-5)
    assert list(batch.carry) == [("expert plan", "f")]          # the next pass through the layer finds its plan
    assert torch.allclose(part.forward(x, batch, extra=extra).sum(0).double(), want + extra.sum(0).double(), atol=1e-5)
    if experts > 1:
        part.table[3, 0] = experts
        with pytest.raises(ValueError, match="different experts"):
            part.finalize()
        if top > 1:
            part.table[3] = 0
            with pytest.raises(ValueError, match="different experts"):
                part.finalize()


def test_stream_entry_replaces_the_stream(monkeypatch):
    """The stream with its pending update and bias beside the embedding's output, twice in a step; a product in parts
    leaves its other parts pending."""
    from forge_engine_amd.kernels import ops
    from forge_engine_amd.parts.base import Residual
    from forge_engine_amd.parts.entry import ConcatProjection
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(2)
    part = ConcatProjection(_ctx(), "loop.in", hidden_size=6, leaf="")
    w = _fill(part, g, 0.5)["loop.in"]
    x0, update, bias = torch.randn(5, 6, generator=g), torch.randn(2, 5, 6, generator=g), torch.randn(6, generator=g)
    for parts in (None, 3):
        if parts:
            monkeypatch.setattr(ops, "linear_update", lambda x, weight: torch.stack([(x @ weight.T) / parts] * parts))
        residual, batch = Residual(x0.clone()), SimpleNamespace(carry={})
        part.begin(residual, batch)
        part.forward(residual, batch)
        first = torch.cat([x0, x0], dim=1).double() @ w.T
        residual.add(update.clone(), bias)
        part.forward(residual, batch)
        want = torch.cat([first + update.sum(0) + bias, x0.double()], dim=1) @ w.T
        assert torch.allclose(residual.flush().double(), want, atol=1e-5), parts


class _Inner:
    """A plain function between two matrices, as a part of a layer."""
    takes_stream = takes_extra = False

    def __init__(self, g, width, n, k, joint, bias=False):
        from forge_engine_amd.parts.base import JointEnds
        self.first, self.last = torch.randn(n, width, generator=g) * 0.4, torch.randn(width, k, generator=g) * 0.4
        self.bias, self.k, self.released = (torch.randn(width, generator=g) if bias else None), k, False
        self.ends = JointEnds(self.first, self.last, self.bias) if joint else None

    def joint_ends(self):
        return self.ends

    def release_ends(self):
        self.released = True

    def inner(self, z):
        return torch.tanh(z[:, :self.k]) + z[:, -self.k:]

    def forward_joint(self, z, out, *rest):
        out.copy_(self.inner(z))

    def forward(self, x, *rest, extra=None):
        y = self.inner(x @ self.first.T) @ self.last.T
        return y if self.bias is None else y + self.bias

    def plain(self, x):
        y = self.inner(x @ self.first.double().T) @ self.last.double().T
        return y if self.bias is None else y + self.bias.double()


@pytest.mark.parametrize("mixer_joint,ff_joint", [(True, True), (True, False), (False, True), (False, False), (True, None), (False, None)])
def test_parallel_arrangement(mixer_joint, ff_joint, monkeypatch):
    """Both sublayers read one norm; joined products, apart, or one of each; two layers in a row and the last norm over
    chosen rows, so that pending updates and biases meet every kind of reader."""
    from forge_engine_amd.parts.base import Residual
    from forge_engine_amd.parts.block import ParallelBlock
    from forge_engine_amd.parts.norm import LayerNorm, RMSNorm
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(5)
    width, tokens, eps = 12, 7, 1e-3
    norms = {role: LayerNorm(_ctx(), role, size=width, eps=eps, leaf="", bias_leaf=None) for role in ("input", "last")}
    nw = {role: _fill(norm, g, 0.8)[role] for role, norm in norms.items()}
    mixer = _Inner(g, width, 9, 5, mixer_joint, bias=True)
    ff = None if ff_joint is None else _Inner(g, width, 10, 8, ff_joint)
    block = ParallelBlock(_ctx(), mixer, ff, {"input": norms["input"]})
    block.assemble()
    assert mixer.released == mixer_joint and (ff is None or ff.released == (mixer_joint and ff_joint))
    x0 = torch.randn(tokens, width, generator=g)
    h = x0.double()
    for _ in range(2):
        x = plain.layer_norm(h, nw["input"], eps)
        h = h + mixer.plain(x) + (0 if ff is None else ff.plain(x))
    for reader in ("layer_norm", "rms_norm"):
        residual = Residual(x0.clone())
        block.forward(residual, None, None)
        block.forward(residual, None, None)
        rows = torch.tensor([5, 0], dtype=torch.int32)
        if reader == "layer_norm":
            got, want = norms["last"].forward(residual, rows=rows), plain.layer_norm(h, nw["last"], eps)[rows.long()]
        else:
            other = RMSNorm(_ctx(), "r", size=width, eps=eps, leaf="")
            weight = _fill(other, g, 1.0)["r"]
            got, want = other.forward(residual), plain.rms_unit(h, eps) * weight
        assert torch.allclose(got.double(), want, atol=1e-5), reader
        assert torch.allclose(residual.flush().double(), h, atol=1e-5)


def test_mixers_side_by_side_summed(monkeypatch):
    """The sum of branches, joined and apart; a branch without joint ends keeps all of them apart."""
    from forge_engine_amd.parts.parallel import ParallelMixers
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(6)
    for joint in ((True, True), (True, False)):
        part = ParallelMixers.__new__(ParallelMixers)
        part.combine, part.spans, part.hidden_size = "sum", [], 8
        part.branches = {"a": _Inner(g, 8, 7, 3, joint[0], bias=True), "b": _Inner(g, 8, 4, 4, joint[1])}
        x = torch.randn(5, 8, generator=g)
        want = sum(b.plain(x.double()) for b in part.branches.values())
        assert torch.allclose(part.forward(x, None, None).sum(0).double(), want, atol=1e-5)
        ends = part.joint_ends()
        assert (ends is not None) == all(joint)
        if ends is not None:
            inner = torch.zeros(5, ends.last.shape[1])
            part.forward_joint(x @ ends.first.T, inner, None, None)
            assert torch.allclose((inner @ ends.last.T + ends.bias).double(), want, atol=1e-5)


def test_dense_feed_forward_and_norm(monkeypatch):
    from forge_engine_amd.models.talapel import DENSE_NAMES
    from forge_engine_amd.parts.base import Residual
    from forge_engine_amd.parts.mlp import SwiGLU
    from forge_engine_amd.parts.norm import LayerNorm
    kernel_refs.install(monkeypatch)
    g = torch.Generator().manual_seed(9)
    part = SwiGLU(_ctx(), "f", hidden_size=10, intermediate_size=16, names=DENSE_NAMES)
    w = _fill(part, g, 0.5)
    x = torch.randn(6, 10, generator=g)
    want = plain.dense_feed_forward(x.double(), w, "f")
    assert torch.allclose(part.forward(x).double(), want, atol=1e-5)
    ends = part.joint_ends()
    inner = torch.zeros(6, 16)
    part.forward_joint(x @ ends.first.T, inner)
    assert torch.allclose((inner @ ends.last.T).double(), want, atol=1e-5)
    norm = LayerNorm(_ctx(), "n", size=10, eps=1e-2, leaf="", bias_leaf=None)
    weight = _fill(norm, g, 1.0)["n"]
    assert torch.allclose(norm.forward(Residual(3.0 * x + 5.0)).double(), plain.layer_norm(3.0 * x.double() + 5.0, weight, 1e-2), atol=1e-5)


def test_tables_of_cosines_are_formed_once_a_step(monkeypatch):
    from forge_engine_amd.kernels import ops
    from forge_engine_amd.parts.rotary import NoPosition, RotaryPosition
    kernel_refs.install(monkeypatch)
    calls = []
    monkeypatch.setattr(ops, "rotary_table", lambda *a: calls.append(a) or kernel_refs.rotary_table(*a))
    batch = _batch([3, 1], [0, 70], [0, 1])
    one, two = (RotaryPosition(_ctx(), head_dim=8, theta=100.0, precise=True) for _ in range(2))
    other = RotaryPosition(_ctx(), head_dim=8, theta=100.0, rotary_dim=4, precise=True)
    table = one.table(batch)
    assert two.table(batch) is table and other.table(batch).shape == (4, 2, 2) and len(calls) == 2
    x = torch.randn(4, 2, 8, dtype=torch.float64)
    turned = plain.rotate_half_layout(x, batch.positions, 8, 100.0)
    cos, sin = table[:, None, :, 0].double(), table[:, None, :, 1].double()
    assert torch.allclose(torch.cat([x[..., :4] * cos - x[..., 4:] * sin, x[..., 4:] * cos + x[..., :4] * sin], -1), turned, atol=1e-5)
    assert NoPosition(_ctx()).table(batch) is None


def test_matrices_stored_in_different_widths_stay_apart(monkeypatch, tmp_path):
    """A checkpoint that stores one branch's matrices in 32-bit: its products are not joined with the others', and the
    model still computes the same."""
    kernel_refs.install(monkeypatch)

    def widen(tensors):
        tu.enlarge(tensors)
        for name in list(tensors):
            if ".right." in name:
                tensors[name] = tensors[name].float()
    folder = tu.write_model(tu.SMALL_B, 3, tmp_path / "model", change=widen)
    _, model = load_model(folder, dtype="bfloat16", device="cpu")
    assert model.layers[0].first is None and model.layers[1].first is not None
    requests = requests_of("B", 3, (9, 14))
    got = ru.run_trace(folder, "bfloat16", ru.trace_portions(requests), tmp_path / "out", block_size=8, device="cpu", on_cpu=True)
    tu.compare(got, tu.plain_logits(folder, requests), "bfloat16", fraction=0.06)
