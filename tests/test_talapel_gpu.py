"""Talapel on the GPU: its kernels alone against their plain references (tests/kernel_refs.py), and
the model against the plain implementation (tests/plain_talapel.py) in float32 and bfloat16 over
traces that cut the same requests in different ways."""

from __future__ import annotations

import pytest
import torch

import kernel_refs as refs
import replay_util as ru
import talapel_util as tu

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
plain = tu.plain
DTYPES = [torch.float32, torch.bfloat16]

CONFIGS = dict(tu.CONFIGS, M=tu.MEDIUM)
LENGTHS = {"A": (5, 1, 14, 27, 90), "B": (2, 9, 21, 33, 64), "C": (7, 18, 3, 1, 40), "D": (12, 1, 25, 6, 50), "M": (4, 45, 170, 83, 1)}
BLOCKS = dict(tu.BLOCK_SIZE, M=16)


def close(got, want, dtype, loose=1.0):
    tolerance = (2e-5 if dtype == torch.float32 else 2e-2) * loose
    torch.testing.assert_close(got.float().cpu(), want.float(), rtol=tolerance, atol=tolerance)


def to_dev(*tensors):
    return [None if t is None else t.to(DEV) for t in tensors]


def layout(q_lens, slots, before=None):
    """(cu_q, token_seq, positions) of a step."""
    cu = [0]
    for n in q_lens:
        cu.append(cu[-1] + n)
    before = before or [0] * len(q_lens)
    return (torch.tensor(cu, dtype=torch.int32), torch.tensor([s for s, n in enumerate(q_lens) for _ in range(n)], dtype=torch.int32),
            torch.tensor([b + i for n, b in zip(q_lens, before) for i in range(n)], dtype=torch.int32))


def unit_scale(x):
    return x / x.abs().max().clamp(min=1.0)


# ------------------------------------------------------------------ the recurrence

SIZES = [  # heads, share, key dim, value dim, turned dims
    (3, 1, 12, 8, 6), (2, 2, 1, 5, 0), (4, 2, 16, 16, 16), (2, 1, 20, 70, 8), (6, 3, 48, 48, 0), (2, 1, 64, 64, 64),
    (3, 3, 64, 130, 16), (2, 1, 80, 33, 80), (4, 1, 128, 64, 96), (2, 2, 128, 128, 0), (1, 1, 150, 20, 30), (2, 1, 192, 65, 192),
    (2, 1, 256, 96, 256), (1, 1, 255, 9, 0)]


@pytest.mark.parametrize("heads,share,key_dim,value_dim,turned", SIZES)
@pytest.mark.parametrize("steps", [False, True])
@pytest.mark.parametrize("dtype", DTYPES)
def test_head_recurrence_kernels(heads, share, key_dim, value_dim, turned, steps, dtype):
    """Sequences of unequal length in one step (a single token, one short of a chunk, a whole number of chunks, an empty
    one that pads the step with a slot beyond the pool), whole and in segments, then a step of single tokens from the
    state they left; every count of key tiles, vector and single loads, inputs through strided views."""
    from forge_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(heads * 1000 + key_dim + value_dim)
    slots, shared = 6, heads // share * key_dim
    start = torch.randn(slots, heads, value_dim, key_dim, generator=g)
    inv_freq = torch.rand(turned // 2, generator=g) if turned else None
    if steps:
        rate = -torch.exp(torch.randn(heads, generator=g) * 0.7 - 1.0)
        dt_bias, skip = torch.randn(heads, generator=g) - 1.0, torch.randn(heads, generator=g)
    else:
        rate = torch.log(torch.tensor([1.0 - 2.0 ** -(1 + 2 * h) for h in range(heads)]))
        dt_bias = skip = None
    padding = 8 * (-(shared + heads * value_dim + heads) % 8 == 0) + 8
    for segment in (0, 32, 96):
        ref, gpu = start.clone(), start.clone().to(DEV)
        for q_lens in ([1, 37, 0, 64, 130], [31, 2, 0, 200, 1], [1, 1, 1, 1, 1]):
            single = max(q_lens) == 1
            cu_q, _, positions = layout(q_lens, slots, [0, 40, 0, 7, 300])
            tokens = sum(q_lens)
            state_slots = torch.tensor([3, 0, slots if not single else 1, 4, 5], dtype=torch.int32)
            wide = torch.randn(tokens, 2 * shared + heads * value_dim + heads + padding, generator=g)
            wide = (wide * (key_dim ** -0.25)).to(dtype)
            at = [padding, padding + shared, padding + 2 * shared, padding + 2 * shared + heads * value_dim]
            q, k, v = (wide[:, at[i]:at[i + 1]] for i in range(3))
            dt = wide[:, at[3]:at[3] + heads] if steps else None
            table = None if inv_freq is None else refs.rotary_table(positions, inv_freq)
            if table is not None:
                close(ops.rotary_table(positions.to(DEV), inv_freq.to(DEV)), table, torch.float32)
            kw = dict(num_seqs=5, heads=heads, share=share, key_dim=key_dim, value_dim=value_dim, q_scale=0.7, k_scale=1.1)
            want = refs.head_recurrence(q, k, v, ref, cu_q, state_slots, rate=rate, table=table, dt=dt, dt_bias=dt_bias, skip=skip, **kw)
            wide_gpu = wide.to(DEV)
            q, k, v = (wide_gpu[:, at[i]:at[i + 1]] for i in range(3))
            dt = wide_gpu[:, at[3]:at[3] + heads] if steps else None
            rate_g, table_g, bias_g, skip_g = to_dev(rate, table, dt_bias, skip)
            got = ops.head_recurrence(q, k, v, gpu, cu_q.to(DEV), state_slots.to(DEV), rate=rate_g, table=table_g, dt=dt,
                                      dt_bias=bias_g, skip=skip_g, single_tokens=single, segment=None if single else segment, **kw)
            scale = float(want.abs().max())
            assert float((got.cpu() - want).abs().max()) <= 3e-6 * scale * (1 + key_dim) ** 0.5, (segment, q_lens)
            assert float((gpu.cpu() - ref).abs().max()) <= 3e-6 * float(ref.abs().max()) * 4, (segment, q_lens)
            assert torch.equal(gpu[2].cpu(), start[2])          # nobody else's slot was touched


def test_decays_that_differ_by_orders_of_magnitude_within_a_chunk():
    """One token whose step wipes the state in front of tokens that keep nearly all of it: the products of the later
    tokens' decays must not be formed from sums that the large one has eaten the digits of."""
    from forge_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(4)
    heads, key_dim, value_dim, tokens = 2, 32, 16, 96
    rate, dt_bias = torch.tensor([-20.0, -16.0]), torch.zeros(heads)
    dt = torch.full((tokens, heads), -12.0)           # decays of about 1 - 1e-4
    dt[3] = dt[40] = 30.0                             # decays of e^-600
    q, k, v = (torch.randn(tokens, heads * n, generator=g) for n in (key_dim, key_dim, value_dim))
    ref = torch.randn(1, heads, value_dim, key_dim, generator=g)
    gpu = ref.clone().to(DEV)
    cu_q, slots = torch.tensor([0, tokens], dtype=torch.int32), torch.zeros(1, dtype=torch.int32)
    kw = dict(num_seqs=1, heads=heads, key_dim=key_dim, value_dim=value_dim)
    want = refs.head_recurrence(q, k, v, ref, cu_q, slots, rate=rate, dt=dt, dt_bias=dt_bias, **kw)
    got = ops.head_recurrence(*to_dev(q, k, v), gpu, cu_q.to(DEV), slots.to(DEV), rate=rate.to(DEV), dt=dt.to(DEV), dt_bias=dt_bias.to(DEV),
                              segment=0, **kw)
    for lo, hi in ((0, 3), (3, 4), (4, 40), (40, 41), (41, 96)):      # the runs differ in size: each by its own
        assert float((got.cpu() - want)[lo:hi].abs().max()) <= 1e-5 * float(want[lo:hi].abs().max()), (lo, hi)


@pytest.mark.parametrize("heads,key_dim,value_dim,turned", [(3, 12, 8, 6), (2, 64, 64, 64), (4, 128, 256, 128), (1, 256, 1024, 32), (2, 9, 700, 0), (2, 192, 130, 192)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_single_tokens_with_norm_and_gate(heads, key_dim, value_dim, turned, dtype):
    from forge_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(key_dim)
    slots, seqs = 5, 4
    ref = torch.randn(slots, heads, value_dim, key_dim, generator=g) * 0.3
    gpu = ref.clone().to(DEV)
    cu_q, _, positions = layout([1] * seqs, slots, [0, 5, 900, 3])
    state_slots = torch.tensor([2, 4, 0, slots], dtype=torch.int32)        # the last one's slot is beyond the pool: left alone
    table = refs.rotary_table(positions, torch.rand(turned // 2, generator=g)) if turned else None
    rate = torch.log(torch.rand(heads, generator=g))
    q, k, v, gate = (torch.randn(seqs, heads * n, generator=g).to(dtype) for n in (key_dim, key_dim, value_dim, value_dim))
    want = torch.zeros(seqs, heads * value_dim, dtype=dtype)
    kw = dict(eps=1e-4, heads=heads, key_dim=key_dim, value_dim=value_dim, k_scale=key_dim ** -0.5)
    refs.head_recurrence_gated(q[:3], k[:3], v[:3], ref, cu_q[:4], state_slots[:3], gate[:3], want[:3], num_seqs=3, rate=rate,
                               table=None if table is None else table[:3], **kw)
    out = torch.zeros(seqs, heads * value_dim + 3, dtype=dtype, device=DEV)
    ops.head_recurrence_gated(*to_dev(q, k, v), gpu, cu_q.to(DEV), state_slots.to(DEV), gate.to(DEV), out[:, 3:], num_seqs=seqs,
                              rate=rate.to(DEV), table=None if table is None else table.to(DEV), **kw)
    close(out[:, 3:], want, dtype)
    close(gpu, ref, torch.float32)
    assert float(out[:, :3].abs().max()) == 0.0


# ------------------------------------------------------------------ the smaller kernels

@pytest.mark.parametrize("channels,taps", [(40, 4), (300, 2), (33, 8), (64, 3)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_convolution_of_single_tokens(channels, taps, dtype):
    """Several steps of single tokens, the state's move in the same launch, against the reference."""
    from forge_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(channels)
    weight, bias = torch.randn(channels, taps, generator=g), torch.randn(channels, generator=g)
    ref = torch.randn(4, taps - 1, channels, generator=g)
    gpu = ref.clone().to(DEV)
    cu_q, token_seq, _ = layout([1, 1, 1], 4)
    slots = torch.tensor([3, 0, 1], dtype=torch.int32)
    for _ in range(taps + 2):
        u = torch.randn(3, channels + 5, generator=g).to(dtype)
        want = refs.causal_conv_act(u[:, 5:], weight, bias, ref, token_seq, cu_q, slots, num_seqs=3)
        got = ops.causal_conv_act(u.to(DEV)[:, 5:], weight.to(DEV), bias.to(DEV), gpu, token_seq.to(DEV), cu_q.to(DEV), slots.to(DEV),
                                  num_seqs=3, single_tokens=True)
        close(got, want, dtype)
        close(gpu, ref, torch.float32)


@pytest.mark.parametrize("rows,width,groups", [(3, 40, 1), (5, 96, 4), (2, 6000, 1), (7, 2048, 2), (1, 9, 3), (130, 512, 8)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_gate_then_norm_in_parts(rows, width, groups, dtype):
    from forge_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    y, z = torch.randn(rows, width, generator=g) * torch.rand(rows, 1, generator=g), torch.randn(rows, width + 7, generator=g).to(dtype)
    weight = torch.randn(width, generator=g)
    want = torch.empty(rows, width, dtype=dtype)
    refs.gated_group_norm(y, z[:, 7:], weight, want, groups=groups, eps=1e-3)
    for pad in (0, 8):
        out = torch.zeros(rows, width + pad, dtype=dtype, device=DEV)
        zg = (torch.nn.functional.pad(z[:, 7:], (pad, 0)) if pad else z[:, 7:].contiguous()).to(DEV)
        ops.gated_group_norm(y.to(DEV), zg[:, pad:], weight.to(DEV), out[:, pad:], groups=groups, eps=1e-3)
        close(out[:, pad:], want, dtype)


@pytest.mark.parametrize("rows,width,parts", [(1, 24, 0), (5, 40, 1), (3, 256, 4)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_stream_sum_and_bias_on_an_update(rows, width, parts, dtype):
    """The stream with its update and a bias: in the compute dtype beside something else, and through the layer norm's
    kernel (written back, and for chosen rows)."""
    from forge_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    h, shift, weight = torch.randn(rows, width, generator=g), torch.randn(width, generator=g), torch.randn(width, generator=g)
    update = None if parts == 0 else torch.randn(parts, rows, width, generator=g)
    for bias in (None, shift):
        want = refs.stream_sum_cast(h, update, bias, torch.empty(rows, width, dtype=dtype))
        out = torch.zeros(rows, 2 * width, dtype=dtype, device=DEV)
        ops.stream_sum_cast(*to_dev(h, update, bias), out[:, width:])
        close(out[:, width:], want, dtype)
        assert float(out[:, :width].abs().max()) == 0.0
    for chosen in (None, torch.tensor([rows - 1, 0], dtype=torch.int32)):
        ref, gpu = h.clone()[None], h.clone()[None].to(DEV)
        count = rows if chosen is None else 2
        want = refs.hyper_norm(ref, update, None, None, None, weight, None, 1e-5, torch.empty(count, width, dtype=dtype), rows=chosen,
                               store=chosen is None, shift=shift)
        got = ops.hyper_norm(gpu, *to_dev(update), None, None, None, weight.to(DEV), None, 1e-5, torch.empty(count, width, dtype=dtype, device=DEV),
                             rows=None if chosen is None else chosen.to(DEV), store=chosen is None, shift=shift.to(DEV))
        close(got, want, dtype)
        close(gpu, ref, torch.float32)
    ref, gpu = h.clone()[None], h.clone()[None].to(DEV)
    refs.hyper_norm(ref, update, None, None, None, None, None, 0.0, None, shift=shift)
    ops.hyper_norm(gpu, *to_dev(update), None, None, None, None, None, 0.0, None, shift=shift.to(DEV))
    close(gpu, ref, torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
def test_strided_rows_of_activations_and_gates(dtype):
    from forge_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(1)
    for rows, inter, pad in ((3, 20, 5), (9, 64, 8)):
        gate_up = torch.randn(rows, 2 * inter + pad, generator=g).to(dtype)
        want = refs.swiglu(gate_up[:, pad:], torch.empty(rows, inter, dtype=dtype))
        out = torch.zeros(rows, inter + pad, dtype=dtype, device=DEV)
        ops.swiglu(gate_up.to(DEV)[:, pad:], out[:, pad:])
        close(out[:, pad:], want, dtype)
        assert float(out[:, :pad].abs().max()) == 0.0
        o, gate = torch.randn(rows, 4, inter // 4, generator=g), torch.randn(rows, inter + pad, generator=g).to(dtype)
        want = refs.head_norm_gate(o, None, gate[:, pad:], torch.empty(rows, inter, dtype=dtype), heads=4, dim=inter // 4, eps=1e-5, act="silu")
        out.zero_()
        ops.head_norm_gate(o.to(DEV), None, gate.to(DEV)[:, pad:], out[:, pad:], heads=4, dim=inter // 4, eps=1e-5, act="silu")
        close(out[:, pad:], want, dtype)
        assert float(out[:, :pad].abs().max()) == 0.0


@pytest.mark.parametrize("tokens,experts,top,hidden,inner", [(1, 3, 1, 40, 24), (23, 5, 2, 64, 96), (7, 4, 4, 48, 20), (700, 6, 2, 128, 160), (90, 16, 3, 256, 64)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_experts_that_a_table_names(tokens, experts, top, hidden, inner, dtype):
    """One matrix an expert and a squared relu, the plan from the token ids alone; an update of the same tokens in parts
    joins the first choice's."""
    from forge_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(tokens)
    vocab = 50
    table = torch.rand(vocab, experts, generator=g).argsort(1)[:, :top].to(torch.int32)
    ids = torch.randint(0, vocab, (tokens,), generator=g, dtype=torch.int32)
    x = torch.randn(tokens, hidden, generator=g).to(dtype)
    up = (torch.randn(experts, inner, hidden, generator=g) * hidden ** -0.5).to(dtype)
    down = (torch.randn(experts, hidden, inner, generator=g) * inner ** -0.5).to(dtype)
    extra = torch.randn(2, tokens, hidden, generator=g)
    offsets, order, weights = ops.moe_plan_table(ids.to(DEV), table.to(DEV), experts)
    chosen = table[ids.long()].reshape(-1)
    assert torch.equal(weights.cpu(), torch.full((tokens, top), 1.0 / top))
    for e in range(experts):
        mine = order[int(offsets[e]):int(offsets[e + 1])].cpu().sort().values
        assert torch.equal(mine.long(), (chosen == e).nonzero().flatten())
    want = refs.moe_experts(x, chosen.view(tokens, top), torch.full((tokens, top), 1.0 / top), up, down, torch.empty(top, tokens, hidden),
                            extra=extra, form="relu_squared")
    got = ops.moe_experts(x.to(DEV), None, weights, up.to(DEV), down.to(DEV), torch.empty(top, tokens, hidden, device=DEV),
                          extra=extra.to(DEV), form="relu_squared", plan=(offsets, order))
    close(got, want, dtype)


ATTENTION = [(4, 2, 64, 64, 16), (8, 1, 128, 128, 32), (4, 2, 48, 96, 16), (3, 3, 10, 6, 4), (6, 2, 128, 64, 8), (2, 1, 64, 128, 16)]


@pytest.mark.parametrize("heads,kv_heads,dim,vdim,block", ATTENTION)
@pytest.mark.parametrize("filled", [False, True])
@pytest.mark.parametrize("dtype", DTYPES)
def test_queries_by_position_and_one_key_that_stands_out(heads, kv_heads, dim, vdim, block, filled, dtype):
    """Biases and the query temperature on the way into the pages, then capped attention with a gate and a factor, into
    rows of another stride: a portion and single tokens at page borders, far behind and right behind the one key that
    stands out; the temperature's runs begin in the middle of a portion.  ``filled``: pages whose rows are wider than the
    heads, as the matrix-core kernels want them (what lies in the rest of a value may be anything)."""
    from forge_engine_amd.kernels import ops
    g = torch.Generator().manual_seed(dim + vdim)
    scale, cap, temp = dim ** -0.5, 6.0, (0.8, 37)
    before = [0, 5 * block, 3 * block - 1, 400]
    q_lens = [40, 1, 2, 1]
    tokens, seqs = sum(q_lens), len(q_lens)
    ctx = torch.tensor([b + n for b, n in zip(before, q_lens)], dtype=torch.int32)
    cu_q, token_seq, positions = layout(q_lens, 0, before)
    pages = [-(-int(c) // block) for c in ctx]
    table = torch.full((seqs, max(pages)), -1, dtype=torch.int32)
    free = torch.randperm(sum(pages), generator=g).tolist()
    for s, n in enumerate(pages):
        table[s, :n] = torch.tensor([free.pop() for _ in range(n)], dtype=torch.int32)
    channels = (heads + kv_heads) * dim + kv_heads * vdim
    row = (64 if max(dim, vdim) <= 64 else 128) if filled else 0
    key_row, value_row = max(row, dim), max(row, vdim)
    for target in ("first", "border"):
        key_pages = torch.zeros(sum(pages), kv_heads, block, key_row, dtype=dtype)
        key_pages[..., :dim] = torch.randn(sum(pages), kv_heads, block, dim, generator=g).to(dtype)
        value_pages = torch.randn(sum(pages), kv_heads, value_row, block, generator=g).to(dtype)
        qkv = torch.randn(tokens, channels + heads * vdim, generator=g).to(dtype)
        bias = torch.randn(channels, generator=g)
        q = torch.empty(tokens, heads * key_row, dtype=dtype)
        for s, n in enumerate(pages):          # a key of every cached context that all queries of its sequence favour
            place = 0 if target == "first" else max(0, (before[s] // block) * block - 1)
            if place < before[s]:
                favourite = qkv[int(cu_q[s + 1]) - 1, :heads * dim].float() + bias[:heads * dim]
                for hk in range(kv_heads):
                    head = favourite[hk * (heads // kv_heads) * dim:][:dim]
                    key_pages[int(table[s, place // block]), hk, place % block, :dim] = (12.0 * head / head.norm()).to(dtype)
        got_pages = [key_pages.clone().to(DEV), value_pages.clone().to(DEV)]
        kw = dict(num_seqs=seqs, q_heads=heads, kv_heads=kv_heads, head_dim=dim, value_dim=vdim, rotary_dim=0, unit_norm_eps=None, taps=0, q_temp=temp)
        slots = torch.zeros(seqs, dtype=torch.int32)
        refs.conv_rope_norm_write(qkv, bias, None, None, None, positions, token_seq, cu_q, slots, table, key_pages, value_pages, q, **kw)
        q_gpu = torch.full((tokens, heads * key_row), 7.0, dtype=dtype, device=DEV)
        wide = qkv.to(DEV)
        ops.conv_rope_norm_write(wide, bias.to(DEV), None, None, None, *to_dev(positions, token_seq, cu_q, slots, table), *got_pages, q_gpu, **kw)
        close(q_gpu, q, dtype)
        for got, want in zip(got_pages, (key_pages, value_pages)):
            close(got, want, dtype)
        want = torch.empty(tokens, heads * vdim, dtype=dtype)
        kw = dict(num_seqs=seqs, max_q_len=max(q_lens), q_heads=heads, kv_heads=kv_heads, head_dim=dim, value_dim=vdim, scale=scale, softcap=cap,
                  factor=-1.7)
        refs.masked_attention(q, key_pages, value_pages, want, cu_q, ctx, table, gate=qkv[:, channels:], **kw)
        out = torch.zeros(tokens, heads * vdim + 8, dtype=dtype, device=DEV)
        ops.masked_attention(q.to(DEV), key_pages.to(DEV), value_pages.to(DEV), out[:, 8:], *to_dev(cu_q, ctx, table), gate=wide[:, channels:],
                             num_decode=2, max_ctx=int(ctx.max()), **kw)
        close(out[:, 8:], want, dtype, loose=2.0)
        assert float(out[:, :8].abs().max()) == 0.0


# ------------------------------------------------------------------ the model

@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    kept = {}

    def of(name, dtype):
        if (name, dtype) not in kept:
            kept[(name, dtype)] = tu.write_model(CONFIGS[name], 7, tmp_path_factory.mktemp(f"talapel_{name}"),
                                                 change=lambda tensors: tu.enlarge(tensors, tu.ENLARGED[dtype]))
        return kept[(name, dtype)]

    return of


@pytest.fixture(scope="module")
def plain_of(folders):
    kept = {}

    def of(name, dtype, seed, lengths):
        key = (name, dtype, seed, lengths)
        if key not in kept:
            requests = ru.make_requests({"vocab_size": CONFIGS[name]["vocab"]}, seed, lengths)
            kept[key] = requests, tu.plain_logits(folders(name, dtype), requests)
        return kept[key]

    return of


TRACES = {"whole": ru.trace_whole, "tail": lambda r: ru.trace_tail(r, 24), "portions": ru.trace_portions,
          "mixed": lambda r: ru.trace_mixed(r, 5, max_live=4)}


@pytest.mark.parametrize("name", sorted(CONFIGS))
@pytest.mark.parametrize("mode", sorted(TRACES))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_traces_match_the_plain_implementation(name, mode, dtype, folders, plain_of, tmp_path):
    requests, want = plain_of(name, dtype, 3, LENGTHS[name])
    got = ru.run_trace(folders(name, dtype), dtype, TRACES[mode](requests), tmp_path, block_size=BLOCKS[name])
    tu.compare(got, want, dtype, float32_factor=2.0)


def sharpen(tensors):
    """Queries and keys larger and decays near one: one key of hundreds, and the first token, reach the logits."""
    tu.enlarge(tensors, 3.0)
    for name in tensors:
        if name.endswith((".left.q", ".left.k")):
            tensors[name] = (tensors[name].float() * 2.0).to(tensors[name].dtype)
        if name.endswith(".A_log"):
            tensors[name] = torch.full_like(tensors[name], -4.0)
        if name.endswith(".dt_bias"):
            tensors[name] = torch.full_like(tensors[name], -2.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_requests_with_sharp_attention_and_a_long_memory(dtype, tmp_path):
    """Prompts of several hundred tokens, so that recurrences are walked in segments: whole, then the last 40 tokens one
    by one, then in portions, then three at once; and the control that the first token moves the last logits."""
    raw = dict(tu.MEDIUM, layers=[dict(layer) for layer in tu.MEDIUM["layers"]])
    raw["layers"][1] = tu.layer(tu.retention(4, 64, 128, 64, decay=[0.999, 0.9999, 0.99, 1.0]), raw["layers"][1]["mlp"])
    folder = tu.write_model(raw, 32, tmp_path / "sharp", change=sharpen)
    requests = ru.make_requests({"vocab_size": raw["vocab"]}, 9, (500, 333, 129))
    want = tu.plain_logits(folder, requests)
    cfg, weights = tu.folder_weights(folder)
    changed = [(requests["r0"][0] + 1) % raw["vocab"]] + requests["r0"][1:]
    last = want[("r0", 499)]
    assert float((plain.forward(cfg, weights, changed)[-1] - last).abs().max()) > 20 * (1e-5 + 1e-4 * float(last.abs().max()))
    for mode, trace in (("whole", ru.trace_whole(requests)), ("tail", ru.trace_tail(requests, 40)),
                        ("portions", ru.trace_portions(requests, sizes=(64, 17, 2, 230, 3, 48, 16, 2, 33), want_all=False)),
                        ("mixed", ru.trace_mixed(requests, 11, max_live=3))):
        got = ru.run_trace(folder, dtype, trace, tmp_path / mode, block_size=16)
        tu.compare(got, want, dtype, fraction=0.06, float32_factor=4.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_captured_steps_equal_eager_steps_and_long_decoding(dtype, folders, plain_of):
    """A prompt and then 150 single tokens, two requests side by side: steps replayed from captured graphs against the
    same steps run eagerly (states move on once a step either way), and both against the plain implementation; then
    portions whose shape repeats, captured and replayed with other contents."""
    from forge_engine_amd.engine import ModelRunner, StepEntry, load_model
    _, model = load_model(folders("M", dtype), dtype=dtype, device=DEV)
    requests, want = plain_of("M", dtype, 21, (160, 171))
    results = {}
    for graphs in (True, False):
        runner = ModelRunner(model, block_size=16, block_capacity=40, num_state_slots=3, use_graphs=graphs, eager_sightings=1)
        got = {}
        for name in requests:
            runner.begin(name)
        at = {"r0": 10, "r1": 21}
        logits = runner.step([StepEntry(n, requests[n][:at[n]], [at[n] - 1]) for n in requests])
        for row, n in zip(logits, requests):
            got[(n, at[n] - 1)] = row.cpu().clone()
        for _ in range(150):
            logits = runner.step([StepEntry(n, [requests[n][at[n]]], [0]) for n in requests])
            for row, n in zip(logits, requests):
                got[(n, at[n])] = row.cpu().clone()
                at[n] += 1
        assert runner.graph_replays >= (140 if graphs else 0) and (graphs or runner.graph_replays == 0)
        for name in requests:
            runner.end(name)
            runner.begin(name)
        replays = runner.portion_graph_replays
        for start in range(0, 160, 40):          # the same shape four times: eager, captured, replayed
            logits = runner.step([StepEntry(n, requests[n][start:start + 40], [39]) for n in requests])
            for row, n in zip(logits, requests):
                got[(n, start + 39, "portions")] = row.cpu().clone()
        assert runner.portion_graph_replays - replays >= (2 if graphs else 0)
        results[graphs] = got
        tu.compare({key[:2]: row for key, row in got.items() if len(key) == 2}, want, dtype, float32_factor=2.0)
        tu.compare({key[:2]: row for key, row in got.items() if len(key) == 3}, want, dtype, float32_factor=2.0)
    for key, row in results[True].items():
        torch.testing.assert_close(row, results[False][key], rtol=0, atol=1e-4 if dtype == "float32" else 3e-2)


def test_first_tokens_and_slot_reuse(folders):
    """A request that takes over the state slot of one that ended starts from empty states in every pass, whatever the
    slot still holds; requests of one and two tokens."""
    from forge_engine_amd.engine import ModelRunner, StepEntry, load_model
    folder = folders("A", "float32")
    _, model = load_model(folder, dtype="float32", device=DEV)
    runner = ModelRunner(model, block_size=4, block_capacity=16, num_state_slots=1)
    cfg, weights = tu.folder_weights(folder)
    for tokens in ([5, 80, 17, 3], [44], [7, 7], [80, 5, 17, 3, 3, 3, 8, 1, 2]):
        runner.begin("only")
        rows = [runner.step([StepEntry("only", [token], [0])])[0].cpu().clone() for token in tokens]
        runner.end("only")
        for got, row in zip(rows, plain.forward(cfg, weights, tokens)):
            assert float((got.double() - row).abs().max()) <= 2e-5 + 2e-4 * float(row.abs().max())


def test_generation_through_the_entry_point_and_the_command_line(folders):
    import os
    import subprocess
    import sys
    from conftest import ROOT
    from forge_engine_amd.config import SchedulerConfig
    from forge_engine_amd.engine import engine_from_folder
    from forge_engine_amd.sampling import SamplingParams

    folder = folders("A", "float32")
    cfg, weights = tu.folder_weights(folder)

    def greedy(prompt, count):
        tokens = list(prompt)
        for _ in range(count):
            tokens.append(int(plain.forward(cfg, weights, tokens)[-1].argmax()))
        return tokens[len(prompt):]

    prompts = list(ru.make_requests({"vocab_size": tu.SMALL_A["vocab"]}, 13, (11, 3, 25)).values())
    want = [greedy(prompt, 8) for prompt in prompts]
    engine = engine_from_folder(folder, scheduler_config=SchedulerConfig(block_size=4, block_capacity=128, token_budget=16),
                                dtype="float32", eos_token_ids=[])
    ids = [engine.submit(prompt, sampling_params=SamplingParams(max_new_tokens=8)) for prompt in prompts]
    engine.run_until_idle()
    assert [list(engine.request(i).output_token_ids) for i in ids] == want
    command = [sys.executable, str(ROOT / "bin" / "forge-engine"), "generate", "--model", str(folder), "--dtype", "float32",
               "--max-new-tokens", "8", "--block-size", "4", "--prompt-ids", ",".join(map(str, prompts[0]))]
    done = subprocess.run(command, capture_output=True, text=True, timeout=300, env=dict(os.environ))
    assert done.returncode == 0, done.stderr[-2000:]
    assert ",".join(map(str, want[0])) in done.stdout.replace(" ", "")
