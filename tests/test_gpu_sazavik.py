"""Sazavik on the GPU: the kernels and kernel forms it added against their plain PyTorch references, every mechanism alone
against the plain implementation (tests/sazavik_plain.py), and whole models through the step function, the scheduler and
the entry points: whole prompts, portions down to two tokens, token-by-token decoding, unequal batches, pages and slots
that are used again, keys far away and just inside and outside every window and chunk, the first tokens, long decoding,
keys that another layer cached, and sizes of many kinds."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import ref_ops
import sazavik_configs
import sazavik_plain
from part_harness import DEV, PartHarness
from test_gpu_pemarax import attention_case, close, feed_every_way, i32, paged, query_tiles_of, rand, rounded

pytestmark = pytest.mark.gpu

F32_GATE = 2e-4
DTYPES = [torch.float32, torch.bfloat16]
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def ops():
    from macllm_infer_amd.kernels import build, ops as module
    build.ensure_modules(["common", "gemm", "moe", "attention", "attention_widths", "decode"])
    return module


def on(tensor):
    return None if tensor is None else tensor.to(DEV)


# ------------------------------------------------------------------ kernels against their references
@pytest.mark.parametrize("out_dtype", DTYPES)
@pytest.mark.parametrize("d, T", [(48, 7), (50, 3), (1, 5), (256, 700), (1022, 2), (4100, 9), (4096, 600), (16384, 3), (16383, 2)])
def test_branches_join_the_stream_through_an_rms_norm_of_their_own(out_dtype, d, T):
    h = rand(T, d, seed=1)
    weights = [rand(d, seed=2) * 0.2 + 1.0, rand(d, seed=3) * 0.2 + 1.0]
    branches = [(rand(T, d, seed=4, scale=3.0).to(torch.bfloat16), 1.0), (rand(T, d, seed=5), -0.5), (rand(T, d, seed=6), 0.25)]
    rows = i32([T - 1, 0, T // 2])
    for count in (1, 2, 3):
        for picked in (None, rows):
            want_h, got_h = h.clone(), h.clone().to(DEV)
            shape = (T if picked is None else len(picked), d)
            want, got = torch.empty(shape, dtype=out_dtype), torch.empty(shape, dtype=out_dtype, device=DEV)
            ref_ops.add_normed_rmsnorm(want_h, branches[:count], (weights[0], 1e-4), weights[1], 1e-5, want, picked)
            ops().add_normed_rmsnorm(got_h, [(on(b), f) for b, f in branches[:count]], (on(weights[0]), 1e-4), on(weights[1]), 1e-5,
                                     got, on(picked))
            close(got.float(), want.float(), out_dtype, f"{count} branches, rows {picked is not None}")
            close(got_h, want_h, torch.float32, "the stream")
            if picked is not None:
                assert torch.equal(got_h.cpu(), h), "a gather leaves the stream as it is"
    ops().add_normed_rmsnorm(got_h, [(on(branches[0][0]), 1.0)], (on(weights[0]), 1e-4), None, 0.0, None)
    ref_ops.add_normed_rmsnorm(want_h := h.clone(), branches[:1], (weights[0], 1e-4), None, 0.0, None)
    close(got_h, want_h, torch.float32, "the add alone")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T, d", [(1, 48), (33, 250), (300, 1024), (700, 1030), (2, 3000), (2, 5000), (3, 16384)])
def test_the_embedding_through_a_norm(dtype, T, d):
    table = rand(50, d, seed=1, scale=3.0).to(dtype)
    ids = torch.randint(0, 50, (T,), generator=torch.Generator().manual_seed(2)).to(torch.int32)
    weight = rand(d, seed=3) * 0.3 + 1.0
    want, got = torch.empty(T, d), torch.empty(T, d, device=DEV)
    ref_ops.embed(ids, table, 0.7, want, norm=(weight, 1e-5))
    ops().embed(ids.to(DEV), table.to(DEV), 0.7, got, norm=(weight.to(DEV), 1e-5))
    close(got, want, torch.float32, "normed rows")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("inner, tile", [(40, 0), (40, 8), (37, 0), (256, 8)])
def test_the_clamped_gate_of_a_dense_feed_forward(dtype, inner, tile):
    from macllm_infer_amd.config import ClampedGLUSpec
    for limit in (0.5, 7.0):
        clamp = ClampedGLUSpec(limit=limit)
        gate_up = rand(19, 2 * inner, seed=1, scale=2.0).to(dtype)
        want, got = torch.empty(19, inner, dtype=dtype), torch.empty(19, inner, dtype=dtype, device=DEV)
        ref_ops.swiglu(gate_up, want, tile, activation="clamped", clamp=clamp)
        ops().swiglu(gate_up.to(DEV), got, tile, activation="clamped", clamp=clamp)
        close(got.float(), want.float(), dtype, f"limit {limit}")


@pytest.mark.parametrize("rows, width, inner", [(1, 64, 24), (5, 96, 40), (16, 1024, 64)])
def test_the_clamped_gate_in_the_product_s_epilogue(rows, width, inner):
    from macllm_infer_amd.config import ClampedGLUSpec
    clamp = ClampedGLUSpec(limit=0.8)
    x = rand(rows, width, seed=1).to(torch.bfloat16)
    weight = (rand(2 * inner, width, seed=2) * 2.0 / width ** 0.5).to(torch.bfloat16)
    got = torch.empty((rows, inner), dtype=torch.bfloat16, device=DEV)
    ops().fused_gemm(weight.to(DEV), None, got, x=x.to(DEV), epilogue=ops().EPI_SWIGLU, gate_activation="clamped", clamp=clamp)
    want = torch.empty((rows, inner), dtype=torch.bfloat16)
    ref_ops.swiglu((x.float() @ weight.float().T).to(torch.bfloat16), want, 8, activation="clamped", clamp=clamp)
    close(got.float(), want.float(), torch.bfloat16, "activated rows")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("Hq, Hkv, dh, dv, rotary, interleaved, head_norm, temperature", [
    (4, 2, 16, 8, 16, True, "before_rotation", None), (3, 1, 12, 20, 6, False, "before_rotation", (0.5, 3)),
    (5, 5, 7, 9, 0, False, "before_rotation", (-0.2, 1)), (6, 2, 128, 64, 32, True, "after_rotation", (0.1, 1000)),
    (2, 1, 250, 256, 250, False, None, (0.3, 7))])
@pytest.mark.parametrize("alone", [False, True])
@pytest.mark.parametrize("T", [21, 600])
def test_a_row_is_made_ready_with_a_temperature_and_without_keys(dtype, Hq, Hkv, dh, dv, rotary, interleaved, head_norm,
                                                                 temperature, alone, T):
    """``alone``: a row of queries whose keys and values another layer has cached.  Few rows go head by head, many as
    whole rows."""
    page, pages = 4, T // 4 + 3
    kv = 0 if alone else Hkv
    width = (Hq + kv) * dh + kv * dv
    qkv = rand(T, width + 5, seed=1).to(dtype)
    positions = i32([3 * t for t in range(T)])
    inv_freq = (torch.rand(rotary // 2, generator=torch.Generator().manual_seed(2)) + 0.01) if rotary else None
    weights = [(rand(dh, seed=s) * 0.2 + 1.0) if head_norm else None for s in (3, 4)]
    cells = None if alone else torch.randperm(page * pages, generator=torch.Generator().manual_seed(5))[:T].to(torch.int32)
    want_k, want_v = torch.zeros((pages, Hkv, page, dh), dtype=dtype), torch.zeros((pages, Hkv, dv, page), dtype=dtype)
    got_k, got_v = paged(want_k, want_v)
    how = dict(interleaved=interleaved, head_norm=head_norm, head_eps=1e-5 if head_norm else 0.0, temperature=temperature)
    want, got = qkv.clone(), qkv.clone().to(DEV)
    ref_ops.attention_prepare(want, Hq, kv, dh, dv, positions, inv_freq, rotary, cells, want_k, want_v, q_head_weight=weights[0],
                              k_head_weight=weights[1], **how)
    ops().attention_prepare(got, Hq, kv, dh, dv, on(positions), on(inv_freq), rotary, on(cells), None if alone else got_k,
                            None if alone else got_v, q_head_weight=on(weights[0]), k_head_weight=on(weights[1]), **how)
    close(got[:, :Hq * dh].float(), want[:, :Hq * dh].float(), dtype, "queries")
    assert torch.equal(got[:, Hq * dh:].cpu(), qkv[:, Hq * dh:]), "only the queries are written back"
    close(got_k.float(), want_k.float(), dtype, "cached keys")
    close(got_v.float(), want_v.float(), dtype, "cached values")


def seen_first(position, window, chunk):
    return position - position % chunk if chunk else max(0, position - window + 1) if window else 0


CASES = [
    # Hq, Hkv, dh, dv, window, chunk, slopes, sink, gate, [(context, new)], page
    (4, 2, 16, 24, None, 9, False, True, True, [(70, 70), (40, 1), (300, 33), (27, 27)], 8),
    (6, 2, 64, 64, None, 100, False, True, True, [(600, 600), (100, 100), (101, 2), (530, 1), (300, 100)], 16),
    (3, 3, 32, 8, None, 300, True, False, False, [(700, 130), (299, 299), (301, 1), (600, 300)], 4),
    (8, 2, 128, 128, 70, None, True, True, True, [(900, 64), (280, 280), (70, 70), (71, 2)], 16),
    (6, 1, 64, 64, None, None, True, False, False, [(257, 257), (1030, 40)], 16),
    (5, 5, 7, 9, 11, None, True, False, True, [(50, 50), (12, 1), (30, 9)], 8),
    (2, 1, 80, 40, None, 64, False, False, True, [(129, 129), (64, 64), (65, 1), (200, 8)], 32),
    (4, 1, 96, 128, 33, None, True, True, False, [(400, 400), (120, 100)], 8),
    (6, 6, 48, 48, None, 257, False, True, True, [(514, 300), (257, 257), (258, 1)], 16),
    (12, 2, 128, 128, None, 48, False, False, False, [(100, 100), (96, 48), (97, 1)], 16),
    (10, 1, 40, 64, 5, None, True, True, True, [(64, 64), (6, 6)], 4),
]


def chunked_case(case, dtype, seed=0):
    Hq, Hkv, dh, dv, window, chunk, slopes, sink, gate, lengths, page = case
    q, k_cache, v_cache, tables, lane_of, positions, cu, starts = attention_case(Hq, Hkv, dh, dv, lengths, page, dtype, seed=seed)
    terms = dict(chunk=chunk, slopes=rand(Hq, seed=8).abs() * 0.1 if slopes else None, sinks=rand(Hq, seed=9) if sink else None,
                 gate=rand(q.shape[0], Hq * dv, seed=10).to(dtype) if gate else None)
    clean_k, clean_v = torch.nan_to_num(k_cache.float()).to(dtype), torch.nan_to_num(v_cache.float()).to(dtype)
    want = torch.empty((q.shape[0], Hq * dv), dtype=dtype)
    ref_ops.paged_attention(q, Hq, Hkv, dh, clean_k, clean_v, tables.clamp(min=0), lane_of, positions, dh ** -0.5, window, want,
                            value_dim=dv, **terms)
    # what no query of the step sees holds NaN: a kernel that reads a cell it should not shows it
    for lane, (context, new) in enumerate(lengths):
        for position in range(0, seen_first(context - new, window, chunk)):
            k_cache[tables[lane, position // page], :, position % page, :] = float("nan")
            v_cache[tables[lane, position // page], :, :, position % page] = float("nan")
    device = dict(terms, slopes=on(terms["slopes"]), sinks=on(terms["sinks"]), gate=on(terms["gate"]))
    return q, (k_cache, v_cache), (clean_k, clean_v), tables, lane_of, positions, cu, starts, want, device


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", CASES)
def test_the_general_kernels_take_chunks_slopes_and_gates(case, dtype):
    Hq, Hkv, dh, dv, window, chunk, _, _, _, lengths, page = case
    q, caches, _, tables, lane_of, positions, cu, _, want, terms = chunked_case(case, dtype)
    for tiled in (False, True):
        got = torch.empty(want.shape, dtype=dtype, device=DEV)
        more = dict(query_tiles=query_tiles_of(cu, 64).to(DEV), tile_tokens=64, cu_seqlens=cu.to(DEV)) if tiled else {}
        ops().paged_attention(q.to(DEV), Hq, Hkv, dh, *paged(*caches), tables.clamp(min=0).to(DEV), lane_of.to(DEV), positions.to(DEV),
                              dh ** -0.5, window, got, max(c for c, _ in lengths), value_dim=dv, **terms, **more)
        close(got.float(), want.float(), dtype, f"tiled={tiled}")


@pytest.mark.parametrize("case", [case for case in CASES if case[2] % 8 == 0 and case[3] % 4 == 0])
def test_the_matrix_core_prompt_kernels_take_chunks_slopes_gates_and_any_width(case):
    Hq, Hkv, dh, dv, window, chunk, _, _, _, lengths, page = case
    q, _, clean, tables, _, _, cu, starts, want, terms = chunked_case(case, torch.bfloat16, seed=3)
    got = torch.empty(want.shape, dtype=torch.bfloat16, device=DEV)
    assert ops().prefill_attention_supported(torch.bfloat16, Hq, Hkv, dh, page, dv)
    ops().prefill_attention(q.to(DEV), Hq, Hkv, dh, *paged(*clean), tables.clamp(min=0).to(DEV), query_tiles_of(cu, 64).to(DEV),
                            cu.to(DEV), starts.to(DEV), dh ** -0.5, window, got, max(c for c, _ in lengths), value_dim=dv, **terms)
    close(got.float(), want.float(), torch.bfloat16, "prompt portions")


@pytest.mark.parametrize("case", [case for case in CASES if case[2] % 8 == 0 and case[10] % 8 == 0 and case[0] // case[1] <= 8])
def test_the_split_context_decode_kernel_takes_chunks_slopes_gates_and_any_key_width(case):
    contexts = [1, 2, 5, 47, 48, 49, 63, 64, 65, 99, 100, 101, 256, 257, 258, 600]
    case = case[:9] + ([(context, 1) for context in contexts], case[10])
    Hq, Hkv, dh, dv, window, chunk, _, _, _, lengths, page = case
    q, _, clean, tables, lane_of, positions, _, _, want, terms = chunked_case(case, torch.bfloat16, seed=5)
    got = torch.empty(want.shape, dtype=torch.bfloat16, device=DEV)
    ops().decode_attention(q.to(DEV), Hq, Hkv, dh, *paged(*clean), tables.clamp(min=0).to(DEV), lane_of.to(DEV), positions.to(DEV),
                           dh ** -0.5, window, max(contexts), got, value_dim=dv, **terms)
    close(got.float(), want.float(), torch.bfloat16, "single tokens")


@pytest.mark.parametrize("T, experts, top", [(1, 5, 2), (37, 12, 3), (300, 70, 8), (9, 4, 4), (64, 130, 1)])
def test_sigmoid_scores_choose_and_weigh_as_they_are(T, experts, top):
    logits = rand(T, experts + 2, seed=experts, scale=2.0)
    how = dict(routing="sigmoid_then_top", renormalize=False)
    want_chosen, want_weights, want_gate = ref_ops.moe_route(logits, experts, top, None, 1.0, 0.0, True, **how)
    chosen, weights, gate = ops().moe_route(logits.to(DEV), experts, top, None, 1.0, 0.0, True, **how)
    assert torch.equal(chosen.cpu(), want_chosen)
    close(weights, want_weights, torch.float32, "weights")
    close(gate, want_gate, torch.float32, "the shared expert's gate")
    # the same scores with a correction, groups and shares of their sum: the other options of the choice
    correction = rand(experts, seed=4) * 0.3
    want_chosen, want_weights, _ = ref_ops.moe_route(logits, experts, top, correction, 2.0, 1e-20, False, routing="sigmoid_then_top")
    chosen, weights, _ = ops().moe_route(logits.to(DEV), experts, top, correction.to(DEV), 2.0, 1e-20, False, routing="sigmoid_then_top")
    assert torch.equal(chosen.cpu(), want_chosen)
    close(weights, want_weights, torch.float32, "shares")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T, experts, top, hidden, inner, pad", [(5, 4, 2, 40, 24, 16), (130, 6, 3, 64, 96, 64), (600, 3, 2, 128, 64, 128),
                                                                 (3, 9, 9, 20, 12, 16), (64, 5, 1, 36, 20, 64)])
def test_weights_multiply_what_an_expert_is_given(dtype, T, experts, top, hidden, inner, pad):
    from macllm_infer_amd.config import SILU_GLU
    x = rand(T, hidden, seed=1).to(dtype)
    matrices = (rand(experts, 2 * inner, hidden, seed=2) * 2.0 / hidden ** 0.5).to(dtype)
    down_matrices = (rand(experts, hidden, inner, seed=3) / inner ** 0.5).to(dtype)
    logits = rand(T, experts, seed=4, scale=2.0)
    how = dict(routing="sigmoid_then_top", renormalize=False)
    chosen, weights, _ = ref_ops.moe_route(logits, experts, top, None, 1.0, 0.0, False, **how)
    shared, gate = rand(T, hidden, seed=5).to(dtype), torch.rand(T, generator=torch.Generator().manual_seed(6))
    plans = [ops().moe_plan(chosen.to(DEV), experts, pad, weights.to(DEV))]
    if T <= ops().ROUTE_PLAN_TOKENS:
        _, _, _, together = ops().moe_route_plan(logits.to(DEV), experts, top, None, 1.0, 0.0, False, experts_with_matrices=experts,
                                                 pad=pad, place_weights=True, **how)
        plans.append(together)
    want_plan = ref_ops.MoePlan(chosen, experts, pad, weights)
    want_inner = torch.empty((want_plan.capacity, inner), dtype=dtype)
    ref_ops.moe_expert_gemm(x, want_plan, matrices, want_inner, True, SILU_GLU, row_scale=want_plan.place_weight)
    want_down = torch.empty((want_plan.capacity, hidden))
    ref_ops.moe_expert_gemm(want_inner, want_plan, down_matrices, want_down, False, None)
    want = torch.empty(T, hidden)
    ref_ops.moe_combine(want_down, want_plan, None, shared, gate, want)
    for plan in plans:
        places = plan.place.cpu().long()
        close(plan.place_weight.cpu()[places], weights.reshape(-1), torch.float32, "weights beside the places")
        padding = torch.ones(plan.capacity, dtype=torch.bool)
        padding[places] = False
        assert float(plan.place_weight.cpu()[padding].abs().sum()) == 0.0
        got_inner = torch.empty((plan.capacity, inner), dtype=dtype, device=DEV)
        ops().moe_expert_gemm(x.to(DEV), plan, matrices.to(DEV), got_inner, gather=True, glu=SILU_GLU, row_scale=plan.place_weight)
        close(got_inner.float().cpu()[places], want_inner.float()[want_plan.place.long()], dtype, "activated rows")
        got_down = torch.empty((plan.capacity, hidden), dtype=torch.float32, device=DEV)
        ops().moe_expert_gemm(got_inner, plan, down_matrices.to(DEV), got_down, gather=False, glu=None)
        got = torch.empty((T, hidden), dtype=torch.float32, device=DEV)
        ops().moe_combine(got_down, plan, None, shared.to(DEV), gate.to(DEV), got)
        close(got, want, dtype, "the sum")


@pytest.mark.parametrize("rows, width, out", [(3, 64, 40), (17, 64, 40), (65, 96, 50), (700, 256, 1000)])
def test_a_bias_that_bfloat16_holds_goes_into_the_library_s_product(rows, width, out):
    x, weight = rand(rows, width, seed=1).to(torch.bfloat16), (rand(out, width, seed=2) / width ** 0.5).to(torch.bfloat16)
    bias = rand(out, seed=3).to(torch.bfloat16).float()
    want = (x.float() @ weight.float().T + bias).to(torch.bfloat16)
    got = ops().linear(x.to(DEV), weight.to(DEV), bias.to(DEV), bias16=bias.to(torch.bfloat16).to(DEV))
    close(got.float(), want.float(), torch.bfloat16, "with the bias in the product")
    apart = ops().linear(x.to(DEV), weight.to(DEV), bias.to(DEV))
    assert float((got.float() - apart.float()).abs().max()) <= 2.0 ** -7 * float(want.abs().max()), "one rounding either way"
    from macllm_infer_amd.parts import BuildContext, Linear
    build = BuildContext(hidden_size=width, dtype=torch.bfloat16, device=torch.device(DEV), max_context=64)
    assert Linear([weight], [bias], build).bias16 is not None and Linear([weight], [bias + 1e-4], build).bias16 is None


# ------------------------------------------------------------------ every mechanism alone
def mixer_parts(layer, hidden, seed, sharpen=1.0):
    """(spec, tensors under the part's names, the design's mixer table, tensors under the stored names)."""
    from macllm_infer_amd.config.sazavik import _FORMS, _attention
    kind, table = layer["type"], layer["mixer"]
    form = sazavik_plain.FORMS[kind]
    spec = _attention(table, "mixer", 1e-5, _FORMS[kind])
    H, G, dim, vdim = table["heads"], table["kv_heads"], table["dim"], table["vdim"]
    shapes = {"q": (H * dim, hidden), "k": (G * dim, hidden), "v": (G * vdim, hidden), "o": (hidden, H * vdim)}
    stored = {name: rand(*shape, seed=seed + i) / shape[1] ** 0.5 for i, (name, shape) in enumerate(shapes.items())}
    if form["gate"]:
        stored["g"] = rand(H * vdim, hidden, seed=seed + 5) * 2.0 / hidden ** 0.5
    if form["bias"]:
        for i, name in enumerate(("q", "k", "v", "o")):
            stored[f"{name}.b"] = rand(shapes[name][0], seed=seed + 6 + i) * 0.3
    if form["sink"]:
        stored["sink"] = rand(H, seed=seed + 11) + 1.0
    for i, name in enumerate(("q.norm", "k.norm")):
        stored[name] = (1.0 + 0.2 * rand(dim, seed=seed + 12 + i)) * sharpen
    tensors = {}
    for name, value in stored.items():
        head, _, rest = name.partition(".")
        if name == "sink":
            tensors[name] = value
        elif rest == "norm":
            tensors[f"{head}_norm.weight"] = value
        else:
            tensors[f"{head}_proj.{'bias' if rest == 'b' else 'weight'}"] = value
    return spec, tensors, table, stored


def plain_mixer(kind, x, table, stored, eps=1e-5):
    get = lambda name: stored[name].double()
    kept = sazavik_plain.keys_and_values(x.double(), table, sazavik_plain.FORMS[kind], get, eps)
    return sazavik_plain.attention(x.double(), kind, table, get, eps, kept).float()


LAYERS = [
    sazavik_configs.chunked(6, 2, 8, 12, 21, 4, base=300.0), sazavik_configs.chunked(4, 1, 64, 64, 40, 64),
    sazavik_configs.chunked(3, 3, 128, 128, 64, 32, base=1e6), sazavik_configs.chunked(5, 1, 24, 40, 5, 24),
    sazavik_configs.chunked(2, 2, 96, 96, 300, 40), sazavik_configs.chunked(4, 2, 16, 16, None, 8),
    sazavik_configs.chunked(4, 2, 20, 12, 33, 20, halves=True), sazavik_configs.chunked(6, 2, 64, 64, 100, 48, halves=True),
    sazavik_configs.chunked(1, 1, 48, 128, 16, 48, halves=True, scale=0.3), sazavik_configs.chunked(2, 1, 128, 128, 1, 128, halves=True),
    sazavik_configs.distant(3, 1, 10, 6, 13, every=7), sazavik_configs.distant(7, 7, 48, 40, 60, coef=0.6, every=32),
    sazavik_configs.distant(6, 2, 64, 64, 37, every=64), sazavik_configs.distant(5, 5, 7, 9, 11, coef=-0.2, every=3),
    sazavik_configs.distant(12, 2, 128, 128, 90, every=1), sazavik_configs.distant(4, 1, 32, 256, None, every=None),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layer", LAYERS)
def test_an_attention_alone(dtype, layer):
    hidden, T = 56, 330
    spec, tensors, table, stored = mixer_parts(layer, hidden, 30)
    tensors, stored = rounded(tensors, dtype), rounded(stored, dtype)
    x = rand(T, hidden, seed=2).to(dtype).float()
    want = plain_mixer(layer["type"], x, table, stored)
    feed_every_way(lambda: PartHarness(spec, tensors, hidden, dtype, page_size=8, capacity=1000), x, want, dtype,
                   beside=rand(40, hidden, seed=3))


def crafted(layer, T, distance, dtype):
    """A mixer fed rows of which the one ``distance`` before the last scores far above all others for the last query,
    if it is seen at all: the same input, norms strong enough that equal rows give a large score, and keys that are
    projected as the queries are.  The distance bias and the temperature are part of the score."""
    hidden = 64
    spec, tensors, table, stored = mixer_parts(layer, hidden, 50)
    H, G, dim = table["heads"], table["kv_heads"], table["dim"]
    # one projection for all heads, so that a key's row equals its query's before the rotation
    one = rand(dim, hidden, seed=70) / hidden ** 0.5
    stored["q"], stored["k"] = one.repeat(H, 1), one.repeat(G, 1)
    for name in ("q.b", "k.b"):
        if name in stored:
            stored[name] = torch.zeros_like(stored[name])
    # equal rows score the same at any distance: the few turned dims weigh next to nothing
    stored["q.norm"] = torch.full((dim,), 3.0)
    stored["q.norm"][:table.get("rot", {}).get("dims", 0)] = 0.05
    stored["k.norm"] = stored["q.norm"].clone()
    tensors.update({"q_proj.weight": stored["q"], "k_proj.weight": stored["k"], "q_norm.weight": stored["q.norm"], "k_norm.weight": stored["k.norm"]})
    for name in ("q", "k"):
        if f"{name}.b" in stored:
            tensors[f"{name}_proj.bias"] = stored[f"{name}.b"]
    tensors, stored = rounded(tensors, dtype), rounded(stored, dtype)
    x = rand(T, hidden, seed=71).to(dtype).float()
    target = T - 1 - distance
    x[target] = 2.0 * x[T - 1]               # the same direction, hence the same key; its value is twice as large
    want = plain_mixer(layer["type"], x, table, stored)
    away = x.clone()
    away[target] = rand(1, hidden, seed=72)[0].to(dtype).float()
    without = plain_mixer(layer["type"], away, table, stored)
    share = float((want[-1] - without[-1]).abs().max() / want[-1].abs().max())
    return spec, tensors, x, want, share


EDGES = ([("chunk", size, T, distance, dim) for dim in (16, 64, 96) for size, T in ((100, 700), (64, 640), (64, 641), (257, 514))
          for distance in sorted({1, 15, 16, 17, (T - 1) % size - 1, (T - 1) % size, (T - 1) % size + 1, size - 1, size, size + 1})
          if 0 < distance < T]
         + [("window", size, 700, distance, dim) for dim in (16, 64, 96) for size in (40, 64, 257)
            for distance in (1, 15, 16, size - 2, size - 1, size, size + 1, 600)])


@pytest.mark.parametrize("matrix", [False, True])
@pytest.mark.parametrize("kind, size, T, distance, dim", EDGES)
def test_a_key_counts_just_inside_a_chunk_or_window_and_not_outside(kind, size, T, distance, dim, matrix):
    """From a prompt, decoded, and from a portion cut right behind the key, on pages of 16 tokens."""
    dtype = torch.bfloat16 if matrix else torch.float32
    if kind == "chunk":
        layer = sazavik_configs.chunked(2, 1, dim, dim, size, 4, base=1e4, halves=bool(distance % 2))
        seen = (T - 1 - distance) // size == (T - 1) // size
    else:
        # slopes of the only head: 2^-8 a position, which 257 positions do not outweigh
        layer = sazavik_configs.distant(1, 1, dim, dim, size, coef=0.1, every=64)
        seen = distance < size
    layer["mixer"]["scale"] = 2.0 * dim ** -0.5
    spec, tensors, x, want, share = crafted(layer, T, distance, dtype)
    if seen:
        assert share > 0.1, f"the crafted key does not stand out: {share}"
    else:
        assert share < 1e-6, "the crafted key should not be seen"
    target = T - 1 - distance
    harness = PartHarness(spec, tensors, x.shape[1], dtype, page_size=16, capacity=T + 16)
    close(harness.run([("r", x)])[0][-1], want[-1], dtype, "whole")
    harness.cache.finish("r")
    harness.run([("r", x[:T - 1])])
    close(harness.run([("r", x[T - 1:])])[0][-1], want[-1], dtype, "decoded")
    harness.cache.finish("r")
    harness.run([("r", x[:target + 1])])
    close(harness.run([("r", x[target + 1:])])[0][-1], want[-1], dtype, "cut behind the key")


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_first_token_shares_with_its_sink_and_its_gate(dtype):
    """One token: its own key and the sink.  A head's output is its value times e^s / (e^s + e^sink), then its gate."""
    layer = sazavik_configs.chunked(3, 1, 16, 8, 7, 4)
    hidden = 24
    spec, tensors, table, stored = mixer_parts(layer, hidden, 90)
    tensors, stored = rounded(tensors, dtype), rounded(stored, dtype)
    x = rand(1, hidden, seed=5).to(dtype).float()
    row = x[0].double()
    d = {name: value.double() for name, value in stored.items()}
    unit = lambda v: v / torch.sqrt((v * v).mean() + 1e-5)
    key, value = unit(d["k"] @ row) * d["k.norm"], d["v"] @ row
    heads = []
    for head in range(3):
        query = unit((d["q"] @ row)[16 * head:16 * head + 16]) * d["q.norm"]
        share = torch.sigmoid(table["scale"] * (query @ key) - d["sink"][head])
        heads.append(share * value * torch.sigmoid((d["g"] @ row)[8 * head:8 * head + 8]))
    by_hand = (d["o"] @ torch.cat(heads)).float()
    close(plain_mixer("attention", x, table, stored)[0], by_hand, torch.float32, "the plain implementation against the closed form")
    got, = PartHarness(spec, tensors, hidden, dtype, page_size=8, capacity=64).run([("r", x)])
    close(got[0], by_hand, dtype, "the engine's")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden, experts, top, inner, shared, T", [
    (40, 6, 3, 24, 20, 33), (64, 12, 4, 80, 64, 200), (48, 3, 1, 8, None, 1), (128, 7, 5, 64, 32, 700), (56, 5, 1, 40, None, 17),
    (128, 4, 4, 32, 96, 16), (36, 1, 1, 12, 20, 65)])
def test_the_mixture_alone(dtype, hidden, experts, top, inner, shared, T):
    from macllm_infer_amd.config.sazavik import _moe
    from macllm_infer_amd.kernels import build
    from macllm_infer_amd.parts import BuildContext, part_class
    table = sazavik_configs.moe(experts, top, inner, shared)
    spec = _moe(table, "mlp")
    stored = {"router": rand(experts, hidden, seed=1) * 2.0 / hidden ** 0.5}
    for e in [f"e{n}" for n in range(experts)] + (["shared"] if shared else []):
        width = shared if e == "shared" else inner
        for i, (name, shape) in enumerate((("gate", (width, hidden)), ("up", (width, hidden)), ("down", (hidden, width)))):
            stored[f"{e}.{name}"] = rand(*shape, seed=100 + 10 * (experts if e == "shared" else int(e[1:])) + i) * 1.5 / shape[1] ** 0.5
    if shared:
        stored["shared.sg"] = rand(1, hidden, seed=7) / hidden ** 0.5
    stored = rounded(stored, dtype)
    x = rand(T, hidden, seed=3).to(dtype).float()
    margins = []
    want = sazavik_plain.mixture(x.double(), lambda name: stored[name].double(), table, margins).float()
    tensors = {f"p.{name}.weight": value for name, value in stored.items()}
    if dtype == torch.bfloat16:
        tensors = {name: value.to(torch.bfloat16) for name, value in tensors.items()}
    cls = part_class(spec)
    build.ensure_modules(cls.kernel_modules)
    part = cls(spec, "p", tensors, BuildContext(hidden_size=hidden, dtype=dtype, device=torch.device(DEV), max_context=64))
    got = part.forward(x.to(dtype).to(DEV)).float().cpu()
    clear = margins[0] > (1e-6 if dtype == torch.float32 else 0.002)           # 16-bit rounding may turn a close choice
    assert int(clear.sum()) * 4 >= 3 * T
    close(got[clear], want[clear], dtype, "tokens whose choice is clear")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("hidden, inner, limit, T", [(40, 24, 0.5, 5), (64, 37, 1.5, 100), (128, 96, 7.0, 1), (96, 64, 0.2, 16), (96, 64, 0.2, 300)])
def test_the_dense_feed_forward_alone(dtype, hidden, inner, limit, T):
    from macllm_infer_amd.config.sazavik import _dense
    from macllm_infer_amd.kernels import build
    from macllm_infer_amd.parts import BuildContext, part_class
    stored = {"gate": rand(inner, hidden, seed=1) * 2.0 / hidden ** 0.5, "up": rand(inner, hidden, seed=2) * 2.0 / hidden ** 0.5,
              "down": rand(hidden, inner, seed=3) / inner ** 0.5}
    stored = rounded(stored, dtype)
    spec = _dense({"ff": inner, "limit": limit, "kind": "dense"}, "mlp")
    x = rand(T, hidden, seed=4).to(dtype).float()
    want = sazavik_plain.clamped_feed_forward(x.double(), lambda name: stored[name].double(), limit).float()
    tensors = {f"p.{name}_proj.weight": value.to(dtype) for name, value in stored.items()}
    cls = part_class(spec)
    build.ensure_modules(cls.kernel_modules)
    part = cls(spec, "p", tensors, BuildContext(hidden_size=hidden, dtype=dtype, device=torch.device(DEV), max_context=64))
    close(part.forward(x.to(dtype).to(DEV)).float().cpu(), want, dtype)


# ------------------------------------------------------------------ whole models
def model_dir(name, folder, dtype, seed=31):
    return sazavik_configs.make_model_dir(name, folder, seed=seed, storage_dtype=torch.bfloat16 if dtype == "bfloat16" else torch.float32)


def engine_for(name, folder, dtype, capacity=512, page=8, requests=4, **more):
    from macllm_infer_amd.engine import Engine
    raw, tensors = model_dir(name, folder, dtype)
    engine = Engine(str(folder), dtype=dtype, device=DEV, kv_cache_block_tokens=page, kv_cache_capacity_tokens=capacity,
                    max_active_sequences=requests, **more)
    return engine, raw, tensors


def tokens_for(raw, count, seed):
    return torch.randint(0, raw["vocab"], (count,), generator=torch.Generator().manual_seed(seed)).tolist()


class Plain:
    """The plain model's logits of a sequence and, when asked, how far 16-bit rounding of the activations alone moves
    them at every position and by how much every position's choices are decided."""

    def __init__(self, raw, tensors, tokens):
        self.raw, self.tensors, self.tokens = raw, tensors, tokens
        self.logits = sazavik_plain.forward(raw, tensors, tokens).float()
        self._noise = self._margin = None

    @property
    def margin(self):
        if self._margin is None:
            self._margin = sazavik_plain.choice_margins(self.raw, self.tensors, self.tokens).float()
        return self._margin

    @property
    def noise(self):
        if self._noise is None:
            self._noise = sazavik_plain.rounding_noise(self.raw, self.tensors, self.tokens).float()
        return self._noise


def same(got, plain, rows, dtype, what):
    """Float32: every position within 2e-4 of the logits' scale.  Bfloat16: the gate at a position is what rounding
    alone does to the plain model there (a choice of experts that turns moves a small random model far): four times
    that, or 6 % of the scale where that is more; and the median position within 3 % of the scale or twice the plain
    model's median.  A position one of whose choices is decided by less than 0.003 is left out (a few samples of the
    rounding need not turn that choice, the engine's may); at most a third of the positions are."""
    want = plain.logits[rows]
    got = got.float().cpu()
    scale = max(1.0, float(plain.logits.abs().max()))
    if dtype == "float32":
        error = float((got - want).abs().max())
        assert error <= F32_GATE * scale, f"{what}: max error {error:.3e}"
        return
    noise = plain.noise[rows]
    error = (got - want).abs().max(dim=-1).values
    close_call = plain.margin[rows] < 0.003
    assert int(close_call.sum()) * 3 <= max(len(rows), 3), f"{what}: too many positions with close choices"
    error = torch.where(close_call, torch.zeros_like(error), error)
    gate = torch.maximum(4.0 * noise, torch.full_like(noise, 0.06 * scale))
    worst = int((error - gate).argmax())
    assert bool((error <= gate).all()), (f"{what}: row {rows[worst]} is off by {float(error[worst]):.3f} of {scale:.2f}; "
                                         f"rounding alone moves the plain model by {float(noise[worst]):.3f} there")
    if len(rows) >= 8:
        assert float(error.median()) <= max(0.03 * scale, 2.0 * float(noise.median())), \
            f"{what}: the median position is off by {float(error.median()):.3f} of {scale:.2f}"


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_the_stream_behind_every_layer(tmp_path, name, monkeypatch):
    """The residual stream after each layer in float32, against the plain model's: a fault shows in its layer."""
    engine, raw, tensors = engine_for(name, tmp_path, "float32")
    from macllm_infer_amd.engine import Lane
    from macllm_infer_amd.parts import norm as norm_module
    tokens = tokens_for(raw, 150, 5)
    behind = []
    sazavik_plain.forward(raw, tensors, tokens, streams=behind)
    seen = []
    for block in engine.model.blocks:
        original = block.forward

        def wrapped(residual, step, caches, original=original):
            original(residual, step, caches)
            norm_module.fold_pending(residual)
            seen.append(residual.h.clone())
        monkeypatch.setattr(block, "forward", wrapped)
    engine.add_request("r")
    engine.step([Lane("r", tokens, [])])
    assert len(seen) == len(behind)
    for index, (got, want) in enumerate(zip(seen, behind)):
        error = float((got.cpu().double() - want).abs().max())
        assert error <= 2e-4 * max(1.0, float(want.abs().max())), f"layer {index} ({raw['layers'][index]['type']}): {error:.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_whole_cut_decoded_and_mixed_steps_match_the_plain_model(tmp_path, name, dtype):
    from macllm_infer_amd.engine import Lane
    engine, raw, tensors = engine_for(name, tmp_path, dtype, capacity=640, page=8)
    long_tokens, short_tokens, other_tokens = tokens_for(raw, 230, 1), tokens_for(raw, 37, 2), tokens_for(raw, 95, 3)
    long_plain, short_plain, other_plain = (Plain(raw, tensors, t) for t in (long_tokens, short_tokens, other_tokens))
    engine.add_request("whole")
    got = engine.step([Lane("whole", long_tokens, list(range(230)))])
    same(got, long_plain, list(range(230)), dtype, "whole")
    engine.finish("whole")
    # in portions of many sizes, down to two tokens and one, in the slot and on the pages the first request gave back
    engine.add_request("cut")
    sizes, cursor, pieces = [9, 2, 31, 1, 1, 64, 2, 17, 3, 100], 0, []
    for size in sizes:
        pieces.append(engine.step([Lane("cut", long_tokens[cursor:cursor + size], list(range(size)))]))
        cursor += size
    same(torch.cat(pieces), long_plain, list(range(230)), dtype, "portions")
    engine.finish("cut")
    engine.add_request("decode")
    pieces = [engine.step([Lane("decode", long_tokens[:90], [89])])]
    for position in range(90, 230):
        pieces.append(engine.step([Lane("decode", long_tokens[position:position + 1], [0])]))
    same(torch.cat(pieces), long_plain, list(range(89, 230)), dtype, "decoded")
    engine.finish("decode")
    # unequal requests side by side: portions of one beside single tokens of others, one joining late, one leaving early
    for request in ("a", "b"):
        engine.add_request(request)
    rows = {"a": [], "b": [], "c": []}
    at = {"a": 0, "b": 0, "c": 0}
    feeds = {"a": long_tokens, "b": short_tokens, "c": other_tokens}
    plan = [dict(a=40, b=1), dict(a=1, b=2), dict(a=64, b=1), dict(a=2, b=30, c=7), dict(a=1, b=1, c=1), dict(a=100, b=2, c=60),
            dict(a=1, c=1), dict(a=21, c=26)]
    for turn in plan:
        if "c" in turn and at["c"] == 0:
            engine.add_request("c")
        lanes = []
        for request, count in turn.items():
            lanes.append(Lane(request, feeds[request][at[request]:at[request] + count], list(range(count))))
            at[request] += count
        got = engine.step(lanes)
        cursor = 0
        for request, count in turn.items():
            rows[request].append(got[cursor:cursor + count])
            cursor += count
        if at["b"] == len(short_tokens) and engine.has_request("b"):
            engine.finish("b")
    for request, plain in (("a", long_plain), ("b", short_plain), ("c", other_plain)):
        same(torch.cat(rows[request]), plain, list(range(at[request])), dtype, f"request {request} beside others")
    engine.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C"])
def test_long_decoding_and_the_first_tokens_beside_requests_that_come_and_go(tmp_path, name, dtype):
    """300 tokens decoded one by one through captured steps from the first token on, in a pool that holds far fewer (every
    layer's keys pass out of its window or chunk), beside requests of one and two tokens whose slot and pages are used
    again and again."""
    from macllm_infer_amd.engine import Lane
    engine, raw, tensors = engine_for(name, tmp_path, dtype, capacity=168, page=8, requests=2)
    tokens = tokens_for(raw, 300, 7)
    plain = Plain(raw, tensors, tokens)
    short = Plain(raw, tensors, tokens_for(raw, 2, 8))
    engine.add_request("r")
    pieces = [engine.step([Lane("r", tokens[:1], [0])]), engine.step([Lane("r", tokens[1:3], [0, 1])])]
    beside = []
    for position in range(3, 300):
        lanes = [Lane("r", tokens[position:position + 1], [0])]
        if position % 3 == 0:
            engine.add_request(f"s{position}")
            lanes.append(Lane(f"s{position}", short.tokens[:1], [0]))
        elif position % 3 == 1:
            lanes.append(Lane(f"s{position - 1}", short.tokens[1:], [0]))
        got = engine.step(lanes)
        pieces.append(got[:1])
        beside += [(row, position % 3) for row in got[1:]]
        if position % 3 == 1:
            engine.finish(f"s{position - 1}")
    same(torch.cat(pieces), plain, list(range(300)), dtype, "long decoding")
    for row, at in beside[:4] + beside[-4:]:
        same(row.reshape(1, -1), short, [at], dtype, "a short request in a slot used again")
    engine.cache.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_captured_steps_replay_what_launched_steps_compute(tmp_path, dtype):
    """Decode steps and portions through HIP graphs against the same steps launched kernel by kernel, several replays
    with other work between them.  A captured portion has its capacity's rows, more than were launched, and may take
    other kernels for its products: in bfloat16 such a rounding may turn a position's choice of experts, so there one
    position in twenty may differ by more."""
    from macllm_infer_amd.engine import Engine, Lane
    raw, tensors = model_dir("C", tmp_path, dtype)
    engines = [Engine(str(tmp_path), dtype=dtype, device=DEV, kv_cache_block_tokens=16, kv_cache_capacity_tokens=1024,
                      max_active_sequences=4, decode_graphs=graphs, measured_paths=False) for graphs in (True, False)]
    feeds = {f"r{i}": tokens_for(raw, 150, 40 + i) for i in range(3)}
    for engine in engines:
        for request in feeds:
            engine.add_request(request)
    at = 0
    for turn, count in enumerate([17, 17, 17, 1, 1, 1, 1, 2, 1, 1, 17, 1, 1, 40, 1, 17]):
        rows = []
        for engine in engines:
            lanes = [Lane(request, tokens[at:at + count], list(range(count))) for request, tokens in feeds.items()]
            rows.append(engine.step(lanes).float().cpu())
            torch.cuda.synchronize()
        at += count
        scale = float(rows[1].abs().max())
        difference = (rows[0] - rows[1]).abs().max(dim=-1).values
        if dtype == "float32":
            assert float(difference.max()) <= F32_GATE * scale, f"turn {turn}"
        else:
            assert int((difference > 0.02 * scale).sum()) <= max(len(difference) // 20, 1), f"turn {turn}"
            assert float(difference.median()) <= 0.01 * scale, f"turn {turn}"
    assert engines[0].graphs is not None


def replay(folder, dtype, steps, max_tokens, out):
    lines = "".join(json.dumps(step) + "\n" for step in steps)
    done = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(folder), "--dtype", dtype,
                           "--out", str(out), "--max-tokens", str(max_tokens), "--page-tokens", "16"],
                          input=lines, capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [line for line in done.stdout.splitlines() if line.startswith("done ")] == [f"done {s['step']}" for s in steps]


@pytest.mark.parametrize("name, dtype", [("A", "float32"), ("B", "bfloat16"), ("C", "float32"), ("C", "bfloat16")])
def test_replays_through_the_trace_runner_match_the_plain_model(tmp_path, name, dtype):
    raw, tensors = model_dir(name, tmp_path / "model", dtype)
    first, second, third = tokens_for(raw, 200, 1), tokens_for(raw, 70, 2), tokens_for(raw, 3, 3)
    plains = {"x": Plain(raw, tensors, first), "y": Plain(raw, tensors, second), "z": Plain(raw, tensors, third)}
    steps = [
        {"step": 0, "entries": [{"id": "x", "tokens": first[:90], "want": [0, 89]}, {"id": "z", "tokens": third[:2], "want": [1]}], "end": []},
        {"step": 1, "entries": [{"id": "x", "tokens": first[90:92], "want": [0, 1]}, {"id": "y", "tokens": second[:64], "want": [63]},
                                {"id": "z", "tokens": third[2:], "want": [0]}], "end": ["z"]},
        {"step": 2, "entries": [{"id": "y", "tokens": second[64:65], "want": []}], "end": []},
        {"step": 3, "entries": [{"id": "x", "tokens": first[92:200], "want": [107]}, {"id": "y", "tokens": second[65:], "want": [0, 4]}],
         "end": ["x", "y"]},
    ]
    wanted = {0: [("x", 0), ("x", 89), ("z", 1)], 1: [("x", 90), ("x", 91), ("y", 63), ("z", 2)], 3: [("x", 199), ("y", 65), ("y", 69)]}
    out = tmp_path / "out"
    replay(tmp_path / "model", dtype, steps, 384, out)
    assert not (out / "2.f32").exists(), "a step that wants nothing writes nothing"
    for step, rows in wanted.items():
        got = torch.from_numpy(np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(len(rows), raw["vocab"]))
        for index, (request, position) in enumerate(rows):
            same(got[index:index + 1], plains[request], [position], dtype, f"step {step} row {index}")


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_greedy_generation_through_the_entry_point(tmp_path, name):
    from macllm_infer_amd import LLM, EngineConfig, SamplingParams
    raw, tensors = model_dir(name, tmp_path, "float32")
    prompts = [tokens_for(raw, 33, 1), tokens_for(raw, 5, 2), tokens_for(raw, 61, 3)]
    llm = LLM(str(tmp_path), dtype="float32", kv_cache_block_tokens=8, kv_cache_capacity_tokens=384,
              engine_config=EngineConfig(max_active_sequences=2, scheduler_token_budget=24, prefill_token_quantum=7))
    greedy = SamplingParams(max_new_tokens=12, temperature=0.0, top_k=0, top_p=1.0, repetition_penalty=1.0)
    results = llm.generate(prompts, greedy)
    for prompt, result in zip(prompts, results):
        assert result.finish_reason == "length" and len(result.token_ids) == 12
        logits = sazavik_plain.forward(raw, tensors, prompt + result.token_ids).float()
        for index, token in enumerate(result.token_ids):
            row = logits[len(prompt) - 1 + index]
            assert row[token] >= row.max() - 1e-3 * row.abs().max(), f"token {index} is not the plain model's best"


# ------------------------------------------------------------------ configurations drawn at random
def drawn_configuration(seed):
    """A configuration whose every size, option and order of layers is drawn: heads of 4 to 128 dims (sizes of the
    matrix-core kernels beside ones they do not take), values narrower and wider than keys, chunks and windows of 1 to
    300 and none, layers that read earlier layers' keys through masks of their own, 1 to 9 experts, layers without a
    feed-forward, with and without a cap on the logits."""
    import random
    draw = random.Random(seed)
    width = draw.choice([24, 36, 40, 50, 64, 96, 128])
    layers, own = [], []
    for index in range(draw.choice([3, 4, 5, 6])):
        reads = own and draw.random() < 0.35
        if reads:
            source, kind, shared = draw.choice(own)
        else:
            kind = draw.choice(["attention", "attention_2", "attention_3"])
            groups, dim = draw.choice([1, 1, 2, 3, 5]), draw.choice([4, 8, 12, 16, 24, 40, 48, 64, 80, 96, 128])
            rot = 2 * draw.randint(1, dim // 2)
            shared = (groups, dim, draw.choice([dim, dim, 4, 20, 36, 64, 128]), rot, draw.choice([50.0, 1e4, 1e6]))
            source = None
            own.append((index, kind, shared))
        groups, dim, vdim, rot, base = shared
        heads = groups * draw.choice([1, 2, 3, 6])
        size = draw.choice([1, 2, 7, 16, 30, 33, 64, 100, 300, None])
        scale = draw.choice([None, None, 0.3])
        if kind == "attention_3":
            layer = sazavik_configs.distant(heads, groups, dim, vdim, size, draw.choice([0.5, 0.1, -0.1]), draw.choice([1, 5, 64, None]), scale, source)
        else:
            layer = sazavik_configs.chunked(heads, groups, dim, vdim, size, rot, base, kind == "attention_2", scale, source)
        which = draw.random()
        mlp = None
        if which < 0.45:
            experts = draw.choice([1, 2, 3, 5, 9])
            mlp = sazavik_configs.moe(experts, draw.randint(1, min(experts, 4)), draw.choice([8, 16, 40, 64]), draw.choice([None, 8, 32, 64]))
        elif which < 0.85:
            mlp = sazavik_configs.dense(draw.choice([20, 48, 96]), draw.choice([0.3, 1.0, 7.0]))
        layers.append(sazavik_configs.with_mlp(layer, mlp))
    raw = {"architecture": "Sazavik", "width": width, "vocab": draw.choice([31, 100, 257]), "norm": {"eps": draw.choice([1e-5, 1e-6])},
           "layers": layers}
    if draw.random() < 0.6:
        raw["logit_softcap"] = draw.choice([5.0, 30.0])
    return raw


DRAWN = [(seed, "float32") for seed in range(6100, 6116)] + [(seed, "bfloat16") for seed in range(6100, 6116, 2)]


@pytest.mark.parametrize("seed, dtype", DRAWN)
def test_randomly_drawn_configurations_whole_cut_and_side_by_side(tmp_path, seed, dtype):
    """Whole, in portions beside another request's single tokens, and decoded: float32 at every position, bfloat16 by
    the rounding gate."""
    from macllm_infer_amd.engine import Engine, Lane
    raw, tensors = sazavik_configs.make_model_dir(drawn_configuration(seed), tmp_path, seed=seed,
                                                  storage_dtype=torch.float32 if dtype == "float32" else torch.bfloat16)
    engine = Engine(str(tmp_path), dtype=dtype, device=DEV, kv_cache_block_tokens=(4, 8, 16, 32)[seed % 4],
                    kv_cache_capacity_tokens=640, max_active_sequences=3)
    tokens, other = tokens_for(raw, 150, seed), tokens_for(raw, 30, seed + 1)
    plain, beside = Plain(raw, tensors, tokens), Plain(raw, tensors, other)
    engine.add_request("whole")
    same(engine.step([Lane("whole", tokens, list(range(150)))]), plain, list(range(150)), dtype, f"seed {seed} whole")
    engine.finish("whole")
    engine.add_request("cut")
    engine.add_request("other")
    pieces, others, cursor, fed = [], [], 0, 0
    for size in (5, 2, 40, 1, 1, 23, 64, 2, 12):
        lanes = [Lane("cut", tokens[cursor:cursor + size], list(range(size)))]
        if fed < 30:
            count = 1 if fed else 4
            lanes.append(Lane("other", other[fed:fed + count], list(range(count))))
        got = engine.step(lanes)
        pieces.append(got[:size])
        if fed < 30:
            others.append(got[size:])
            fed += count
        cursor += size
    same(torch.cat(pieces), plain, list(range(150)), dtype, f"seed {seed} portions")
    same(torch.cat(others), beside, list(range(fed)), dtype, f"seed {seed} the request beside")
    engine.cache.check()
