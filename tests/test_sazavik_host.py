"""Sazavik through the engine on the CPU, the kernels replaced by their plain PyTorch references: configuration,
tensor names, cache handling, the step function and the scheduler against the plain whole-sequence implementation
(tests/sazavik_plain.py)."""
import json
import math

import pytest
import torch

import ref_ops
import sazavik_configs
import sazavik_plain
from macllm_infer_amd.cache.manager import CacheManager, KVNeed
from macllm_infer_amd.config import ConfigError, SazavikConfig, config_from_dict
from macllm_infer_amd.engine import Engine, EngineConfig, Lane, Scheduler
from macllm_infer_amd.engine.model import DecoderModel
from macllm_infer_amd.sampling import Sampler, SamplingParams


@pytest.fixture
def host_ops(monkeypatch):
    ref_ops.install(monkeypatch)


def engine_for(name, folder, capacity=256, page=8, requests=4):
    raw, tensors = sazavik_configs.make_model_dir(name, folder)
    engine = Engine(str(folder), dtype="float32", device="cpu", kv_cache_block_tokens=page,
                    kv_cache_capacity_tokens=capacity, max_active_sequences=requests, check_device=False)
    return engine, raw, tensors


def tokens_for(raw, count, seed):
    return torch.randint(0, raw["vocab"], (count,), generator=torch.Generator().manual_seed(seed)).tolist()


def plain(raw, tensors, tokens):
    return sazavik_plain.forward(raw, tensors, tokens).to(torch.float32)


def test_the_configuration_is_read_from_its_own_keys_and_round_trips():
    config = config_from_dict(sazavik_configs.SAZ_A)
    assert isinstance(config, SazavikConfig)
    spec = config.to_model_spec()
    assert spec.hidden_size == 48 and spec.vocab_size == 101 and len(spec.layers) == 4 and spec.logit_softcap == 20.0
    assert [entry.kv_from for entry in spec.schedule] == [None, None, None, 1]
    assert all(layer.arrangement == "sandwich" and layer.mixer_norm.weight_offset == 1.0 and layer.mixer_post_norm.kind == "rmsnorm"
               for layer in spec.layers) and spec.final_norm.weight_offset == 1.0 and spec.embedding_norm.weight_offset == 1.0
    first, distant, halves, reader = (layer.mixers[0].spec for layer in spec.layers)
    assert (first.num_heads, first.num_kv_heads, first.head_dim, first.value_width, first.chunk, first.window) == (6, 2, 8, 12, 21, None)
    assert first.sink and first.out_gate and not first.qkv_bias and first.position.kind == "rope_interleaved" and first.position.rotary_dim == 4
    assert halves.position.kind == "rope" and halves.chunk == 9 and not halves.sink and not halves.out_gate
    assert (distant.window, distant.chunk, distant.query_temperature, distant.position.kind) == (13, None, (0.3, 7), "linear_distance")
    assert distant.qkv_bias and distant.out_bias and distant.out_gate and not distant.sink and distant.own_rows and not reader.own_rows
    assert reader.window == 30 and reader.query_temperature == (0.8, 20)
    assert all(one.head_norm == "before_rotation" and one.head_norm_weight for one in (first, distant, halves, reader))
    assert distant.position.slopes == tuple(2.0 ** (-8.0 * h / 3) for h in (1, 2, 3))
    routed, whole, none, small = (layer.ffn for layer in spec.layers)
    assert (routed.num_experts, routed.top_k, routed.shared_size, routed.routing) == (6, 2, 20, "sigmoid_then_top")
    assert routed.input_weighted and not routed.renormalize and not routed.corrected and routed.shared_gated
    assert (whole.kind, whole.intermediate_size, whole.clamp.limit, whole.clamp.alpha, whole.clamp.up_offset) == ("swiglu", 40, 0.9, 1.702, 1.0)
    assert none is None and (small.num_experts, small.top_k, small.shared_size) == (5, 1, None)
    assert SazavikConfig.from_dict(json.loads(json.dumps(config.to_dict()))) == config
    assert config_from_dict(sazavik_configs.SAZ_B).to_model_spec().logit_softcap is None
    shapes = {spec.stored_name(expect.name): expect.shapes[0] for expect in DecoderModel.expected_tensors(spec)}
    assert {"embed", "embed.norm", "head", "final.norm", "l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l0.mix.q", "l0.mix.k",
            "l0.mix.v", "l0.mix.o", "l0.mix.g", "l0.mix.sink", "l0.mix.q.norm", "l0.mix.k.norm", "l0.mlp.router", "l0.mlp.e5.down",
            "l0.mlp.shared.sg", "l1.mix.q.b", "l1.mix.k.b", "l1.mix.v.b", "l1.mix.o.b", "l1.mix.g", "l1.mlp.gate", "l1.mlp.down",
            "l3.mix.q", "l3.mix.q.b", "l3.mix.q.norm", "l3.mix.g", "l3.mix.o.b", "l3.mlp.e4.gate"} <= set(shapes)
    assert not set(shapes) & {"l0.mix.q.b", "l0.mix.g.b", "l1.mix.g.b", "l1.mix.sink", "l2.mix.g", "l2.mix.sink", "l3.mix.k", "l3.mix.v",
                              "l3.mix.k.b", "l3.mix.v.b", "l3.mix.k.norm", "l0.mlp.correction", "l0.mlp.router.b", "l2.mlp.gate",
                              "l3.mlp.shared.up"}
    assert shapes["l0.mix.g"] == (72, 48) and shapes["l0.mix.o"] == (48, 72) and shapes["l1.mix.q.norm"] == (10,) and shapes["l0.mix.sink"] == (6,)


def broken(change):
    raw = json.loads(json.dumps(sazavik_configs.SAZ_A))
    change(raw["layers"])
    return raw


@pytest.mark.parametrize("raw, text", [
    (dict(sazavik_configs.SAZ_A, layers=[]), "layers"), (dict(sazavik_configs.SAZ_A, norm={}), "norm.eps"),
    (dict(sazavik_configs.SAZ_A, logit_softcap=-1.0), "cap on the logits"),
    (broken(lambda layers: layers[0].update(type="conv")), "type"),
    (broken(lambda layers: layers[1]["mlp"].update(kind="wide")), "mlp.kind"),
    (broken(lambda layers: layers[1]["mlp"].pop("limit")), "mlp.limit"),
    (broken(lambda layers: layers[0]["mixer"].pop("scale")), "mixer.scale"),
    (broken(lambda layers: layers[1]["mixer"]["q_temp"].update(every=0)), "q_temp.every"),
    (broken(lambda layers: layers[1]["mixer"]["q_temp"].update(every=2.5)), "q_temp.every"),
    (broken(lambda layers: layers[0]["mixer"]["rot"].update(dims=10)), "rotary_dim 10"),
    (broken(lambda layers: layers[0]["mixer"]["mask"].update(size=0)), "chunks must be positive"),
    (broken(lambda layers: layers[0]["mixer"].update(kv_heads=4)), "not a multiple"),
    (broken(lambda layers: layers[3]["mixer"].update(kv_from=3)), r"layers\[3\].mixer.kv_from.*does not run before"),
    (broken(lambda layers: layers[3]["mixer"].update(kv_from=0)), r"kv_from.*differ"),
    (broken(lambda layers: layers[3]["mixer"].update(vdim=8)), r"kv_from.*differ"),
    (broken(lambda layers: layers[0]["mlp"]["router"].update(top=7)), "7 experts of 6")])
def test_a_broken_configuration_names_its_key(raw, text):
    with pytest.raises(ConfigError, match=text):
        config_from_dict(raw)


def test_a_layer_cannot_read_from_one_that_caches_nothing():
    raw = json.loads(json.dumps(sazavik_configs.SAZ_A))
    raw["layers"].append(sazavik_configs.with_mlp(sazavik_configs.distant(2, 1, 10, 6, 5, kv_from=3), None))
    with pytest.raises(ConfigError, match="caches no keys of its own"):
        config_from_dict(raw)


def test_sizes_that_no_kernel_takes_are_refused_at_load_with_their_key():
    with pytest.raises(ConfigError, match=r"mixer.dim.*258"):
        Engine(config=broken(lambda layers: layers[0]["mixer"].update(dim=258)), tensors=None, dtype="float32", device="cpu", check_device=False)
    with pytest.raises(ConfigError, match=r"router.experts.*1025"):
        Engine(config=broken(lambda layers: layers[0]["mlp"]["router"].update(experts=1025)), tensors=None, dtype="float32", device="cpu",
               check_device=False)


def test_the_plain_mechanisms_worked_by_hand():
    seen = sazavik_plain.in_chunk(7, 3)
    assert [row.nonzero().flatten().tolist() for row in seen] == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]
    seen = sazavik_plain.in_window(5, 2)
    assert [row.nonzero().flatten().tolist() for row in seen] == [[0], [0, 1], [1, 2], [2, 3], [3, 4]]
    assert sazavik_plain.slopes(4).tolist() == [2.0 ** -2, 2.0 ** -4, 2.0 ** -6, 2.0 ** -8]
    temperature = sazavik_plain.temperature(torch.tensor([0, 2, 3, 6, 7]), 0.5, 4)
    assert torch.allclose(temperature, torch.tensor([1.0, 1.0, 1 + 0.5 * math.log(2), 1 + 0.5 * math.log(2), 1 + 0.5 * math.log(3)], dtype=torch.float64))
    # one key and a sink of its score: half the value
    out = sazavik_plain.weighted_values(torch.full((1, 1, 1), 0.7, dtype=torch.float64), torch.ones(1, 1, dtype=torch.bool),
                                        torch.full((1, 1, 2), 4.0, dtype=torch.float64), torch.tensor([0.7], dtype=torch.float64))
    assert torch.allclose(out, torch.full((1, 1, 2), 2.0, dtype=torch.float64))
    # a weight goes through the expert's activation: the output is not linear in it
    tensors = {"router": torch.zeros(1, 1), "e0.gate": torch.ones(1, 1), "e0.up": torch.ones(1, 1), "e0.down": torch.ones(1, 1)}
    mixed = sazavik_plain.mixture(torch.full((1, 1), 2.0, dtype=torch.float64), lambda name: tensors[name].double(),
                                  {"router": {"experts": 1, "top": 1}})
    assert torch.allclose(mixed, torch.tensor([[1.0 / (1.0 + math.exp(-1.0))]], dtype=torch.float64))       # silu(1) * 1


def test_pages_of_a_passed_chunk_are_given_back_at_its_end():
    needs = {(0, "chunked"): [KVNeed(1, 8, chunk=12)], (1, "window"): [KVNeed(1, 8, 12)]}
    cache = CacheManager(needs, {}, 4, 64, 1, torch.float32, "cpu")
    cache.add_request("r")
    held = []
    for _ in range(30):
        cache.reserve([("r", 1)])
        cache.commit("r", 1)
        held.append(tuple(len(cache.table(group, "r").live_pages()) for group in (0, 1)))
    # at a multiple of 12 the next query's chunk holds nothing yet; before that every page since the chunk's start
    assert [pages for pages, _ in held[8:14]] == [3, 3, 3, 0, 1, 1] and held[23][0] == 0 and held[28][0] == 2
    assert all(window >= 3 for _, window in held[11:])
    cache.finish("r")
    cache.check()


@pytest.mark.parametrize("source, reader, kept", [
    (dict(window=6), dict(window=9), dict(window=9)), (dict(window=9), dict(window=6), dict(window=9)),
    (dict(window=6), dict(), dict()), (dict(), dict(window=6), dict()), (dict(chunk=8), dict(chunk=8), dict(chunk=8)),
    (dict(chunk=8), dict(chunk=12), dict(window=12)), (dict(chunk=8), dict(window=5), dict(window=8)),
    (dict(window=6, keep_first=3), dict(window=4), dict(window=6, keep_first=3))])
def test_rows_that_others_read_stay_as_long_as_any_of_them_sees_them(source, reader, kept):
    cache = CacheManager({0: [KVNeed(1, 8, **source)], 1: [KVNeed(1, 8, **reader)]}, {1: 0}, 4, 64, 1, torch.float32, "cpu")
    assert len(cache.groups) == 1 and cache.groups[0].need == KVNeed(1, 8, **kept)
    assert not cache.entry(1).owns_kv and cache.entry(1).k_cache.data_ptr() == cache.entry(0).k_cache.data_ptr()


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_whole_cut_and_token_by_token_match_the_plain_model(host_ops, tmp_path, name):
    engine, raw, tensors = engine_for(name, tmp_path)
    tokens = tokens_for(raw, 61, 3)
    expected = plain(raw, tensors, tokens)
    engine.add_request("whole")
    got = engine.step([Lane("whole", tokens, list(range(len(tokens))))])
    assert torch.allclose(got, expected, atol=2e-4, rtol=1e-4)
    engine.add_request("cut")
    rows, at = [], 0
    for size in (2, 7, 1, 1, 9, 2, 19, 1, 1, 1, 17):          # portions down to two tokens, single tokens between
        rows.append(engine.step([Lane("cut", tokens[at:at + size], list(range(size)))]))
        at += size
    assert at == len(tokens)
    assert torch.allclose(torch.cat(rows), expected, atol=2e-4, rtol=1e-4)
    engine.finish("whole")
    engine.finish("cut")
    engine.cache.check()


def test_layers_that_read_another_s_keys_have_no_pages_of_their_own(host_ops, tmp_path):
    engine, raw, _ = engine_for("B", tmp_path)
    needs = sorted((group.need.head_dim, group.need.window or 0, group.need.chunk or 0, len(group.members)) for group in engine.cache.groups)
    assert needs == [(7, 0, 0, 1), (16, 64, 0, 1), (20, 0, 5, 1)]      # the window's rows stay for the reader that has none
    reader, source = engine.cache.entry((2, "mix")), engine.cache.entry((0, "mix"))
    assert not reader.owns_kv and source.owns_kv and reader.k_cache.data_ptr() == source.k_cache.data_ptr()
    assert engine.config.kv_bytes_per_token(2) == 2 * (5 * 16 + 32 + 3 * 24) and engine.config.fixed_state_bytes(2) == 0


def test_unequal_requests_in_one_batch_and_reused_slots_and_pages(host_ops, tmp_path):
    engine, raw, tensors = engine_for("A", tmp_path, capacity=96, page=8, requests=3)
    prompts = {name: tokens_for(raw, count, seed) for name, count, seed in (("a", 21, 1), ("b", 5, 2), ("c", 33, 3))}
    expected = {name: plain(raw, tensors, tokens) for name, tokens in prompts.items()}
    for turn in range(2):                                      # the second turn takes the slots and pages of the first
        for name in prompts:
            engine.add_request(name)
        at = {name: 0 for name in prompts}
        got = {name: [] for name in prompts}
        sizes = {"a": [4, 1, 1, 15], "b": [1, 1, 1, 2], "c": [16, 9, 7, 1]}
        for step in range(4):
            lanes = [Lane(name, prompts[name][at[name]:at[name] + sizes[name][step]], list(range(sizes[name][step])))
                     for name in prompts]
            rows = engine.step(lanes)
            first = 0
            for name in prompts:
                size = sizes[name][step]
                got[name].append(rows[first:first + size])
                first += size
                at[name] += size
        for name in prompts:
            assert torch.allclose(torch.cat(got[name]), expected[name], atol=2e-4, rtol=1e-4), (turn, name)
            engine.finish(name)
        engine.cache.check()


@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_through_the_scheduler(host_ops, tmp_path, name):
    engine, raw, tensors = engine_for(name, tmp_path, capacity=256, page=8, requests=3)
    sampler = Sampler(engine.vocab_size, "cpu", check_device=False)
    scheduler = Scheduler(engine, sampler, EngineConfig(max_active_sequences=3, scheduler_token_budget=24,
                                                        prefill_token_quantum=7))
    prompts = [tokens_for(raw, 19, 1), tokens_for(raw, 3, 2), tokens_for(raw, 8, 3), tokens_for(raw, 1, 4)]
    greedy = SamplingParams(max_new_tokens=5, temperature=0.0, top_k=0, top_p=1.0, repetition_penalty=1.0)
    for index, prompt in enumerate(prompts):
        scheduler.submit(index, prompt, greedy)
    finished = scheduler.run()
    for index, prompt in enumerate(prompts):
        tokens = list(prompt)
        for _ in range(5):
            tokens.append(int(plain(raw, tensors, tokens)[-1].argmax()))
        assert finished[index].generated == tokens[len(prompt):], index
    stats = engine.cache.stats()
    assert stats["live_requests"] == 0 and stats["free_slots"] == 3


def test_random_weights_of_the_design_load_back(tmp_path):
    from macllm_infer_amd.weights.random_init import write_random_model
    write_random_model(sazavik_configs.config_of("B"), 5, str(tmp_path))
    engine = Engine(str(tmp_path), dtype="bfloat16", device="cpu", kv_cache_capacity_tokens=64, check_device=False)
    assert engine.model.embedding_norm is not None and engine.model.blocks[2].mixers[0][1].qkv.out_features == 10 * 7 + 10 * 9
