"""Benolix without a GPU: the plain implementation against itself (whole prompts against continuation, mechanisms that
must show, hand-made cases of each), the configuration reader, the weights' names, the memory that several layers with
windows of their own read, and the engine's bookkeeping (pages, state slots, cuts, mixed batches, generation) with plain
stand-ins for the kernels."""

import copy
import math

import pytest
import torch

import benolix_tiny as bt
import plain_benolix as pb
import replay
from plain_kernels import PlainKernels
from atom_amd.cache.kinds import kind_of
from atom_amd.config import BenolixConfig, ConfigError, build_model, model_config_from_dict
from atom_amd.engine.core import StepEntry, load_model
from atom_amd.models.model import LayerRun
from atom_amd.parts.base import KVCacheNeed, LatentCacheNeed, StateNeed
from atom_amd.weights.loader import expected_tensors

LENGTHS = {"A": [1, 7, 33, 70], "B": [2, 19, 45, 64], "C": [3, 52], "D": [1, 2, 30, 41], "E": [2, 45]}
WHICH = sorted(LENGTHS)


def _requests(which, seed=0):
    return {f"r{k}": bt.ids(which, n, seed * 100 + k) for k, n in enumerate(LENGTHS[which])}


# ------------------------------------------------------------------ the plain implementation


@pytest.mark.parametrize("which", WHICH)
def test_plain_whole_equals_continuation(which):
    tokens = bt.ids(which, 57, 5)
    full = bt.oracle(which, tokens)
    model = pb.PlainBenolix(bt.CONFIGS[which], bt.tensors(which))
    rows, at = [], 0
    for cut in [9, 1, 1, 2, 13, 1, 30]:
        rows.append(model.forward(tokens[at:at + cut]))
        at += cut
    assert float((torch.cat(rows) - full).abs().max()) < 1e-9


def _other(which, path, value, tokens):
    cfg = copy.deepcopy(bt.CONFIGS[which])
    at = cfg
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    return pb.PlainBenolix(cfg, bt.tensors(which)).forward(tokens)


def test_plain_mechanisms_show():
    """Dropping or misplacing a mechanism's tensor or constant changes the logits."""
    tokens = bt.ids("A", 40, 2)
    base = bt.oracle("A", tokens)
    flip = lambda t: torch.flip(t, dims=[0])  # noqa: E731
    zero = lambda t: t * 0  # noqa: E731
    for name, change in [("l0.mix.dq.norm", flip), ("l1.mix.dq.norm", flip), ("l0.mix.dkv.norm", flip), ("l2.mix.dkv", flip),
                         ("l0.mix.uq", flip), ("l1.mix.uk", zero), ("l1.mix.uv", flip), ("l3.mix.uv", flip),
                         ("l0.mix.g", zero), ("l1.mix.g", flip), ("l0.norm1", zero), ("l0.norm2", flip), ("l2.norm1", flip),
                         ("l1.mlp.correction", zero), ("l1.mlp.router", flip), ("l1.mlp.e1.up", zero),
                         ("l3.mlp.e0.gate", zero), ("final.norm", zero)]:
        changed = dict(bt.tensors("A"))
        changed[name] = change(changed[name])
        other = pb.PlainBenolix(bt.CONFIGS["A"], changed).forward(tokens)
        assert float((other - base).abs().max()) > 1e-3 * float(base.abs().max()), name
    for path, value in [(("postln_alpha",), 1.0), (("norm", "eps"), 1e-1), (("embedding", "scale"), 1.0),
                        (("layers", 0, "mixer", "scale"), 0.1), (("layers", 0, "mixer", "rot", "base"), 10.0),
                        (("layers", 0, "mixer", "rot", "dims"), 4), (("layers", 0, "mixer", "mask", "size"), 8),
                        (("layers", 1, "mixer", "mask", "size"), 22), (("layers", 1, "mixer", "mask", "size"), 24),
                        (("layers", 3, "mixer", "mask"), None), (("layers", 1, "mlp", "expert", "limit"), 1e9),
                        (("layers", 1, "mlp", "router", "scale"), 1.0), (("layers", 1, "mlp", "router", "top"), 2)]:
        other = _other("A", path, value, tokens)
        assert float((other - base).abs().max()) > 1e-3 * float(base.abs().max()), path


@pytest.mark.parametrize("which,layer", [("A", 0), ("A", 1), ("A", 3), ("B", 0), ("B", 1), ("B", 2), ("B", 3), ("C", 0),
                                         ("C", 1), ("C", 2), ("D", 2), ("E", 0), ("E", 1), ("E", 3)])
@pytest.mark.parametrize("off", [-1, 1])
def test_plain_a_window_one_token_off_shows(which, layer, off):
    """With these weights a window that is one token off is seen, from the first position it can matter at."""
    size = bt.CONFIGS[which]["layers"][layer]["mixer"]["mask"]["size"]
    if size + off == 0:
        return
    tokens = bt.ids(which, size + 30, 9)
    base = bt.oracle(which, tokens)
    diff = (_other(which, ("layers", layer, "mixer", "mask", "size"), size + off, tokens) - base).abs().amax(-1) / base.abs().max()
    first = min(size, size + off)
    assert float(diff[:first].max()) < 1e-12
    assert float(diff[first:].max()) > 3e-3, float(diff.max())


def test_plain_window_counts_the_token_itself():
    seen = pb.window_mask(torch.arange(3, 6), torch.arange(6), 3)
    assert seen.tolist() == [[False, True, True, True, False, False], [False, False, True, True, True, False],
                             [False, False, False, True, True, True]]
    assert pb.window_mask(torch.arange(4), torch.arange(4), 1).tolist() == torch.eye(4, dtype=torch.bool).tolist()
    assert pb.window_mask(torch.arange(4), torch.arange(4), None).sum() == 10


def test_plain_rotation_turns_neighbours():
    x = torch.zeros(1, 1, 6, dtype=torch.float64)
    x[0, 0, 2] = 1.0                                     # entries 2 and 3 are a pair and turn at base^(-2/4)
    y = pb.rotate_neighbours(x, torch.tensor([10]), 4, 100.0)
    assert float(y[0, 0, 2]) == pytest.approx(math.cos(1.0)) and float(y[0, 0, 3]) == pytest.approx(math.sin(1.0))
    assert float(y[0, 0, 0]) == 0 and float(y[0, 0, 4]) == 0
    x = torch.ones(1, 6, dtype=torch.float64)
    assert pb.rotate_neighbours(x, torch.tensor([3]), 4, 100.0)[0, 4:].tolist() == [1.0, 1.0]


def test_plain_gate_is_clamped_on_one_side_and_up_on_both():
    g = torch.tensor([5.0, -5.0, 1.0], dtype=torch.float64)
    u = torch.tensor([-9.0, 9.0, 0.5], dtype=torch.float64)
    got = pb.clamped_gate(g, u, 2.0)
    want = [2 / (1 + math.exp(-3.404)) * (-2 + 1), -5 / (1 + math.exp(1.702 * 5)) * 3, 1 / (1 + math.exp(-1.702)) * 1.5]
    assert got.tolist() == pytest.approx(want)


def test_plain_router_correction_is_for_the_choice_only():
    s = torch.tensor([[0.5, 0.3, 0.15, 0.05]], dtype=torch.float64)
    chosen, w = pb.routed_choice(s, torch.tensor([0.0, -1.0, 0.0, 0.4], dtype=torch.float64), 2, 3.0)
    assert chosen.sort().values.tolist() == [[0, 3]]
    assert dict(zip(chosen[0].tolist(), w[0].tolist())) == pytest.approx({0: 3.0 * 0.5 / 0.55, 3: 3.0 * 0.05 / 0.55})


def test_plain_identity_experts_pass_the_input_on():
    h = torch.tensor([[1.0, -2.0], [0.5, 4.0]], dtype=torch.float64)
    w = {"router": torch.zeros(3, 2, dtype=torch.float64), "correction": torch.tensor([0.0, 9.0, 8.0], dtype=torch.float64),
         "e0.gate": torch.ones(1, 2, dtype=torch.float64), "e0.up": torch.ones(1, 2, dtype=torch.float64),
         "e0.down": torch.ones(2, 1, dtype=torch.float64)}
    mlp = {"expert": {"limit": 1.0}, "router": {"experts": 1, "identity": 2, "top": 2, "scale": 2.5}}
    assert torch.allclose(pb.routed_ff(h, w, mlp), 2.5 * h)


# ------------------------------------------------------------------ configuration and weights


def test_config_reads_every_size_and_round_trips():
    cfg = model_config_from_dict(bt.BENO_A)
    assert isinstance(cfg, BenolixConfig) and cfg.vocab_size == 89 and cfg.hidden_size == 44
    assert (cfg.norm_eps, cfg.postln_alpha, cfg.embedding_scale) == (3e-5, 1.4, 2.5)
    assert model_config_from_dict(cfg.to_dict()) == cfg
    model = build_model(cfg)
    assert [(r.layer, r.reads_run) for r in model.order] == [(0, None), (1, 0), (2, None), (3, 2)]
    assert model.embedding.scale == 2.5 and all(b.alpha == 1.4 for b in model.blocks) and model.final_norm.one_plus
    assert all(b.mixer_norm.one_plus and b.mixer_norm.eps == 3e-5 for b in model.blocks)
    first, second, third, fourth = (b.mixer for b in model.blocks)
    assert (first.num_heads, first.head_dim, first.rot_dim, first.value_dim, first.kv_rank, first.query_rank) == (3, 10, 6, 7, 20, 14)
    assert first.gate == "entry" and first.own_keys and first.window == 9 and not first.has_sink
    assert (first.rope.dims, first.rope.base, first.rope.scaling) == (6, 500.0, None)
    assert not second.own_keys and second.window == 23 and second.query_rank == 9
    assert third.window is None and model.blocks[2].ffn is None and fourth.window == 5
    moe = model.blocks[1].ffn
    assert (moe.num_experts, moe.identity, moe.top, moe.expert_size) == (5, 2, 3, 24)
    assert moe.weight_rule == {"renormalize": True, "score": "softmax", "eps": 1e-20, "scale": 1.7}
    assert moe.gate_options == {"limit": 1.5, "slope": 1.702, "shift": 1.0}
    assert model.blocks[3].ffn.identity == 0 and model.blocks[0].ffn.activation == "silu"


@pytest.mark.parametrize("which", WHICH)
def test_names_and_shapes_are_the_designs(which):
    model, _ = load_model(bt.folder(which), dtype=torch.float32, device="cpu")
    names = {name: tuple(shape) for name, (shape, _) in expected_tensors(model).items()}
    assert names == {k: tuple(v) for k, v in bt.shapes(which).items()}


def test_constants_left_out_take_their_obvious_values():
    raw = copy.deepcopy(bt.BENO_C)
    full = build_model(model_config_from_dict(raw))
    del raw["embedding"], raw["postln_alpha"], raw["layers"][0]["mlp"]["router"]["scale"]
    model = build_model(model_config_from_dict(raw))
    assert model.embedding.scale == full.embedding.scale == 1.0 and model.blocks[0].alpha == 1.0
    assert model.blocks[0].ffn.weight_rule == full.blocks[0].ffn.weight_rule


@pytest.mark.parametrize("path,value", [(("layers", 0, "type"), "mamba"), (("layers", 0, "mixer", "heads"), 0),
                                        (("layers", 0, "mixer", "q_rank"), None), (("layers", 0, "mixer", "rot", "dims"), 5),
                                        (("layers", 0, "mixer", "rot", "dims"), 8), (("layers", 0, "mixer", "mask", "size"), 0),
                                        (("layers", 0, "mixer", "scale"), None), (("layers", 1, "mixer", "kv_from"), 1),
                                        (("layers", 1, "mixer", "kv_from"), 3), (("layers", 3, "mixer", "kv_from"), 1),
                                        (("layers", 1, "mixer", "kv_rank"), 24), (("layers", 1, "mixer", "rot", "base"), 400.0),
                                        (("layers", 1, "mlp", "router", "top"), 8), (("layers", 1, "mlp", "router", "identity"), -1),
                                        (("layers", 1, "mlp", "expert", "limit"), 0.0), (("layers", 1, "mlp", "expert"), None),
                                        (("layers", 0, "mlp", "kind"), "sparse"), (("norm", "eps"), None)])
def test_config_refuses_what_does_not_fit(path, value):
    raw = copy.deepcopy(bt.BENO_A)
    at = raw
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    with pytest.raises(ConfigError):
        model_config_from_dict(raw)


# ------------------------------------------------------------------ memory that several runs read


def test_a_memory_is_kept_for_the_widest_window_that_reads_it():
    a = build_model(model_config_from_dict(bt.BENO_A))
    assert a.memory_needs() == [LatentCacheNeed(26, 23)] * 2 + [LatentCacheNeed(16, None)] * 2
    b = build_model(model_config_from_dict(bt.BENO_B))
    assert b.memory_needs() == [LatentCacheNeed(40, 41)] * 3 + [LatentCacheNeed(64, 33)]
    kind = kind_of(LatentCacheNeed(8))
    assert kind.joined(LatentCacheNeed(8, 5), LatentCacheNeed(8, None)).window is None
    assert kind.joined(LatentCacheNeed(8, 5), LatentCacheNeed(8, 3)).window == 5
    with pytest.raises(ValueError):
        kind.joined(LatentCacheNeed(8, 5), LatentCacheNeed(9, 5))
    kv = kind_of(KVCacheNeed(2, 4))
    assert kv.joined(KVCacheNeed(2, 4, 7), KVCacheNeed(2, 4, 9)) == KVCacheNeed(2, 4, 9)
    with pytest.raises(ValueError):
        kv.joined(KVCacheNeed(2, 4, 7, 16), KVCacheNeed(2, 4, 7, 8))
    with pytest.raises(ValueError):
        kind_of(StateNeed((3,))).joined(StateNeed((3,)), StateNeed((4,)))
    a.order = [LayerRun(0), LayerRun(2, reads_run=0)]
    with pytest.raises(ValueError, match="run 1 cannot read the cache of run 0"):
        a.memory_needs()


def test_groups_pages_and_bindings():
    core = bt.core("A", "float32", PlainKernels(), "cpu", num_pages=12, page_size=8, max_num_seqs=2)
    assert [(g.window, g.num_pages) for g in core.plan.groups] == [(23, 12), (None, 12)]
    assert core.plan.run_group == [0, 0, 1, 1]
    assert core.plan.bytes_per_page == [26 * 8 * 4, 16 * 8 * 4]        # a memory is counted once, with its owner
    owner, reader, full, full_reader = core.storage.bindings
    assert owner.writes and not reader.writes and reader.pages.data_ptr() == owner.pages.data_ptr()
    assert full_reader.pages.data_ptr() == full.pages.data_ptr() != owner.pages.data_ptr()
    assert not core.prefix_caching
    # the window group holds the pages that the wider window still sees, and gives the older ones back
    core.step([StepEntry("a", bt.ids("A", 60, 1), [])])
    table = core.manager.block_table("a", 0)
    assert [p >= 0 for p in table] == [False] * 4 + [True] * 4         # positions 38 .. 59 are seen by position 60
    assert all(p >= 0 for p in core.manager.block_table("a", 1))


def test_prefix_cache_where_nothing_is_dropped():
    """Layers without windows keep every latent: a second request takes the first one's pages over."""
    from atom_amd import LLMEngine, SamplingParams
    from atom_amd.weights.random_init import write_random_model

    raw = copy.deepcopy(bt.BENO_D)
    del raw["layers"][2]
    config = model_config_from_dict(raw)
    folder = write_random_model(f"{bt._TMP.name}/open_windows", config, seed=4, std=0.3)
    from safetensors.torch import load_file

    plain = {k: v.double() for k, v in load_file(f"{folder}/model.safetensors").items()}
    llm = LLMEngine(folder, dtype="fp32", ops=PlainKernels(), device="cpu", kv_cache_block_size=8, num_kvcache_blocks=30,
                    max_num_seqs=2, max_num_batched_tokens=32, max_model_len=96, enforce_eager=True)
    assert llm.core.prefix_caching
    prompt = bt.ids("D", 29, 3)
    for _ in range(2):
        out = llm.generate([prompt], SamplingParams(temperature=0.0, max_tokens=3, ignore_eos=True))[0]["token_ids"]
        tokens = list(prompt)
        for token in out:
            assert token == int(pb.PlainBenolix(raw, plain).forward(tokens)[-1].argmax())
            tokens.append(token)
    assert llm.core.manager.pools[0].hits == 3


# ------------------------------------------------------------------ the engine's bookkeeping


@pytest.mark.parametrize("which", WHICH)
@pytest.mark.parametrize("cut", ["whole", "tail", "portions", "mixed"])
def test_cuts_match_plain(which, cut):
    requests = _requests(which)
    oracle = {rid: bt.oracle(which, tokens) for rid, tokens in requests.items()}
    steps = getattr(replay, cut)(requests, **({"last": 9} if cut == "tail" else {}))
    pages = -(-replay.peak_tokens(steps, 8) // 8)
    core = bt.core(which, "float32", PlainKernels(), "cpu", num_pages=pages, page_size=8)
    results = replay.run_in_process(core, steps)
    replay.check(steps, results, requests, oracle, "float32", f"{which}/{cut}")
    assert not core.manager.live_requests()
    assert all(pool.num_free == pool.num_pages for pool in core.manager.pools)


def test_pages_and_slots_used_again_start_clean():
    """One slot and few pages: a request that takes over a finished one's sees nothing of it."""
    core = bt.core("B", "float32", PlainKernels(), "cpu", num_pages=10, page_size=8, max_num_seqs=1)
    first, second = bt.ids("B", 57, 1), bt.ids("B", 39, 2)
    for rid, tokens in (("x", first), ("y", second), ("z", first)):
        got = core.step([StepEntry(rid, tokens[:11], list(range(11)))])
        got = torch.cat((got, core.step([StepEntry(rid, tokens[11:], list(range(len(tokens) - 11)))])))
        core.close(rid)
        want = bt.oracle("B", tokens)
        assert float((got.double() - want).abs().max()) < 3e-5 * float(want.abs().max()), rid


def test_batches_of_unequal_requests_match_each_alone():
    core = bt.core("A", "float32", PlainKernels(), "cpu", num_pages=40, page_size=8, max_num_seqs=4)
    reqs = {"a": bt.ids("A", 50, 7), "b": bt.ids("A", 3, 8), "c": bt.ids("A", 21, 9)}
    core.step([StepEntry("a", reqs["a"][:40], []), StepEntry("c", reqs["c"][:20], [])])
    got = core.step([StepEntry("c", reqs["c"][20:], [0]), StepEntry("b", reqs["b"], [0, 1, 2]),
                     StepEntry("a", reqs["a"][40:], list(range(10)))]).double()
    want = torch.cat((bt.oracle("A", reqs["c"])[20:], bt.oracle("A", reqs["b"]), bt.oracle("A", reqs["a"])[40:]))
    assert float((got - want).abs().max()) < 3e-5 * float(want.abs().max())


@pytest.mark.parametrize("which", ["A", "D"])
def test_greedy_generation_through_the_engine(which):
    from atom_amd import LLMEngine, SamplingParams

    llm = LLMEngine(bt.folder(which), dtype="fp32", ops=PlainKernels(), device="cpu", kv_cache_block_size=8,
                    num_kvcache_blocks=40, max_num_seqs=3, max_num_batched_tokens=16, max_model_len=128,
                    enforce_eager=True)
    prompts = [bt.ids(which, n, 60 + n) for n in (1, 9, 30, 17)]
    outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=6, ignore_eos=True))
    for prompt, out in zip(prompts, outs):
        tokens = list(prompt)
        for token in out["token_ids"]:
            assert token == int(bt.oracle(which, tokens)[-1].argmax())
            tokens.append(token)
    assert all(p.num_free == p.num_pages for p in llm.core.manager.pools)
