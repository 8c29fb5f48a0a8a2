"""Benolix on the GPU: the kernels' new forms alone against the plain implementation's function of the same mechanism
(float32 and bfloat16), a key that stands out just inside and just outside a window in every form of the attention
kernels, then the engine on tiny models: whole prompts, token-by-token tails, portions down to two tokens, mixed batches
with pages and slots used again, decode steps replayed from graphs, long decoding past every window, greedy generation
through ``LLMEngine``, and ``bin/trace_run``."""

import pytest
import torch

import benolix_tiny as bt
import plain_benolix as pb
import replay
from helpers import gpu_ops
from atom_amd.engine.core import StepEntry
from atom_amd.kernels.hip import AttentionMeta, KernelError, QueryTurn

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]
TOL = {torch.float32: 2e-5, torch.bfloat16: 2e-2}


def rnd(shape, seed, scale=1.0):
    return torch.randn(shape, generator=torch.Generator().manual_seed(seed)) * scale


def close(got, want, dtype, what=""):
    got, want = got.double().cpu(), want.double()
    scale = max(1e-6, float(want.abs().max()))
    err = float((got - want).abs().max())
    assert err <= TOL[dtype] * scale, f"{what}: {err:.3e} > {TOL[dtype] * scale:.3e}"


def i32(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


def frequencies(dims, base):
    return (base ** (-2 * torch.arange(dims // 2, dtype=torch.float64) / dims)).to(DEV)


# ------------------------------------------------------------------ latents: norms, rotation, per-head products


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("cq,rank,rot,dims", [(14, 20, 6, 4), (64, 128, 32, 32), (300, 40, 8, 8), (5, 16, 2, 0)])
def test_query_latent_and_key_rows(dtype, cq, rank, rot, dims):
    """Both norms and the keys' rotation in one launch; the query latent alone (a layer that reads another's rows);
    the keys alone (a layer whose queries have no latent)."""
    ops = gpu_ops()
    T, pre, eps = 9, 3, 3e-5
    proj = rnd((T, pre + cq + rank + rot + 5), 1)
    positions = torch.tensor([0, 1, 2, 700, 701, 40000, 15, 16, 17])
    slots = torch.tensor([4, 5, 6, -1, 0, 1, 2, 3, 11])
    wq, wk = 1 + rnd((cq,), 2, 0.2), 1 + rnd((rank,), 3, 0.2)
    p = proj.double()
    want_q = pb.rms(p[:, pre:pre + cq], eps) * wq.double()
    off = pre + cq
    keys = torch.cat((pb.rms(p[:, off:off + rank], eps) * wk.double(),
                      pb.rotate_neighbours(p[:, off + rank:off + rank + rot], positions, dims, 777.0)), 1)
    want = torch.zeros((12, rank + rot), dtype=torch.float64)
    for t in range(T):
        if slots[t] >= 0:
            want[slots[t]] = keys[t]
    turns = ops.rotation_table(positions.int().to(DEV), frequencies(dims, 777.0)) if dims else None
    dev, dslots = proj.to(DEV), slots.int().to(DEV)
    for with_query, with_keys in ((True, True), (True, False), (False, True)):
        out = torch.zeros((T, cq), dtype=dtype, device=DEV)
        pages = torch.zeros((3, 4, rank + rot), dtype=dtype, device=DEV)
        ops.latent_prepare(dev, pages, dslots if with_keys else None, off, rank, rot, wk.to(DEV) if with_keys else None, eps,
                           turns, (pre, wq.to(DEV), out) if with_query else None)
        close(out, want_q if with_query else 0 * want_q, dtype, "query latent")
        close(pages.view(12, -1), want if with_keys else 0 * want, dtype, "pages")
    with pytest.raises(KernelError):
        ops.latent_prepare(dev, pages, dslots, proj.shape[1] - 3, rank, rot, wk.to(DEV), eps, turns)
    if dims:
        with pytest.raises(KernelError):
            ops.latent_prepare(dev, pages, dslots, off, rank, dims - 2, wk.to(DEV), eps, turns)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("x_dtype", DTYPES)
@pytest.mark.parametrize("H,m,n,k", [(3, 70, 21, 16), (2, 200, 100, 40), (5, 33, 64, 128), (3, 5, 24, 32), (4, 9, 7, 13),
                                     (2, 3, 5, 13), (2, 130, 128, 512), (16, 8, 128, 512), (1, 1, 1, 1),
                                     (3, 97, 132, 40), (2, 300, 256, 72), (1, 128, 20, 8), (2, 200, 130, 96)])
def test_per_head_products_with_a_gate_per_entry(dtype, x_dtype, H, m, n, k):
    """Every kernel of the per-head product (few rows, tiles, matrix cores) with one gate value per output entry."""
    ops = gpu_ops()
    ldx, hsx, ldy, hsy = H * (k + 8) + 16, k + 8, H * (n + 3) + 1, n + 3
    x = rnd((m, ldx), 1).to(x_dtype)
    w = rnd((H, n, k), 2, k ** -0.5).to(dtype)
    y = torch.full((m, ldy), 3.0, dtype=dtype, device=DEV)
    gate = rnd((m, H * n + 7), 3, 2.0)
    ops.heads_gemm(x.to(DEV), 8, ldx, hsx, w.to(DEV), y, 1, ldy, hsy, H, m, n, k, alpha=0.7, gate=gate.to(DEV),
                   gate_offset=5, ldg=H * n + 7, gate_entries=True)
    tol = torch.bfloat16 if torch.bfloat16 in (dtype, x_dtype) else dtype
    for h in range(H):
        want = 0.7 * x.double()[:, 8 + h * hsx:8 + h * hsx + k] @ w.double()[h].T * pb.sigmoid(gate.double()[:, 5 + h * n:5 + h * n + n])
        close(y[:, 1 + h * hsy:1 + h * hsy + n], want, tol, f"head {h}")
        assert float((y[:, 1 + h * hsy + n:1 + (h + 1) * hsy].float() - 3).abs().max()) == 0
    with pytest.raises(KernelError):
        ops.heads_gemm(x.to(DEV), 8, ldx, hsx, w.to(DEV), y, 1, ldy, hsy, H, m, n, k, gate=gate.to(DEV), gate_offset=8,
                       ldg=H * n + 7, gate_entries=True)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,m,d,rot,dims,rank", [(3, 70, 8, 6, 4, 24), (16, 5, 128, 64, 64, 512), (5, 200, 16, 16, 16, 40),
                                                 (2, 9, 13, 5, 2, 11), (4, 3, 7, 3, 0, 20), (3, 65, 32, 8, 8, 64),
                                                        (4, 150, 24, 8, 8, 200), (2, 257, 128, 64, 64, 512)])
def test_absorbing_product_turns_the_rotated_parts(dtype, H, m, d, rot, dims, rank):
    ops = gpu_ops()
    width, ld = rank + rot, H * (d + rot)
    q = rnd((m, ld), 1)
    up = rnd((H, rank, d), 2, d ** -0.5).to(dtype)
    positions = torch.randint(0, 60000, (m,), generator=torch.Generator().manual_seed(3))
    out = torch.zeros((m, H, width), dtype=dtype, device=DEV)
    turns = ops.rotation_table(positions.int().to(DEV), frequencies(dims, 5e5)) if dims else None
    ops.heads_gemm(q.to(DEV), 0, ld, d + rot, up.to(DEV), out, 0, H * width, width, H, m, rank, d, alpha=0.3,
                   turn=QueryTurn(d, rank, rot, turns, 0.3))
    heads = q.double().view(m, H, d + rot)
    close(out[..., :rank], torch.stack([heads[:, h, :d] @ up[h].double().T for h in range(H)], 1) * 0.3, dtype, "absorbed")
    close(out[..., rank:], pb.rotate_neighbours(heads[..., d:], positions, dims, 5e5) * 0.3, dtype, "turned")


# ------------------------------------------------------------------ attention over latents: windows


def _attend(q_abs, rows, rank, pos, window):
    """One query position against the plain mask: [heads, rank]."""
    seen = pb.window_mask(torch.tensor([pos]), torch.arange(rows.shape[0]), window)[0]
    return torch.softmax(q_abs @ rows[seen].T, dim=-1) @ rows[seen][:, :rank]


SIZES = [(32, 8, 3, 16), (64, 16, 16, 8), (20, 6, 5, 4), (128, 64, 20, 16), (256, 64, 8, 16), (512, 64, 16, 16), (48, 8, 70, 4),
         (32, 16, 2, 5), (160, 32, 33, 32), (512, 64, 3, 7), (512, 64, 32, 16), (128, 64, 70, 4), (256, 64, 40, 8), (128, 64, 16, 16)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank,rot,heads,page", SIZES)
@pytest.mark.parametrize("window", [1, 2, 31, 33, 64, 150, 257])
def test_attention_keys_just_inside_and_just_outside_the_window(dtype, rank, rot, heads, page, window):
    """Requests whose queries look for one key that stands out: the oldest one their window holds, and the one before
    it.  Portions of several tokens and single tokens (a row's keys on one block or over several); requests at the
    start of a sequence, around page borders and far into it; given-back pages hold another request's rows."""
    ops = gpu_ops()
    n, width = 420, rank + rot
    hot = torch.zeros(width)
    hot[:8] = 3.0                                        # a row that scores about 20 above the others
    # (positions of the request's tokens in this step, position of the row that stands out or None)
    groups = [([0], 0), ([0, 1, 2], 0), ([page - 1, page, page + 1], 0)]
    for last in (window - 1, window, window + 1, 300, n - 1):
        if 2 <= last < n:
            for stands in (last - window + 1, last - window):
                if stands >= 0:
                    groups.append((list(range(max(0, last - 3), last + 1)), stands))
                    groups.append(([last], stands))
    rows, tables, want, q_all, token_seq, positions, starts, contexts = [], [], [], [], [], [], [0], []
    num_pages = sum(-(-(g[0][-1] + 1) // page) for g in groups) + 1
    order = (torch.randperm(num_pages - 1, generator=torch.Generator().manual_seed(4)) + 1).tolist()
    pages = torch.zeros((num_pages, page, width), dtype=dtype)
    pages[0] = hot.to(dtype)                             # what a table's empty places (0) would read
    most = -(-n // page)
    groups.sort(key=lambda g: len(g[0]) == 1)            # portions come first on the token axis
    for b, (at, stands) in enumerate(groups):
        ctx = at[-1] + 1
        mine = rnd((ctx, width), 20 + b, 0.3)
        mine[:, :8] = 0.0
        mine[stands] = 0.2 * mine[stands] + hot
        mine = mine.to(dtype)
        table = torch.zeros(most, dtype=torch.int32)
        first_seen = max(0, at[0] - window + 1)
        for j in range(ctx):
            if j // page >= first_seen // page:          # pages wholly behind the window have been given back
                if table[j // page] == 0:
                    table[j // page] = order.pop()
                pages[table[j // page], j % page] = mine[j]
        tables.append(table)
        q = rnd((len(at), heads, width), 200 + b, 0.3)
        q[..., :8] = 0.9
        q = q.to(dtype)
        for i, pos in enumerate(at):
            want.append(_attend(q[i].double(), mine[:pos + 1].double(), rank, pos, window))
        q_all.append(q)
        token_seq += [b] * len(at)
        positions += at
        starts.append(starts[-1] + len(at))
        contexts.append(ctx)
    want = torch.stack(want)
    q_all = torch.cat(q_all)
    portions = sum(len(g[0]) > 1 for g in groups)

    def run(lo, hi, parts):
        t0, t1 = starts[lo], starts[hi]
        meta = AttentionMeta(token_seq=i32([s - lo for s in token_seq[t0:t1]]), positions=i32(positions[t0:t1]),
                             block_tables=torch.stack(tables[lo:hi]).to(DEV), cu_seqlens_q=i32([s - t0 for s in starts[lo:hi + 1]]),
                             context_lens=i32(contexts[lo:hi]), num_seqs=hi - lo, num_tokens=t1 - t0,
                             max_q_len=max(len(g[0]) for g in groups[lo:hi]), max_context_len=max(contexts[lo:hi]),
                             page_size=page, num_prefill=max(0, portions - lo))
        out = torch.full((t1 - t0, heads, rank), 7.0, dtype=dtype, device=DEV)
        ops.latent_attention(q_all[t0:t1].to(DEV), pages.to(DEV), out, meta, rank, None, window, parts=parts)
        close(out, want[t0:t1], dtype, f"requests {lo}..{hi} parts {parts}")

    run(0, len(groups), None)                            # portions beside single tokens
    for parts in (None, 1, 3):
        run(portions, len(groups), parts)                # single tokens alone
    # the row that stands out decides where it is seen: its first entries are the result's
    for b, (at, stands) in enumerate(groups):
        last = starts[b + 1] - 1
        seen = at[-1] - stands < window
        assert (float(want[last, 0, 0]) > 1.5) == seen


# ------------------------------------------------------------------ routers and experts


@pytest.mark.parametrize("outputs,top", [(7, 3), (5, 1), (20, 2), (80, 6), (4, 4), (530, 3), (100, 66)])
@pytest.mark.parametrize("scale", [1.0, 2.7])
def test_router_softmax_scores(outputs, top, scale):
    """Softmax over all outputs, the correction for the choice only, weights over their sum, scaled; more outputs than a
    wave holds and more choices than it has lanes take the general kernel.  Large logits do not overflow."""
    ops = gpu_ops()
    logits = rnd((60, outputs), 1, 2.0)
    logits[7] += 300.0
    logits[8] -= 300.0
    correction = rnd((outputs,), 2, 0.1)
    z = logits.double()
    e = torch.exp(z - z.amax(-1, keepdim=True))
    scores = e / e.sum(-1, keepdim=True)
    sure = pb.routed_margin(scores, correction.double(), top) > 1e-6
    ids, weights = pb.routed_choice(scores, correction.double(), top, scale)
    got_ids, got_w = ops.router_choose(logits.to(DEV), correction.to(DEV), top, renormalize=True, score="softmax", eps=1e-20,
                                       scale=scale)
    order = got_ids.cpu().long()
    assert torch.equal(order.sort(-1).values[sure], ids.sort(-1).values[sure]) and int(sure.sum()) > 30
    by_id = torch.zeros_like(scores).scatter(1, ids, weights)
    close(got_w[sure.to(DEV)], by_id.gather(1, order)[sure], torch.float32, "weights")
    if top < outputs:
        plain, _ = pb.routed_choice(scores, 0 * correction.double(), top, scale)
        assert not torch.equal(plain.sort(-1).values, ids.sort(-1).values), "the correction must matter here"
    _, bare = ops.router_choose(logits.to(DEV), None, top, score="softmax")
    close(bare.sum(-1), torch.gather(scores, 1, torch.topk(scores, top).indices).sum(-1), torch.float32, "not renormalised")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff,experts,identity,top,tokens", [
    (48, 40, 5, 2, 2, 13), (40, 16, 6, 0, 3, 1), (64, 32, 8, 8, 1, 70), (48, 40, 2, 5, 4, 300), (136, 72, 33, 7, 4, 129),
    (44, 18, 5, 2, 3, 50), (264, 88, 10, 3, 2, 64), (32, 24, 1, 1, 2, 8), (56, 36, 3, 1, 2, 90),
    (128, 64, 3, 1, 2, 300), (192, 128, 5, 0, 3, 250), (64, 192, 2, 1, 2, 515), (320, 64, 9, 3, 4, 161)])
def test_experts_with_clamped_gates_and_identities(dtype, width, ff, experts, identity, top, tokens):
    """Few and many (token, choice) pairs, sizes the grouped products take and not; gate and up rows reach the clamp;
    some tokens have identity experts only, some none."""
    ops = gpu_ops()
    limit, scale = 1.25, 1.9
    x = rnd((tokens, width), 1).to(dtype)
    w = {"router": rnd((experts + identity, width), 2, 0.3).to(dtype), "correction": rnd((experts + identity,), 3, 0.1)}
    for e in range(experts):
        w[f"e{e}.gate"], w[f"e{e}.up"] = (rnd((ff, width), s + e, 2 * width ** -0.5).to(dtype) for s in (10, 130))
        w[f"e{e}.down"] = rnd((width, ff), 250 + e, ff ** -0.5).to(dtype)
    wd = {k: v.double() for k, v in w.items()}
    scores = pb.router_scores(x.double(), wd)
    chosen, weights = pb.routed_choice(scores, wd["correction"], top, scale)
    if identity:
        only = chosen >= experts
        assert bool(only.any())
    want = pb.routed_ff(x.double(), wd, {"expert": {"limit": limit}, "router": {"experts": experts, "identity": identity,
                                                                                  "top": top, "scale": scale}})
    both = x.double() @ wd["e0.up"].T
    assert float((both.abs() > limit).double().mean()) > 0.2, "the clamp must matter here"
    gate_up = torch.stack([torch.cat((w[f"e{e}.gate"], w[f"e{e}.up"])) for e in range(experts)]).to(DEV)
    down = torch.stack([w[f"e{e}.down"] for e in range(experts)]).to(DEV)
    got = ops.experts_forward(x.to(DEV), gate_up, down, chosen.int().to(DEV), weights.float().to(DEV), "silu", limit=limit,
                              slope=1.702, shift=1.0)
    close(got, want, dtype)
    with pytest.raises(KernelError):
        ops.experts_forward(x.to(DEV), gate_up, down, chosen.int().to(DEV), weights.float().to(DEV), "relu", limit=limit)


# ------------------------------------------------------------------ the engine

LENGTHS = {"A": [1, 7, 33, 150, 64, 300], "B": [2, 19, 45, 260, 128], "C": [3, 40, 17, 200, 140], "D": [1, 2, 40, 130, 33], "E": [2, 33, 310, 200, 17]}
WHICH = sorted(LENGTHS)
# float32: every position, against the largest logit of its request.  bfloat16: an expert chosen by a hair may be
# another one after rounding, which changes that token and, through its cached latents, later ones a little; so tokens
# whose router margin is small are left to the float32 run and nearly all of the rest must be within rounding.
F32_TOL = dict(max=5e-5, mean=1e-5)
BF16_TOL = dict(max=6e-2, mean=1e-2, over=0.08, median=6e-3)
CLOSE_CALL = 0.01


def _requests(which, seed=0):
    return {f"r{k}": bt.ids(which, n, seed * 100 + k) for k, n in enumerate(LENGTHS[which])}


def _check(steps, results, requests, which, dtype, what):
    rows = replay.collect(steps, results)
    errors, over = [], []
    for rid, tokens in requests.items():
        want, margin = bt.oracle(which, tokens), bt.router_margin(which, tokens)
        scale = float(want.abs().max())
        assert len(rows[rid]) == len(tokens)
        for pos, got in sorted(rows[rid].items()):
            assert torch.isfinite(got).all(), f"{what} request {rid} position {pos}: not finite"
            diff = (got.double() - want[pos]).abs()
            worst, mean = float(diff.max()) / scale, float(diff.mean()) / scale
            if dtype == "float32":
                if float(margin[pos]) > 1e-6:
                    assert worst <= F32_TOL["max"] and mean <= F32_TOL["mean"], \
                        f"{what} request {rid} position {pos}: max {worst:.3e} mean {mean:.3e} of the largest logit"
                continue
            if float(margin[pos]) < CLOSE_CALL:
                continue
            errors.append(mean)
            if worst > BF16_TOL["max"] or mean > BF16_TOL["mean"]:
                over.append((rid, pos, worst, mean))
    if dtype == "bfloat16":
        assert len(errors) >= 0.3 * sum(len(t) for t in requests.values()), "too few tokens are judged"
        assert len(over) <= max(1, BF16_TOL["over"] * len(errors)), f"{what}: {len(over)} of {len(errors)} over: {over[:5]}"
        assert sorted(errors)[len(errors) // 2] <= BF16_TOL["median"], f"{what}: typical error {sorted(errors)[len(errors) // 2]:.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", WHICH)
@pytest.mark.parametrize("cut", ["whole", "tail", "portions", "mixed"])
def test_cuts_match_plain(which, cut, dtype):
    requests = _requests(which)
    steps = getattr(replay, cut)(requests)
    pages = -(-replay.peak_tokens(steps, 16) // 16)
    core = bt.core(which, dtype, gpu_ops(), DEV, num_pages=pages, page_size=16, graph_sizes=[1, 2, 4] if cut != "whole" else None)
    results = replay.run_in_process(core, steps)
    _check(steps, results, requests, which, dtype, f"{which}/{cut}/{dtype}")
    assert all(pool.num_free == pool.num_pages for pool in core.manager.pools)
    if cut == "tail":
        assert core.graphs is not None and core.graphs.replays >= 32, "single tokens replay captured graphs"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("which", ["A", "C", "E"])
def test_small_pages_slots_used_again_and_long_decoding(which, dtype):
    """Pages of 4 tokens, two state slots for five requests, and 200 tokens decoded one by one past every window, each of
    them compared."""
    requests = {"long": bt.ids(which, 330, 1), "b": bt.ids(which, 23, 2), "c": bt.ids(which, 50, 3), "d": bt.ids(which, 9, 4),
                "e": bt.ids(which, 31, 5)}
    steps = replay.mixed(requests, seed=6, max_live=2, decode_tail=200)
    pages = -(-replay.peak_tokens(steps, 4) // 4)
    core = bt.core(which, dtype, gpu_ops(), DEV, num_pages=pages, page_size=4, max_num_seqs=2, graph_sizes=[1, 2])
    results = replay.run_in_process(core, steps)
    _check(steps, results, requests, which, dtype, f"{which}/page4/{dtype}")


@pytest.mark.parametrize("which", ["A", "B", "E"])
def test_logits_do_not_depend_on_the_batch_or_the_cut(which):
    """float32: a request's logits alone, cut in portions, and beside others differ by rounding of sums only."""
    requests = _requests(which)
    runs = []
    for cut in ("whole", "portions", "mixed"):
        steps = getattr(replay, cut)(requests)
        core = bt.core(which, "float32", gpu_ops(), DEV, num_pages=80, page_size=16)
        runs.append(replay.collect(steps, replay.run_in_process(core, steps)))
    for rid in requests:
        for pos in runs[0][rid]:
            for other in runs[1:]:
                assert float((runs[0][rid][pos] - other[rid][pos]).abs().max()) <= 2e-5 * float(runs[0][rid][pos].abs().max())


@pytest.mark.parametrize("which", WHICH)
def test_stream_after_every_layer(which):
    """float32: the stream after each layer against the plain implementation's, so that a fault shows at the layer
    that makes it."""
    tokens = bt.ids(which, 75, 8)
    trail = []
    pb.PlainBenolix(bt.CONFIGS[which], bt.tensors(which)).forward(tokens, trail)
    core = bt.core(which, "float32", gpu_ops(), DEV, num_pages=8, page_size=16)
    got = []
    blocks = core.model.blocks

    def watch(inner):
        def forward(ctx, hidden, residual, cache):
            out = inner(ctx, hidden, residual, cache)
            got.append(out[0].clone().cpu())
            return out
        return forward

    for b in blocks:
        b.forward = watch(b.forward)
    core.step([StepEntry("a", tokens, [len(tokens) - 1])])
    assert len(got) == len(trail)
    for layer, (mine, want) in enumerate(zip(got, trail)):
        close(mine, want, torch.float32, f"after layer {layer}")


@pytest.mark.parametrize("which,dtype", [("A", "fp32"), ("B", "fp32"), ("C", "fp32"), ("D", "fp32"), ("B", "bf16"), ("E", "bf16")])
def test_greedy_generation_through_the_engine(which, dtype):
    from atom_amd import LLMEngine, SamplingParams

    llm = LLMEngine(bt.folder(which), dtype=dtype, ops=gpu_ops(), kv_cache_block_size=16, num_kvcache_blocks=64,
                    max_num_seqs=4, max_num_batched_tokens=64, max_model_len=384)
    prompts = [bt.ids(which, n, 70 + n) for n in (1, 9, 40, 130, 65)]
    outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10, ignore_eos=True))
    for prompt, out in zip(prompts, outs):
        tokens = list(prompt)
        assert len(out["token_ids"]) == 10
        for token in out["token_ids"]:
            logits = bt.oracle(which, tokens)[-1]
            best = int(logits.argmax())
            slack = 0.0 if dtype == "fp32" else 0.06 * float(logits.abs().max())
            sure = dtype == "fp32" or float(bt.router_margin(which, tokens)[-1]) >= CLOSE_CALL
            assert token == best or float(logits[best] - logits[token]) <= slack or not sure
            tokens.append(token)
    assert all(p.num_free == p.num_pages for p in llm.core.manager.pools)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_program(dtype, tmp_path):
    requests = {k: v for k, v in list(_requests("B").items())[:4]}
    steps = replay.mixed(requests, seed=2, max_live=3)
    results = replay.run_program(bt.folder("B"), dtype, steps, str(tmp_path / "out"), replay.peak_tokens(steps, 64),
                                 bt.CONFIGS["B"]["vocab"])
    _check(steps, results, requests, "B", dtype, f"program/{dtype}")


def test_command_line():
    """``python -m atom_amd.examples.simple_inference`` on a Benolix folder: the registry picks the design from
    config.json; greedy completions are the plain implementation's."""
    import random
    import re
    import subprocess
    import sys

    cmd = [sys.executable, "-m", "atom_amd.examples.simple_inference", "--model", bt.folder("A"), "--temperature", "0",
           "--max-tokens", "6", "--block_size", "16", "--num-kvcache-blocks", "32", "--max-num-seqs", "4", "--dtype", "fp32",
           "--max-model-len", "256", "--seed", "3"]
    res = subprocess.run(cmd, cwd=replay.ROOT, capture_output=True, text=True, timeout=300)
    assert res.returncode == 0, res.stderr[-2000:]
    assert res.stdout.count("Completion:") == 3 and res.stdout.count("finish_reason=max_tokens") == 3
    rng = random.Random(3)
    prompts = [[rng.randrange(bt.CONFIGS["A"]["vocab"]) for _ in range(n)] for n in (5, 17, 33)]
    shown = [eval(m) for m in re.findall(r"Completion: (\[.*?\])", res.stdout)]
    for prompt, out in zip(prompts, shown):
        tokens = list(prompt)
        for token in out:
            assert token == int(bt.oracle("A", tokens)[-1].argmax())
            tokens.append(token)
