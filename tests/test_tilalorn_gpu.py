"""The Tilalorn design on the GPU through the framework's step function, cache manager, scheduler and entry point, against the plain
implementation: every way of cutting requests in both dtypes, the residual after every layer, long decoding from the first token over many
windows, slots and pages used again (the windows' pages given back, the others' kept), decode steps replayed as graphs, layers that read
another's keys and values, a token far back that must show in the logits through the causal layers alone, configurations drawn at random,
random weights made on the GPU, and greedy generation."""
import pytest
import torch

import plain_tilalorn
import scenarios
import tiny_tilalorn

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
FP32_TOL = dict(atol=4e-4, rtol=2e-4)        # logits of order ten; sums in another order than the 64-bit evaluation


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("tilalorn")
    return {name: tiny_tilalorn.write(name, root) for name in tiny_tilalorn.CONFIGS}


_weights_cache: dict = {}


def _weights(name, sharpen=1.0):
    key = (name, sharpen)
    if key not in _weights_cache:
        _weights_cache[key] = {k: v.double() for k, v in tiny_tilalorn.tensors_for(name, sharpen).items()}
    return _weights_cache[key]


def _rounded(t):
    return t.to(torch.bfloat16).double()


def _bf16_bound(conf, w, seqs, refs):
    """Three times what rounding to bfloat16 every tensor that separate kernels hand to each other does to the logits in a 64-bit evaluation."""
    return dict(atol=3 * max(float((plain_tilalorn.forward(conf, w, t, stored=_rounded)[0] - refs[r]).abs().max()) for r, t in seqs.items()), rtol=0.0)


def _tolerance(dtype, name, seqs, refs, sharpen=1.0):
    return FP32_TOL if dtype == "float32" else _bf16_bound(tiny_tilalorn.CONFIGS[name], _weights(name, sharpen), seqs, refs)


def _runner(folder, name, dtype, pages, slots=4, graphs=False):
    from torchlet_amd.engine.loading import load_model, make_runner
    _, model = load_model(folder, dtype)
    return make_runner(model, page_size=tiny_tilalorn.PAGE_SIZES[name], num_pages=pages, max_requests=slots, use_graphs=graphs)


def _replay(runner, steps):
    from torchlet_amd.engine.batch import StepEntry
    out = {}
    for s in steps:
        logits = runner.step([StepEntry(e["id"], e["tokens"], e["want"]) for e in s["entries"]])
        if logits is not None:
            out[s["step"]] = logits.cpu().numpy()
        for r in s["end"]:
            runner.release(r)
        runner.cache.check()
    return out


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_every_way_of_cutting_requests_equals_plain(folders, name, dtype):
    """Whole requests; most of a request and its last tokens one by one; portions of changing size down to two tokens; up to four live
    requests with portions beside single tokens, in a pool that holds no more than the live ones need, so pages and slots are used
    again.  The requests are several windows long."""
    lengths = [37, 5, 70, 1, 18, 33] if name != "B" else [90, 1, 47, 130]
    seqs, refs = tiny_tilalorn.sequences(name, _weights(name), lengths)
    tol = _tolerance(dtype, name, seqs, refs)
    page = tiny_tilalorn.PAGE_SIZES[name]
    for mode in ("whole", "tail_singles", "portions", "mixed"):
        steps = scenarios.number(getattr(scenarios, mode)(seqs) if mode != "tail_singles" else scenarios.tail_singles(seqs, tail=9))
        runner = _runner(folders[name], name, dtype, pages=-(-scenarios.max_tokens_needed(steps, unit=page) // page) + 1)
        scenarios.check(steps, _replay(runner, steps), refs, tol, f"{name}/{mode}/{dtype}")
        assert runner.cache.live_requests() == [] and runner.cache.free_pages() == runner.cache.capacity()


def test_stream_after_every_layer(folders):
    """The residual after every layer, in 32-bit (what the next norm's kernel sees once the pending output has been added times its
    factor): layer by layer against the plain implementation."""
    from torchlet_amd.engine.batch import StepEntry
    from torchlet_amd.kernels import ops
    name = "A"
    ids = [5, 17, 3, 60, 2, 2, 41, 9, 30, 11, 90, 7, 7, 45, 1, 96]
    _, want = plain_tilalorn.forward(tiny_tilalorn.CONFIGS[name], _weights(name), ids)
    runner = _runner(folders[name], name, "float32", pages=12, slots=1)
    seen = []

    def settled(stream):
        x = stream.residual.clone()
        ops.sandwich_norm(x, stream.pending, None, 0.0, None, torch.ones(1, device=x.device), 1e-5, torch.empty_like(x), branch_gain=stream.gain)
        return x.cpu()

    for block in runner.model.blocks:
        inner = block.forward
        block.forward = lambda stream, ctx, cache, inner=inner: (lambda s: (seen.append(settled(s)), s)[1])(inner(stream, ctx, cache))
    runner.step([StepEntry("a", ids, [len(ids) - 1])])
    assert len(seen) == len(want)
    for got, ref in zip(seen, want):
        torch.testing.assert_close(got.double(), ref, atol=1e-4, rtol=2e-5)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_from_the_first_token_and_slots_used_again(folders, dtype):
    """300 tokens one by one from an empty cache (many windows, many steps of the temperature; the windows' pages go back, the causal layers' stay)
    equal the plain implementation; the same request once more in the slot and the pages that the first one gave back, after another
    request has used them, gives the same logits bit for bit; and so does the whole request in one step, within the bound."""
    from torchlet_amd.engine.batch import StepEntry
    name = "B"
    seqs, refs = tiny_tilalorn.sequences(name, _weights(name), [300], seed=40)
    tol = _tolerance(dtype, name, seqs, refs)
    ids = seqs["r0"]
    runner = _runner(folders[name], name, dtype, pages=-(-300 // 16) + 1, slots=1)
    groups = runner.cache.groups
    assert sorted(g.need.window or 0 for g in groups) == [0, 21, 40] and sum(len(g.runs) for g in groups) == 3      # (the fourth layer has no cache)

    def one_by_one(req):
        rows = []
        for n, t in enumerate(ids):
            rows.append(runner.step([StepEntry(req, [t], [0])]).cpu())
            for i, g in enumerate(groups):
                held = runner.cache.capacity()[i] - runner.cache.free_pages()[i]
                assert held <= ((g.need.window + 14) // 16 + 1 if g.need.window else n // 16 + 1), (i, held)
        runner.release(req)
        return torch.cat(rows)

    first = one_by_one("a")
    torch.testing.assert_close(first.double(), refs["r0"], **tol)
    runner.step([StepEntry("other", ids[50:150], [])])          # leaves its own rows in the pages
    runner.release("other")
    assert torch.equal(one_by_one("b"), first)
    whole = runner.step([StepEntry("c", ids, list(range(300)))]).cpu()
    torch.testing.assert_close(whole.double(), refs["r0"], **tol)


@pytest.mark.parametrize("dtype", DTYPES)
def test_decode_steps_replayed_as_graphs(folders, dtype):
    """Three requests of unequal lengths decode together from static buffers under a recorded graph (padding rows use the page that
    belongs to no request): replays give what eager steps give."""
    from torchlet_amd.engine.batch import StepEntry
    name = "B"
    seqs, refs = tiny_tilalorn.sequences(name, _weights(name), [80, 9, 53], seed=7)
    got = {}
    for graphs in (False, True):
        runner = _runner(folders[name], name, dtype, pages=20, slots=3, graphs=graphs)
        assert runner.use_graphs == graphs
        rows = {r: [] for r in seqs}
        for r, t in seqs.items():
            rows[r].append(runner.step([StepEntry(r, t[:5], list(range(5)))]).cpu())
        for i in range(5, 80):
            live = [r for r, t in seqs.items() if i < len(t)]
            out = runner.step([StepEntry(r, [seqs[r][i]], [0]) for r in live]).cpu()
            for j, r in enumerate(live):
                rows[r].append(out[j: j + 1])
        got[graphs] = {r: torch.cat(v) for r, v in rows.items()}
        if graphs:
            assert runner.graph_replays > 30
    tol = _tolerance(dtype, name, seqs, refs)
    for r in seqs:
        torch.testing.assert_close(got[True][r].double(), refs[r], **tol)
        torch.testing.assert_close(got[True][r], got[False][r], atol=tol["atol"] / 2, rtol=0.0)


@pytest.mark.parametrize("seed", range(8))
def test_configurations_drawn_at_random(tmp_path, seed):
    """Layers of any kind in any order, sizes of the matrix-core kernels (even seeds) or small odd ones: whole requests, portions and
    mixed batches in both dtypes against the plain implementation, every pool full at the end."""
    import random
    from torchlet_amd.engine.loading import load_model, make_runner
    rnd = random.Random(700 + seed)
    conf = tiny_tilalorn.random_config(rnd, big=seed % 2 == 0)
    page = 16 if seed % 2 == 0 else rnd.choice([4, 8, 16])
    folder = tiny_tilalorn.write(f"random{seed}", tmp_path, config=conf, seed=seed)
    w = {k: v.double() for k, v in tiny_tilalorn.tensors_for("", 1.0, conf, seed).items()}
    seqs, refs = tiny_tilalorn.sequences("", w, [rnd.randint(1, 120) for _ in range(4)], seed=seed, config=conf, min_gap=0.01)
    for dtype in DTYPES:
        tol = dict(atol=8e-4, rtol=3e-4) if dtype == "float32" else _bf16_bound(conf, w, seqs, refs)
        _, model = load_model(folder, dtype)
        for mode in ("whole", "portions", "mixed"):
            steps = scenarios.number(getattr(scenarios, mode)(seqs))
            runner = make_runner(model, page_size=page, num_pages=-(-scenarios.max_tokens_needed(steps, unit=page) // page) + 1, max_requests=4)
            scenarios.check(steps, _replay(runner, steps), refs, tol, f"{conf}/{mode}/{dtype}")
            assert runner.cache.live_requests() == [] and runner.cache.free_pages() == runner.cache.capacity()


MIDDLE = dict(architecture="Tilalorn", vocab=1000, width=320, norm=dict(eps=1e-6), residual_mult=0.4, layers=[
    dict(type="latent_attention", mixer=dict(heads=8, dim=96, rot_dim=32, vdim=48, kv_rank=224, scale=0.1, rot=dict(dims=32, base=20000.0), mask=dict(size=100)),
         mlp=dict(kind="moe", expert=dict(ff=128), router=dict(experts=8, top=2, scale=2.0, groups=dict(count=4, keep=1)))),
    dict(type="attention", mixer=dict(heads=8, kv_heads=2, dim=128, vdim=112, scale=0.09, softcap=15.0, q_temp=dict(coef=0.4, every=50)),
         mlp=dict(kind="dense", ff=640)),
    dict(type="attention", mixer=dict(heads=6, kv_heads=6, dim=64, vdim=96, scale=0.13, softcap=6.0, q_temp=dict(coef=0.7, every=20)),
         mlp=dict(kind="moe", expert=dict(ff=96), router=dict(experts=6, top=3, scale=1.5, groups=dict(count=3, keep=2)))),
    dict(type="attention", mixer=dict(heads=4, kv_heads=2, dim=128, vdim=112, scale=0.11, softcap=9.0, q_temp=dict(coef=0.2, every=33), kv_from=1), mlp=None),
    dict(type="latent_attention", mixer=dict(heads=20, dim=32, rot_dim=16, vdim=64, kv_rank=144, scale=0.18, rot=dict(dims=16, base=500.0), mask=dict(size=40)),
         mlp=dict(kind="dense", ff=384)),
    dict(type="attention", mixer=dict(heads=12, kv_heads=6, dim=64, vdim=96, scale=0.1, softcap=20.0, q_temp=dict(coef=0.5, every=64), kv_from=2),
         mlp=dict(kind="dense", ff=256)),
])


@pytest.mark.parametrize("dtype", DTYPES)
def test_sizes_between_the_tiny_ones_and_a_real_model(tmp_path, dtype):
    """Widths and heads at which the products run on their tile kernels and the attentions in whole tiles: whole requests, portions and
    mixed batches against the plain implementation."""
    from torchlet_amd.engine.loading import load_model, make_runner
    folder = tiny_tilalorn.write("middle", tmp_path, config=MIDDLE, seed=51)
    w = {k: v.double() for k, v in tiny_tilalorn.tensors_for("middle", 1.0, MIDDLE, 51).items()}
    seqs, refs = tiny_tilalorn.sequences("", w, [230, 3, 121, 64], seed=3, config=MIDDLE, min_gap=0.02)
    tol = dict(atol=8e-4, rtol=3e-4) if dtype == "float32" else _bf16_bound(MIDDLE, w, seqs, refs)
    _, model = load_model(folder, dtype)
    for mode in ("whole", "portions", "mixed"):
        steps = scenarios.number(getattr(scenarios, mode)(seqs))
        runner = make_runner(model, page_size=16, num_pages=-(-scenarios.max_tokens_needed(steps, unit=16) // 16) + 1, max_requests=4)
        scenarios.check(steps, _replay(runner, steps), refs, tol, f"middle/{mode}/{dtype}")
        assert runner.cache.live_requests() == [] and runner.cache.free_pages() == runner.cache.capacity()


SHARP = dict(architecture="Tilalorn", vocab=80, width=64, norm=dict(eps=1e-5), residual_mult=0.5, layers=[
    dict(type="latent_attention", mixer=dict(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=48, scale=0.3, rot=dict(dims=16, base=10000.0), mask=dict(size=24)),
         mlp=dict(kind="dense", ff=64)),
    dict(type="latent_attention", mixer=dict(heads=2, dim=32, rot_dim=32, vdim=48, kv_rank=64, scale=0.3, rot=dict(dims=32, base=500.0), mask=dict(size=17)),
         mlp=dict(kind="dense", ff=64)),
])
CAUSAL = dict(type="attention", mixer=dict(heads=4, kv_heads=2, dim=32, vdim=48, scale=0.9, softcap=30.0, q_temp=dict(coef=0.5, every=40)), mlp=dict(kind="dense", ff=64))
READER = dict(type="attention", mixer=dict(heads=2, kv_heads=2, dim=32, vdim=48, scale=1.1, softcap=20.0, q_temp=dict(coef=0.3, every=64), kv_from=2), mlp=None)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layers", ["windows", "windows and causal", "windows, causal and a reader of its keys"])
def test_context_behind_the_windows_reaches_the_logits_through_the_causal_layers_only(tmp_path, dtype, layers):
    """Two latent attentions in windows of 24 and 17 positions, attention sharpened: the last of 200 tokens sees 40 positions back through both.
    Changing the token 39 positions back moves its logits, changing the one 40 back moves nothing at all; with a causal layer behind them every
    token moves the logits, and the 32-bit engine's logits move as the plain ones do, in a whole prompt and with the last token decoded
    alone after two portions."""
    from torchlet_amd.engine.batch import StepEntry
    from torchlet_amd.engine.loading import load_model, make_runner
    conf = dict(SHARP, layers=SHARP["layers"] + {"windows": [], "windows and causal": [CAUSAL], "windows, causal and a reader of its keys": [CAUSAL, READER]}[layers])
    sharpen = 3.0
    folder = tiny_tilalorn.write("sharp", tmp_path, sharpen=sharpen, config=conf, seed=31)
    w = {k: v.double() for k, v in tiny_tilalorn.tensors_for("sharp", sharpen, conf, 31).items()}
    g = torch.Generator().manual_seed(2)
    ids = torch.randint(0, conf["vocab"], (200,), generator=g).tolist()
    ref = plain_tilalorn.forward(conf, w, ids)[0]
    tol = FP32_TOL if dtype == "float32" else dict(atol=3 * float((plain_tilalorn.forward(conf, w, ids, stored=_rounded)[0] - ref).abs().max()), rtol=0.0)
    _, model = load_model(folder, dtype)
    runner = make_runner(model, page_size=16, num_pages=15, max_requests=2)

    def engine_last(tokens, cut):
        if cut:
            runner.step([StepEntry("d", tokens[:150], [])])
            runner.step([StepEntry("d", tokens[150:199], [])])
            out = runner.step([StepEntry("d", tokens[199:], [0])]).cpu()
        else:
            out = runner.step([StepEntry("d", tokens, [199])]).cpu()
        runner.release("d")
        return out[0].double()

    base = {cut: engine_last(ids, cut) for cut in (False, True)}
    torch.testing.assert_close(base[True], ref[199], **tol)
    torch.testing.assert_close(base[False], ref[199], **tol)
    for at in (199 - 39, 199 - 40, 48, 0):       # just inside the two windows, just outside, a page's border far back, the first token
        changed = ids[:at] + [(ids[at] + 1) % conf["vocab"]] + ids[at + 1:]
        other = plain_tilalorn.forward(conf, w, changed)[0][-1]
        move = other - ref[-1]
        for cut in (False, True):
            got = engine_last(changed, cut)
            if layers == "windows" and at < 199 - 39:
                assert float(move.abs().max()) == 0.0 and torch.equal(got, base[cut]), (at, cut)
                continue
            assert float(move.abs().max()) > (0 if at == 160 else 10) * FP32_TOL["atol"], at
            torch.testing.assert_close(got, other, **tol)
            if dtype == "float32":
                assert float((got - base[cut] - move).abs().max()) < 0.05 * float(move.abs().max()) + FP32_TOL["atol"], (at, cut)


def test_random_weights_made_on_the_gpu():
    """The random-weights mode draws on the device: matrices that are put together from several tensors and filled up with zero rows are made there."""
    from torchlet_amd.config import TilalornConfig
    from torchlet_amd.engine.batch import StepEntry
    from torchlet_amd.engine.loading import build_model, make_runner
    from torchlet_amd.weights.random_init import RandomTensors
    cfg = TilalornConfig.from_dict(tiny_tilalorn.CONFIGS["A"])
    model = build_model(cfg, "bfloat16", tensors=RandomTensors(cfg, seed=2, dtype=torch.bfloat16, device="cuda"))
    out = make_runner(model, page_size=4, num_pages=12, max_requests=1).step([StepEntry("a", list(range(20)), [19])])
    assert out.shape == (1, 97) and bool(torch.isfinite(out).all())


def _greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(plain_tilalorn.forward(cfg, w, ids)[0][-1].argmax()))
    return ids[len(prompt):]


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_entry_point(folders, dtype):
    """``LLM(folder).generate``: the registry picks the architecture from config.json, the scheduler cuts the prompts into portions of at
    most 16 tokens beside decode tokens, four requests share three slots, decode steps run as graphs with steps enqueued ahead."""
    from torchlet_amd import LLM
    name = "B"
    cfg, w = tiny_tilalorn.CONFIGS[name], _weights(name)
    g = torch.Generator().manual_seed(5)
    prompts = [torch.randint(0, cfg["vocab"], (n,), generator=g).tolist() for n in (5, 60, 1, 23)]
    llm = LLM(str(folders[name]), max_decode_slots=3, kv_block_size=16, max_num_blocks=24, dtype=dtype, max_num_batched_tokens=16,
              max_model_len=128)
    outs = llm.generate(prompts, max_new_tokens=7)
    assert [len(o) for o in outs] == [7] * 4 and len({tuple(o) for o in outs}) > 1
    for p, o in zip(prompts, outs):
        if dtype == "float32":
            assert o == _greedy(cfg, w, p, 7)
        else:                                   # a reduced-precision engine may pick another token among near-ties
            ids = list(p)
            for tok in o:
                logits = plain_tilalorn.forward(cfg, w, ids)[0][-1]
                assert float(logits.max() - logits[tok]) <= 0.4
                ids.append(tok)
    assert llm.runner.cache.live_requests() == []
