"""The Vabelorn design on the GPU through the framework's step function, cache manager, scheduler and entry point, against the plain
implementation: every way of cutting requests in both dtypes, the stream after every layer, long decoding from the first token, slots and
pages used again, decode steps replayed as graphs, a token far back that must show in the logits through the state alone and through the
attention alone, configurations drawn at random, and greedy generation."""
import pytest
import torch

import plain_vabelorn
import scenarios
import tiny_vabelorn

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
FP32_TOL = dict(atol=3e-4, rtol=3e-4)        # logits of order one to four; sums in another order than the 64-bit evaluation


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("vabelorn")
    return {name: tiny_vabelorn.write(name, root) for name in tiny_vabelorn.CONFIGS}


def _double(tensors):
    return {k: v.double() for k, v in tensors.items()}


def _weights(name):
    return _double(tiny_vabelorn.tensors_for(name))


def _rounded(t):
    return t.to(torch.bfloat16).double()


def _tolerance(dtype, conf, w, seqs, refs, fp32=FP32_TOL):
    """bfloat16: three times what rounding to bfloat16 every tensor that separate kernels hand to each other does in a 64-bit evaluation."""
    if dtype == "float32":
        return fp32
    return dict(atol=3 * max(float((plain_vabelorn.forward(conf, w, t, stored=_rounded)[0] - refs[r]).abs().max()) for r, t in seqs.items()), rtol=0.0)


def _runner(folder, dtype, page, pages, slots=4, graphs=False):
    from torchlet_amd.engine.loading import load_model, make_runner
    _, model = load_model(folder, dtype)
    return make_runner(model, page_size=page, num_pages=pages, max_requests=slots, use_graphs=graphs)


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


def _every_cut(folder, dtype, page, seqs, refs, tol, what):
    for mode in ("whole", "tail_singles", "portions", "mixed"):
        steps = scenarios.number(getattr(scenarios, mode)(seqs) if mode != "tail_singles" else scenarios.tail_singles(seqs, tail=9))
        runner = _runner(folder, dtype, page, pages=-(-scenarios.max_tokens_needed(steps, unit=page) // page) + 1)
        scenarios.check(steps, _replay(runner, steps), refs, tol, f"{what}/{mode}/{dtype}")
        assert runner.cache.live_requests() == [] and runner.cache.free_pages() == runner.cache.capacity()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_every_way_of_cutting_requests_equals_plain(folders, name, dtype):
    """Whole requests; a long portion and then single tokens; uneven portions down to two tokens; up to four live
    requests with portions beside single tokens, in a pool that holds no more than the live ones need, so pages and slots are used again."""
    lengths = [37, 5, 70, 1, 18, 33] if name != "B" else [90, 1, 47, 130]
    conf, w = tiny_vabelorn.CONFIGS[name], _weights(name)
    seqs, refs = tiny_vabelorn.sequences(w, lengths, conf)
    _every_cut(folders[name], dtype, tiny_vabelorn.PAGE_SIZES[name], seqs, refs, _tolerance(dtype, conf, w, seqs, refs), name)


def test_stream_after_every_layer(folders):
    """The 32-bit stream after every layer, once what is pending has been normed and added: layer by layer against the plain implementation."""
    from torchlet_amd.engine.batch import StepEntry
    from torchlet_amd.parts.base import Stream
    for name in ("A", "B"):
        conf = tiny_vabelorn.CONFIGS[name]
        ids = [5, 17, 3, 60, 2, 2, 41, 9, 30, 11, 79, 7, 7, 45, 1, 66]
        _, want = plain_vabelorn.forward(conf, _weights(name), ids)
        runner = _runner(folders[name], "float32", tiny_vabelorn.PAGE_SIZES[name], pages=12, slots=1)
        seen = []
        for block in runner.model.blocks:
            def wrapped(stream, ctx, cache, inner=block.forward, norm=block.mixer_norm):
                stream = inner(stream, ctx, cache)
                copy = Stream(stream.residual.clone(), stream.pending)
                copy.post = stream.post
                norm.settle(copy)
                seen.append(copy.residual.cpu())
                return stream
            block.forward = wrapped
        runner.step([StepEntry("a", ids, [len(ids) - 1])])
        assert len(seen) == len(want) == len(conf["layers"])
        for got, ref in zip(seen, want):
            torch.testing.assert_close(got.double(), ref, atol=1e-4, rtol=2e-5)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding_from_the_first_token_and_slots_used_again(folders, dtype):
    """300 tokens one by one from an empty cache equal the plain implementation; the same request once more in the slot and the pages that the
    first one gave back, after another request has used them, gives the same logits bit for bit; and so does the whole request in one step,
    within the bound."""
    from torchlet_amd.engine.batch import StepEntry
    name = "B"
    conf, w = tiny_vabelorn.CONFIGS[name], _weights(name)
    seqs, refs = tiny_vabelorn.sequences(w, [300], conf, seed=40)
    tol = _tolerance(dtype, conf, w, seqs, refs)
    ids = seqs["r0"]
    runner = _runner(folders[name], dtype, 16, pages=-(-300 // 16) + 1, slots=1)

    def one_by_one(req):
        rows = [runner.step([StepEntry(req, [t], [0])]).cpu() for t in ids]
        runner.release(req)
        return torch.cat(rows)

    first = one_by_one("a")
    torch.testing.assert_close(first.double(), refs["r0"], **tol)
    runner.step([StepEntry("other", ids[50:150], [])])          # leaves its own states, last inputs and rows in the slot and the pages
    runner.release("other")
    assert torch.equal(one_by_one("b"), first)
    whole = runner.step([StepEntry("c", ids, list(range(300)))]).cpu()
    torch.testing.assert_close(whole.double(), refs["r0"], **tol)


@pytest.mark.parametrize("dtype", DTYPES)
def test_decode_steps_replayed_as_graphs(folders, dtype):
    """Three requests of unequal lengths decode together from static buffers under a recorded graph (padding rows use the state row and
    the page that belong to no request): replays give what eager steps give."""
    from torchlet_amd.engine.batch import StepEntry
    name = "B"
    conf, w = tiny_vabelorn.CONFIGS[name], _weights(name)
    seqs, refs = tiny_vabelorn.sequences(w, [80, 9, 53], conf, seed=7)
    tol = _tolerance(dtype, conf, w, seqs, refs)
    got = {}
    for graphs in (False, True):
        runner = _runner(folders[name], dtype, 16, pages=20, slots=3, graphs=graphs)
        assert runner.use_graphs == graphs
        rows = {r: [runner.step([StepEntry(r, t[:5], list(range(5)))]).cpu()] for r, t in seqs.items()}
        for i in range(5, 80):
            live = [r for r, t in seqs.items() if i < len(t)]
            out = runner.step([StepEntry(r, [seqs[r][i]], [0]) for r in live]).cpu()
            for j, r in enumerate(live):
                rows[r].append(out[j: j + 1])
        got[graphs] = {r: torch.cat(v) for r, v in rows.items()}
        if graphs:
            assert runner.graph_replays > 30
    for r in seqs:
        torch.testing.assert_close(got[True][r].double(), refs[r], **tol)
        torch.testing.assert_close(got[True][r], got[False][r], atol=tol["atol"] / 2, rtol=0.0)


@pytest.mark.parametrize("seed", range(8))
def test_configurations_drawn_at_random(tmp_path, seed):
    import random
    rnd = random.Random(70 + seed)
    conf = tiny_vabelorn.random_config(rnd, big=seed % 2 == 0)
    page = 16 if seed % 2 == 0 else rnd.choice([4, 8, 16])
    tensors = tiny_vabelorn.tensors_for("", config=conf, seed=seed)
    folder = tiny_vabelorn.write(f"random{seed}", tmp_path, config=conf, tensors=tensors)
    w = _double(tensors)
    seqs, refs = tiny_vabelorn.sequences(w, [rnd.randint(1, 120) for _ in range(4)], conf, seed=seed)
    for dtype in DTYPES:
        _every_cut(folder, dtype, page, seqs, refs, _tolerance(dtype, conf, w, seqs, refs, dict(atol=8e-4, rtol=3e-4)), str(conf))


MIDDLE = dict(architecture="Vabelorn", vocab=1000, width=256, norm=dict(eps=1e-6), logit_scale=0.2, token_side=dict(dim=64), layers=[
    dict(type="wkv", mixer=dict(heads=6, dim=64, decay_rank=32), mlp=dict(kind="dense", ff=384)),
    dict(type="attention", mixer=dict(heads=8, kv_heads=2, dim=128, vdim=64, scale=0.09,
                                      rot=dict(dims=64, base=100000.0, scaling=dict(factor=8.0, original=256, fast=16.0, slow=1.0))), mlp=dict(kind="dense", ff=640)),
    dict(type="wkv", mixer=dict(heads=2, dim=128, decay_rank=48), mlp=None),
    dict(type="attention", mixer=dict(heads=6, kv_heads=6, dim=96, vdim=128, scale=0.1, rot=dict(dims=96, base=5000.0)), mlp=None),
])


@pytest.mark.parametrize("dtype", DTYPES)
def test_sizes_between_the_tiny_ones_and_a_real_model(tmp_path, dtype):
    """Widths and heads at which the products run on their tile kernels and the attention in whole tiles."""
    tensors = tiny_vabelorn.tensors_for("middle", config=MIDDLE, seed=51)
    folder = tiny_vabelorn.write("middle", tmp_path, config=MIDDLE, tensors=tensors)
    w = _double(tensors)
    seqs, refs = tiny_vabelorn.sequences(w, [230, 3, 121, 64], MIDDLE, seed=3)
    _every_cut(folder, dtype, 16, seqs, refs, _tolerance(dtype, MIDDLE, w, seqs, refs, dict(atol=8e-4, rtol=3e-4)), "middle")


_ATT = lambda heads, kv, dims, base: dict(type="attention", mixer=dict(heads=heads, kv_heads=kv, dim=32, vdim=32, scale=0.4, rot=dict(dims=dims, base=base)), mlp=dict(kind="dense", ff=64))
SHARP = dict(architecture="Vabelorn", vocab=80, width=64, norm=dict(eps=1e-5), logit_scale=0.3, token_side=dict(dim=8), layers=[_ATT(4, 1, 8, 1e4), _ATT(2, 2, 16, 500.0)])
STATES = dict(SHARP, layers=[dict(type="wkv", mixer=dict(heads=2, dim=32, decay_rank=8), mlp=dict(kind="dense", ff=64)),
                             dict(type="wkv", mixer=dict(heads=1, dim=64, decay_rank=4), mlp=None)])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("conf", [SHARP, STATES], ids=["attention", "states"])
def test_a_token_far_back_reaches_the_logits(tmp_path, conf, dtype):
    """Attention alone (sharpened) and time mixing alone (decays close to one).  Changing one of the first tokens, or one in the middle, of a
    200-token request moves the last logits, and the 32-bit engine's logits move as the plain ones do, in a whole prompt and with the last
    token decoded alone after two portions."""
    from torchlet_amd.engine.batch import StepEntry
    tensors = tiny_vabelorn.tensors_for("sharp", sharpen=3.0, config=conf, seed=31, remember=True)
    folder = tiny_vabelorn.write("sharp", tmp_path, config=conf, tensors=tensors)
    w = _double(tensors)
    seqs, refs = tiny_vabelorn.sequences(w, [200], conf, seed=2)
    ids, ref = seqs["r0"], refs["r0"]
    tol = _tolerance(dtype, conf, w, seqs, refs)
    runner = _runner(folder, dtype, 16, pages=15, slots=2)

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
    for at in (0, 1, 17, 100):
        changed = ids[:at] + [(ids[at] + 1) % conf["vocab"]] + ids[at + 1:]
        other = plain_vabelorn.forward(conf, w, changed)[0][-1]
        move = other - ref[-1]
        assert float(move.abs().max()) > 10 * FP32_TOL["atol"], at
        for cut in (False, True):
            got = engine_last(changed, cut)
            torch.testing.assert_close(got, other, **tol)
            if dtype == "float32":
                assert float((got - base[cut] - move).abs().max()) < 0.05 * float(move.abs().max()) + FP32_TOL["atol"] / 3, (at, cut)


def _greedy(cfg, w, prompt, n):
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(plain_vabelorn.forward(cfg, w, ids)[0][-1].argmax()))
    return ids[len(prompt):]


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_entry_point(folders, dtype):
    """``LLM(folder).generate``: the registry picks the architecture from config.json, the scheduler cuts the prompts into portions of at
    most 16 tokens beside decode tokens, four requests share three slots, decode steps run as graphs with steps enqueued ahead."""
    from torchlet_amd import LLM
    name = "B"
    cfg, w = tiny_vabelorn.CONFIGS[name], _weights(name)
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
                logits = plain_vabelorn.forward(cfg, w, ids)[0][-1]
                assert float(logits.max() - logits[tok]) <= 0.15
                ids.append(tok)
    assert llm.runner.cache.live_requests() == []
