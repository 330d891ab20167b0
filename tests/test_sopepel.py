"""Sopepel through the engine against the plain model (`tests/plain/sopepel.py`, written from the design's equations, no
cache, float64): every mechanism alone, every way of cutting a prompt, batches, reused pages and slots, keys at page
borders and just inside and just outside a chunk, the first tokens of a sequence, the token before a portion's first, what
a recurrent state still holds of the first tokens long after, rows that run in pieces and the pieces' borders, the router's
choice, long decoding, sizes that are 1 or equal, and greedy generation through the engine's own entry point. On the CPU the
plain twins of the operations stand in for the HIP kernels (this checks configuration, weights, cache, state and
batching); the `gpu` cases run the HIP kernels, each also alone against its twin."""
from __future__ import annotations

import functools
import json
import pathlib

import pytest
import torch

from tests import helpers as H
from tests import sopepel_models as M
from tests.plain import sopepel as plain
from tests.plain.ops import TorchKernels

DEVICES = [pytest.param("cpu", id="cpu-twin"), pytest.param("cuda", marks=pytest.mark.gpu, id="hip")]
DTYPES = ["float32", "bfloat16"]
MODELS = {"A": (M.CONFIG_A, 11, False, 8), "B": (M.CONFIG_B, 12, False, 16), "C": (M.CONFIG_C, 13, False, 4),
          "A-sharp": (M.CONFIG_A, 14, True, 16), "B-sharp": (M.CONFIG_B, 15, True, 8), "D-sharp": (M.CONFIG_D, 20, True, 16),
          "attention": (M.ONLY_ATTENTION, 16, True, 8), "linear": (M.ONLY_LINEAR, 17, False, 8),
          "dense": (M.ONLY_DENSE, 18, False, 16), "moe": (M.ONLY_MOE, 19, False, 8)}
LENGTHS = (40, 70, 33, 58, 50, 64, 21)
# bfloat16 engine against the float64 plain model, relative rms of the logits: what rounding alone gives on these
# models stays well below this; a lost key, state, gate or expert is far above it.
BF16_RMS = 0.08


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("sopepel")
    return {name: M.make_folder(root / name, cfg, seed, sharp) for name, (cfg, seed, sharp, _) in MODELS.items()}


@functools.lru_cache(maxsize=None)
def _plain(folder: str) -> M.PlainSopepel:
    return M.PlainSopepel(folder)


def _requests(name: str, lengths=LENGTHS) -> dict[str, list[int]]:
    return {f"r{i}": H.random_ids(n, MODELS[name][0]["vocab"], 300 + i) for i, n in enumerate(lengths)}


def _replayer(folder, device, dtype, page, cache_tokens, max_seqs=4, max_model_len=256, kernels=None):
    from holon_amd.engine.loading import load_model
    from holon_amd.engine.replay import Replayer
    if kernels is None and device == "cpu":
        kernels = TorchKernels()
    loaded = load_model(folder, device=device, dtype=dtype, kernels=kernels, page_size=page, max_seqs=max_seqs,
                        max_model_len=max_model_len, max_step_tokens=max_model_len, cache_tokens=cache_tokens)
    return Replayer(loaded)


def _check(folder, dtype, requests, got, what):
    folder = pathlib.Path(folder)
    want = {r: _plain(str(folder)).logits(ids) for r, ids in requests.items()}
    g, w = H.gather(want, got)
    assert torch.isfinite(g).all(), f"{what}: non-finite logits"
    if dtype == "float32":
        r, m = H.rel_rms(g, w), H.max_over_rms(g, w)
        assert r <= 3e-5 and m <= 3e-4, f"{what}: float32 logits differ: rms {r:.3g}, max {m:.3g}"
    else:
        # In bfloat16 a router's close call may fall the other way (its input is rounded), and the position then has
        # another expert's output: the float32 runs hold the choice itself, and here the worst 4 % of positions are
        # set aside for every routed feed-forward a token passes. What a lost key or state does to one position is
        # held by the tests that place it, on models without experts.
        config = json.loads((folder / "config.json").read_text())
        routed = sum((one.get("mlp") or {}).get("kind") == "moe" for one in config["layers"])
        per = (g - w).square().mean(-1).sqrt() / w.square().mean().sqrt()
        if routed:
            per = per.sort().values[: len(per) - int(len(per) * min(0.04 * routed, 0.3)) - 1]
        r = per.square().mean().sqrt().item()
        assert r <= BF16_RMS, f"{what}: bfloat16 logits differ: rms {r:.3g}"
        assert per.max().item() <= 3 * BF16_RMS, f"{what}: one position differs by {per.max().item():.3g}"


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(MODELS))
def test_every_way_of_cutting(folders, name, dtype, device):
    """Whole prompts (the first tokens of a sequence among them), token-by-token decoding from the second token on and
    after a long prompt, portions of changing size down to two tokens; in a pool that holds only the longest request,
    so that every request uses the pages and the slot of the one before."""
    folder, requests = folders[name], _requests(name)
    page = MODELS[name][3]
    rep = _replayer(folder, device, dtype, page, cache_tokens=-(-max(LENGTHS) // page) * page)
    got = H.run_trace(rep, H.trace_whole({**requests, "one": requests["r0"][:1]}))
    assert len(got) == sum(LENGTHS) + 1
    _check(folder, dtype, {**requests, "one": requests["r0"][:1]}, got, f"{name} {dtype} whole")
    rep.cache.check()
    for rid, tail in (("r2", len(requests["r2"]) - 1), ("r1", 32)):       # everything after the first token; a tail
        got = H.run_trace(rep, H.trace_decode_tail(rid, requests[rid], tail))
        assert len(got) == len(requests[rid])
        _check(folder, dtype, requests, got, f"{name} {dtype} decode tail {rid}")
    for rid, sizes in (("r3", [7, 2, 13, 3, 2, 30, 5]), ("r1", [2, 2, 17, 16, 1 + page, 2]), ("r5", [1, 3, page, 2])):
        got = H.run_trace(rep, H.trace_chunks(rid, requests[rid], sizes))
        assert len(got) == len(requests[rid])
        _check(folder, dtype, requests, got, f"{name} {dtype} portions {rid}")
    rep.cache.check()
    assert all(g.pool.free == g.pool.usable for g in rep.cache.groups)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "B-sharp", "C", "D-sharp", "attention", "linear"])
def test_mixed_batches_in_a_small_pool(folders, name, dtype, device):
    """Unequal requests side by side (portions beside single tokens, requests left out of steps) against each alone;
    three slots and a pool of the most that is ever live, so that pages and slots are given back and used again."""
    folder, requests = folders[name], _requests(name)
    page = MODELS[name][3]
    for seed in (0, 1):
        trace = H.trace_mixed(requests, seed=seed, max_live=3, decode_tail=6 + 5 * seed, max_chunk=19)
        rep = _replayer(folder, device, dtype, page, cache_tokens=H.peak_live_tokens(trace, round_to=page), max_seqs=3)
        got = H.run_trace(rep, trace)
        assert len(got) == sum(LENGTHS)
        _check(folder, dtype, requests, got, f"{name} {dtype} mixed seed {seed}")
        rep.cache.check()
        assert all(g.pool.free == g.pool.usable for g in rep.cache.groups)


@pytest.mark.parametrize("device", DEVICES)
def test_float32_does_not_depend_on_the_cut(folders, device):
    """A position's float32 logits whole, in portions, decoded and in a mixed batch: the same to rounding."""
    folder, requests = folders["B"], _requests("B", (45, 38, 27))
    rep = _replayer(folder, device, "float32", 16, cache_tokens=256)
    whole = H.run_trace(rep, H.trace_whole(requests))
    cut = H.run_trace(rep, H.trace_chunks("r0", requests["r0"], [3, 2, 16, 5]))
    tail = H.run_trace(rep, H.trace_decode_tail("r1", requests["r1"], 20))
    mixed = H.run_trace(rep, H.trace_mixed(requests, seed=5, max_live=3, decode_tail=7))
    for other in (cut, tail, mixed):
        for key, row in other.items():
            assert H.rel_rms(row, whole[key]) < 1e-5, f"{key}: logits depend on how the prompt was cut"


@pytest.mark.parametrize("device", DEVICES)
def test_the_stream_after_every_layer(folders, device):
    """The residual stream after each layer, float32, against the plain model's: the block's pending result (of a layer
    without feed-forward: two terms with their scales and the bias between them), normed, added to its rows."""
    from holon_amd.engine.batch import StepRow
    from holon_amd.parts.base import Stream
    from holon_amd.parts.stream32 import Pending
    folder = folders["A"]
    ids = H.random_ids(37, M.CONFIG_A["vocab"], 3)
    rep = _replayer(folder, device, "float32", 8, cache_tokens=40)
    slot = rep.cache.admit()
    rep.cache.reserve(slot, len(ids))
    step, _ = rep.runner.prepare([StepRow(slot, 0, ids, [])])
    model = rep.loaded.model
    stream = Stream(model.embed(step.token_ids, step.token_take, step=step, site=model.embed_site))
    assert stream.h.dtype == torch.float32
    want = _plain(str(folder)).streams(ids)
    assert len(want) == len(model.sites) == 5
    for site, ref in zip(model.sites, want):
        stream = model.blocks[site.layer](stream, step, site)
        d = stream.delta
        term = d.term
        if isinstance(term, Pending):
            term = sum(t.double() * s for t, s in term.terms) + term.row.double()
        x = stream.h.double() + plain.unit(term.double(), d.norm.eps) * d.gain.double()
        assert H.rel_rms(x.cpu(), ref) < 2e-5, f"layer {site.layer}"


def _steps(rep, steps) -> dict:
    """Steps given as [(request, tokens)] lists, every token's logits wanted -> {(request, position): logits}."""
    at, out = {}, {}
    for step in steps:
        logits = rep.step([{"id": r, "tokens": t, "want": list(range(len(t)))} for r, t in step]).cpu()
        row = 0
        for r, t in step:
            for _ in t:
                out[(r, at.get(r, 0))] = logits[row]
                at[r] = at.get(r, 0) + 1
                row += 1
    return out


def _needle(root, dims, chunk, key_at, query_at):
    """One layer of attention alone. A pair of token ids (query token, key token) whose score, with the key at position
    `key_at` and the query at `query_at`, stands out among all pairs', and a filler token whose scores with them and with
    itself are low; the norm of the queries is scaled until the pair's weight among the fillers is nearly all of it. The
    second table is zero, so a token's row does not depend on the one before. Returns the folder and the three ids."""
    dim, vdim, rot = dims
    cfg = M.model(32, 40, [M.layer(M.left(2, 2, dim, vdim, 0.25, chunk, rot, 30.0), M.right(1, 4, 4, 2.0, 2), None, (1.0, 0.0))])
    found = {}

    def edit(t):
        t["bigram"] = torch.zeros_like(t["bigram"])
        t["l0.mix.left.g"] = torch.zeros_like(t["l0.mix.left.g"])                 # every head passes by half
        p = {k: v.double() for k, v in t.items()}
        m, q_ = cfg["layers"][0]["mixer"]["left"], "l0.mix.left."
        n = 40
        q, k = (plain.heads_of(p, q_, p["embed"], s, 2, 1e-6)[:, 0] for s in "qk")

        def turned(x):                                                            # [place, token, dim]
            return plain.turn(x[None].expand(query_at + 1, n, dim), m["rot"])
        score = torch.einsum("ad,pbd->abp", turned(q)[query_at], turned(k)) * m["scale"]
        own = score[torch.arange(n), torch.arange(n), query_at]      # the query always sees its own key
        a, b = divmod(int((score[:, :, key_at] - own[:, None]).argmax()), n)
        worst = score[a].amax(-1)                       # a token's highest score with the query, wherever it stands
        worst[a] = worst[b] = float("inf")
        filler = int(worst.argmin())
        # the pair stands e^12 above any filler and above the query's own key
        gain = 12.0 / max(float(score[a, b, key_at] - max(worst[filler], own[a])), 1e-3)
        t[q_ + "q.norm"] = (p[q_ + "q.norm"] * gain).bfloat16()
        found.update(a=a, b=b, filler=filler)
    folder = M.make_folder(root, cfg, 77, edit=edit)
    return folder, found["a"], found["b"], found["filler"]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dims,chunk,page,key_at,query_at", [
    ((16, 12, 8), 180, 8, 180, 359),      # the first key of a chunk and the chunk's last query
    ((16, 12, 8), 180, 8, 179, 180),      # the last key before a chunk: not seen by the chunk's first query
    ((64, 64, 16), 160, 16, 160, 319), ((64, 64, 16), 160, 16, 159, 318), ((64, 64, 64), 150, 16, 150, 290),
    ((64, 64, 64), 150, 16, 149, 299), ((16, 12, 8), 37, 16, 74, 110), ((16, 12, 8), 37, 16, 73, 74),
    ((24, 24, 24), 300, 8, 7, 299), ((64, 64, 32), 300, 16, 16, 299), ((128, 128, 32), 256, 16, 0, 255),
    ((128, 128, 32), 256, 16, 255, 256)])
def test_a_key_at_the_edge_of_a_chunk(tmp_path, dims, chunk, page, key_at, query_at, dtype, device):
    """One key whose score stands out among hundreds, just inside or just outside the query's chunk, at page borders or
    not: inside it carries the result, outside it leaves none; in a whole prompt, in a prompt cut into portions (down to
    two tokens, the query in one of them; a cut inside the chunk) and when the query is decoded alone."""
    folder, a, b, filler = _needle(tmp_path / "needle", dims, chunk, key_at, query_at)
    plain_model = M.PlainSopepel(folder)
    inside = key_at // chunk == query_at // chunk
    ids = [filler] * key_at + [b] + [filler] * (query_at - key_at - 1) + [a, filler]
    without = [filler] * query_at + [a, filler]
    gap = H.rel_rms(plain_model.logits(ids)[query_at], plain_model.logits(without)[query_at])
    if not inside:
        assert gap < 1e-9
        wide = M.variant(plain_model.config)             # what seeing the key would do
        wide["layers"][0]["mixer"]["left"]["mask"]["size"] = 4096
        other = M.PlainSopepel(folder)
        other.config = wide
        gap = H.rel_rms(other.logits(ids)[query_at], plain_model.logits(ids)[query_at])
    assert gap > 0.1, f"the key does not show: {gap}"
    rep = _replayer(folder, device, dtype, page, cache_tokens=-(-len(ids) // page) * page, max_model_len=416)
    tol = gap / 8
    want = plain_model.logits(ids)[query_at]
    got = H.run_trace(rep, H.trace_whole({"f": ids}))
    _check(folder, dtype, {"f": ids}, got, "whole")
    assert H.rel_rms(got[("f", query_at)], want) < tol
    for sizes in ([query_at - 20, 2, 17, 2], [2, key_at + 1, 2, 7], [61, 2, 40]):
        got = H.run_trace(rep, H.trace_chunks("f", ids, sizes))
        assert H.rel_rms(got[("f", query_at)], want) < tol, f"portions {sizes}"
    got = H.run_trace(rep, H.trace_decode_tail("f", ids, min(len(ids) - 1, 30)))
    _check(folder, dtype, {"f": ids}, got, "decoded")
    assert H.rel_rms(got[("f", query_at)], want) < tol, "decoded alone"
    rep.cache.check()


def test_pages_of_finished_chunks_are_given_back(folders):
    """While a request decodes it holds no page that lies wholly in finished chunks, in every group of its own."""
    folder = folders["A"]
    ids = H.random_ids(70, M.CONFIG_A["vocab"], 5)
    rep = _replayer(folder, "cpu", "float32", 4, cache_tokens=72)
    sizes = sorted({one["mixer"]["left"]["mask"]["size"] for one in M.CONFIG_A["layers"]})
    assert sorted({g.decl.chunk for g in rep.cache.groups}) == sizes
    for at in range(70):
        rep.step([{"id": "x", "tokens": [ids[at]], "want": [0]}])
        slot = rep.slots["x"]
        for g in rep.cache.groups:
            c, n = g.decl.chunk, at + 1
            assert g.first[slot] == (n - n % c) // 4
        rep.cache.check()


def _long_memory(root, dims=(20, 12)):
    """One layer of linear attention whose decays are near one: what the first token wrote is read hundreds of tokens
    later. Some channels decay quickly."""
    cfg = M.model(32, 40, [M.layer(M.left(1, 1, 8, 8, 0.3, 4, 4), M.right(2, *dims, 16.0, 4), None, (0.0, 1.0))])

    def edit(t):
        b = torch.full((2 * dims[0],), 6.0)
        b[::3] = 2.0
        b[1::5] = -3.0
        t["l0.mix.right.a2.b"] = b.bfloat16()
        t["l0.mix.right.a2"] = (0.3 * t["l0.mix.right.a2"].float()).bfloat16()
    return M.make_folder(root, cfg, 5, edit=edit)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("dims", [(20, 12), (64, 80)])
def test_a_state_that_reaches_far_and_the_pieces_borders(tmp_path, dims, dtype, device):
    """A first token that still shows 400 tokens later; rows of that length run in pieces of 128 tokens and blocks of 16,
    and portions end just before, at and just behind a piece's and a block's border, so that a state is handed on at
    every kind of place; then single tokens across the same positions."""
    folder = _long_memory(tmp_path / "m", dims)
    base = M.PlainSopepel(folder)
    ids = H.random_ids(430, 40, 9)
    other = [(ids[0] + 7) % 40] + ids[1:]
    gap = H.rel_rms(base.logits(other)[-1], base.logits(ids)[-1])
    assert gap > 3e-3, f"the first token does not show: {gap}"
    rep = _replayer(folder, device, dtype, 16, cache_tokens=432, max_model_len=432)
    for sizes in ([430], [257, 2, 171], [256, 128, 46], [129, 255, 46], [64, 63, 2, 1, 257, 43], [2, 428], [16, 15, 17, 382]):
        got = H.run_trace(rep, H.trace_chunks("x", ids, sizes))
        _check(folder, dtype, {"x": ids}, got, f"portions {sizes}")
        if dtype == "float32":
            assert H.rel_rms(got[("x", 429)], base.logits(ids)[429]) < gap / 30
    got = H.run_trace(rep, H.trace_chunks("x", ids, [250] + [1] * 12 + [168]))
    _check(folder, dtype, {"x": ids}, got, "single tokens across a piece's border")
    ids2 = H.random_ids(300, 40, 10)
    rep = _replayer(folder, device, dtype, 16, cache_tokens=1040, max_model_len=560)
    got = _steps(rep, [[("a", ids[:130]), ("b", ids2[:1])], [("a", ids[130:131]), ("b", ids2[1:290])],
                       [("b", ids2[290:291]), ("a", ids[131:])], [("b", ids2[291:])]])
    _check(folder, dtype, {"a": ids, "b": ids2}, got, "two long rows side by side")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_the_token_before_a_portion(folders, dtype, device):
    """The row of the second table is chosen by the token before, which a portion's first token takes from the request's
    state: portions of one and two tokens side by side in one batch, a request left out of steps in between, a slot that
    another request has used; against the row of the wrong token, or of none, the logits are far away."""
    folder = folders["dense"]
    base = _plain(str(folder))
    ids, other = H.random_ids(12, 90, 1), H.random_ids(9, 90, 2)
    changed = [ids[0], (ids[1] + 1) % 90] + ids[2:]
    assert H.rel_rms(base.logits(changed)[2], base.logits(ids)[2]) > 0.05, "the token before does not show"
    rep = _replayer(folder, device, dtype, 16, cache_tokens=64, max_seqs=2)
    got = _steps(rep, [[("a", ids[:3]), ("b", other[:1])], [("b", other[1:2])], [("a", ids[3:4]), ("b", other[2:4])],
                       [("a", ids[4:6])], [("b", other[4:5]), ("a", ids[6:7])], [("b", other[5:]), ("a", ids[7:])]])
    _check(folder, dtype, {"a": ids, "b": other}, got, "portions")
    rep.step([], ["a", "b"])
    got = _steps(rep, [[("c", other[:1])], [("c", other[1:])]])
    _check(folder, dtype, {"c": other}, got, "a slot used again")


@pytest.mark.parametrize("device", DEVICES)
def test_each_mechanism_shows(folders, tmp_path, device):
    """Biases, norms, gates, decays, scales, both tables and the router each move the plain model's logits far more than
    the engine differs from it: a mechanism left out or mistaken would not pass the other tests."""
    ids = H.random_ids(60, 90, 4)
    flip = lambda t: t.flip(-1)                    # noqa: E731
    rows = lambda t: t.flip(0)                     # noqa: E731
    none = lambda t: t * 0.0                       # noqa: E731
    cases = [("attention", "l0.mix.left.g", lambda t: -t), ("attention", "l0.mix.left.q.b", none),
             ("attention", "l0.mix.left.k.b", none), ("attention", "l1.mix.left.v.b", none),
             ("attention", "l1.mix.left.o.b", none), ("attention", "l0.mix.left.q.norm", flip),
             ("attention", "l1.mix.left.k.norm", flip), ("attention", "l1.norm1", flip), ("attention", "bigram", rows),
             ("linear", "l0.mix.right.a2.b", flip), ("linear", "l1.mix.right.a1", rows), ("linear", "l0.mix.right.a2", rows),
             ("linear", "l0.mix.right.norm", flip), ("linear", "l1.mix.right.g", rows), ("dense", "l0.norm2", flip),
             ("dense", "l0.mlp.gate", rows), ("moe", "l0.mlp.router", rows), ("moe", "l0.mlp.shared.sg", lambda t: -t),
             ("moe", "final.norm", flip)]
    for name, key, change in cases:
        base = _plain(str(folders[name]))
        cfg, seed, sharp, page = MODELS[name]

        def edit(t, key=key, change=change):
            t[key] = change(t[key].float()).bfloat16()
        other = M.PlainSopepel(M.make_folder(tmp_path / f"{name}-{key}", cfg, seed, sharp, edit=edit))
        gap = H.rel_rms(other.logits(ids), base.logits(ids))
        rep = _replayer(folders[name], device, "float32", page, cache_tokens=64)
        got = H.run_trace(rep, H.trace_chunks("x", ids, [23, 2, 9]))
        g, w = H.gather({"x": base.logits(ids)}, got)
        assert gap > 5e-3 and H.rel_rms(g, w) < gap / 100, f"{name} {key}: gap {gap}"
    for name, path, value in (("attention", ("layers", 0, "mixer", "left", "mask", "size"), 14),
                              ("attention", ("layers", 0, "mixer", "left", "rot", "base"), 900.0),
                              ("attention", ("layers", 1, "mixer", "left", "rot", "dims"), 6),
                              ("attention", ("layers", 0, "mixer", "left", "scale"), 0.25),
                              ("linear", ("layers", 0, "mixer", "right", "tau"), 5.0), ("A", ("layers", 1, "mixer", "left_scale"), 1.0),
                              ("A", ("layers", 2, "mixer", "right_scale"), 0.7), ("linear", ("logit_scale",), 0.75),
                              ("linear", ("embedding", "bigram", "mul_prev"), 6), ("linear", ("embedding", "bigram", "mul_cur"), 4),
                              ("moe", ("layers", 0, "mlp", "router", "top"), 3), ("C", ("norm", "eps"), 0.3)):
        changed = M.variant(MODELS[name][0])
        where = changed
        for key in path[:-1]:
            where = where[key]
        where[path[-1]] = value
        other = M.PlainSopepel(folders[name])             # the same weights, one constant changed
        other.config = changed
        one = [i % MODELS[name][0]["vocab"] for i in ids]
        assert H.rel_rms(other.logits(one), _plain(str(folders[name])).logits(one)) > 3e-3, (name, path)


@pytest.mark.parametrize("device", DEVICES)
def test_the_router_chooses_as_the_plain_model(device):
    """The router's weights on their own: the largest scores, equal ones to the lower index, each weight the score itself
    or its square, the shared expert's gate in the last column."""
    import holon_amd.parts  # noqa: F401
    from holon_amd.kernels.registry import kernel_op
    if device == "cuda":
        from holon_amd.kernels import load_hip
        router_top = load_hip().moe_router_top
    else:
        router_top = kernel_op("moe_router_top").plain
    g = torch.Generator().manual_seed(3)
    for experts, top, width, gated in ((8, 3, 64, 1), (12, 1, 250, 0), (6, 6, 32, 1), (1, 1, 8, 1), (64, 6, 512, 0),
                                       (130, 9, 48, 1), (96, 5, 33, 0)):
        x = torch.randn(50, width, generator=g).to(device)
        router = (2.0 * torch.randn(experts + gated, width, generator=g) * width ** -0.5).to(device)
        if experts > 1:
            router[1] = router[0]                  # two experts with equal scores
        z = x.double().cpu() @ router.double().cpu().T
        for score, power in (("sigmoid", 1), ("sigmoid_squared", 2)):
            got = router_top(x, router, None, experts, top, score=score).cpu().double()
            for t in range(50):
                near = sorted(z[t, :experts].tolist())
                if experts > 2 and min((b - a for a, b in zip(near, near[1:]) if b != a), default=1.0) < 1e-5:
                    continue                       # a call that float32 cannot make
                want = torch.zeros(experts + gated, dtype=torch.float64)
                for e, weight in plain.route(z[t, :experts], top):
                    want[e] = weight ** power
                if gated:
                    want[experts] = plain.sigmoid(z[t, experts])
                assert torch.allclose(got[t], want, atol=2e-6), (experts, top, t)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A-sharp", "D-sharp"])
def test_long_decoding(folders, name, dtype, device):
    """180 tokens one by one after a prompt of 5, over many pages and chunks."""
    folder, page = folders[name], MODELS[name][3]
    ids = H.random_ids(185, MODELS[name][0]["vocab"], 21)
    rep = _replayer(folder, device, dtype, page, cache_tokens=192)
    got = H.run_trace(rep, H.trace_decode_tail("d", ids, 180))
    _check(folder, dtype, {"d": ids}, got, f"long decoding {dtype}")
    rep.cache.check()
    assert all(g.pool.free == g.pool.usable for g in rep.cache.groups)


def test_what_is_kept(folders):
    """The states the parts declare: keys and values in chunks and a matrix a head in every layer, and the embedding's
    last token."""
    rep = _replayer(folders["A"], "cpu", "float32", 8, cache_tokens=64)
    model = rep.loaded.model
    kept = [[(d.name, getattr(d, "chunk", None) or tuple(d.shape)) for d in decls] for decls in model.state_decls()]
    assert kept[0] == [("left.kv", 10), ("right.S", (3, 12, 20))] and kept[-1] == [("token", ())] and len(kept) == 6
    assert model.embed_site.slot_state["token"].dtype == torch.int32
    assert model.sites[0].slot_state["right.S"].dtype == torch.float32
    one = model.blocks[0].mixer
    assert one.inp is not None and one.left.qkv is None and one.right.inp is None       # one product for both mixers


def test_configuration_and_weights_are_checked(tmp_path):
    from holon_amd.config.model import ConfigError
    from holon_amd.registry import resolve
    from holon_amd.weights.loader import WeightError
    cfg, spec = resolve(M.CONFIG_A)
    assert cfg.to_dict()["layers"] == M.CONFIG_A["layers"] and cfg.to_dict()["embedding"] == M.CONFIG_A["embedding"]
    assert resolve(cfg.to_dict())[1].identity() == spec.identity()
    assert resolve(M.variant(M.CONFIG_A, logit_scale=0.3))[1].identity() != spec.identity()

    def changed(path, value):
        c = M.variant(M.CONFIG_A)
        where = c
        for key in path[:-1]:
            where = where[key]
        where[path[-1]] = value
        return c
    mix = ("layers", 0, "mixer")
    for bad in ({k: v for k, v in M.CONFIG_A.items() if k != "norm"}, M.variant(M.CONFIG_A, layers=[]),
                M.variant(M.CONFIG_A, layers=[{"type": "conv", "mixer": {}, "mlp": None}]),
                changed(("embedding", "bigram", "buckets"), 0), changed(("embedding", "bigram", "mul_prev"), 1.5),
                changed((*mix, "left", "kv_heads"), 3), changed((*mix, "left", "rot", "dims"), 7),
                changed((*mix, "left", "rot", "dims"), 18), changed((*mix, "left", "mask", "size"), 0),
                changed((*mix, "right", "tau"), 0.0), changed((*mix, "right", "vdim"), None), changed((*mix, "left_scale"), "1"),
                changed(("layers", 0, "mlp", "router", "top"), 7), changed(("layers", 0, "mlp", "kind"), "polynorm")):
        with pytest.raises(ConfigError):
            resolve(bad)

    def drop(t):
        del t["l1.mix.left.g"]
        t["l0.mix.right.a2.b"] = torch.zeros(5).bfloat16()
        t["l0.mix.right.pb"] = torch.zeros(4).bfloat16()
    folder = M.make_folder(tmp_path / "bad", M.CONFIG_A, 1, edit=drop)
    from holon_amd.engine.loading import load_model
    with pytest.raises(WeightError) as e:
        load_model(folder, device="cpu", dtype="float32", kernels=TorchKernels(), max_model_len=32, max_seqs=2)
    assert "l1.mix.left.g" in str(e.value) and "l0.mix.right.a2.b" in str(e.value) and "l0.mix.right.pb" in str(e.value)

    def idle(t):                                                 # a layer without feed-forward may still list its norm
        t["l2.norm2"] = torch.ones(64).bfloat16()
    load_model(M.make_folder(tmp_path / "idle", M.CONFIG_A, 1, edit=idle), device="cpu", dtype="float32",
               kernels=TorchKernels(), max_model_len=32, max_seqs=2)
    unranked = M.variant(M.CONFIG_A)                             # the decays' rank is the checkpoint's where none is named
    for one in unranked["layers"]:
        del one["mixer"]["right"]["rank"]
    named = M.make_folder(tmp_path / "named", M.CONFIG_A, 1)
    (named / "config.json").write_text(json.dumps(unranked))
    loaded = load_model(named, device="cpu", dtype="float32", kernels=TorchKernels(), max_model_len=32, max_seqs=2)
    assert [b.mixer.right.rank for b in loaded.model.blocks] == [6, 5, 3, 16, 6]


@pytest.mark.parametrize("device", DEVICES)
def test_random_weights_from_the_command_line_replay(tmp_path, device):
    """`holon_amd random` writes a Sopepel folder, and the engine and the plain model agree on it."""
    from holon_amd.cli import main
    (tmp_path / "c.json").write_text(json.dumps(M.CONFIG_A))
    assert main(["random", "--config", str(tmp_path / "c.json"), "--seed", "4", "--out", str(tmp_path / "m")]) == 0
    ids = H.random_ids(30, M.CONFIG_A["vocab"], 2)
    rep = _replayer(tmp_path / "m", device, "float32", 8, cache_tokens=32)
    got = H.run_trace(rep, H.trace_chunks("a", ids, [4, 9]))
    _check(tmp_path / "m", "float32", {"a": ids}, got, "random folder")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("overlap", [True, False])
def test_greedy_generation_through_the_engine(folders, dtype, overlap, device):
    """The engine's own entry point and scheduler: prompts of unequal length generated side by side, with prompt
    portions riding beside decode rows whose tokens may still be on the device, follow the plain model's most likely token
    wherever that is clear."""
    from holon_amd.config import EngineConfig, SamplingParams
    from holon_amd.engine.engine import Engine
    folder = folders["B-sharp"]
    plain_model = _plain(str(folder))
    prompts = [H.random_ids(n, M.CONFIG_B["vocab"], 50 + n) for n in (5, 37, 18, 1)]
    cfg = EngineConfig(model=str(folder), device=device, dtype=dtype, page_size=8, max_seqs=3, max_model_len=96,
                       max_step_tokens=40, chunk_with_decode=16, cache_tokens=192, overlap=overlap)
    engine = Engine(cfg, TorchKernels() if device == "cpu" else None)
    outs = engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=24, ignore_eos=True))
    held = sum(H.assert_greedy_follows(plain_model, p, o, margin=0.02 if dtype == "float32" else 0.25)
               for p, o in zip(prompts, outs))
    assert all(len(o) == 24 for o in outs) and held >= (60 if dtype == "float32" else 20)
    engine.cache.check()
    engine.close()


@pytest.mark.gpu
@pytest.mark.parametrize("name,dtype", [("A-sharp", "float32"), ("A-sharp", "bfloat16"), ("D-sharp", "float32")])
def test_graph_replays_equal_eager_steps(folders, name, dtype):
    """Decode steps replayed from HIP graphs give the tokens of eager steps, over many replays with the program's own
    eager work (prompt steps, sampling, host synchronisation) between them, while the batch shrinks through the
    buckets and pages are taken and given back."""
    from holon_amd.config import EngineConfig, SamplingParams
    from holon_amd.engine.engine import Engine
    vocab = MODELS[name][0]["vocab"]
    prompts = [H.random_ids(n, vocab, 80 + n) for n in (3, 17, 8, 25, 40, 1)]
    outs = {}
    for graphs in (False, True):
        engine = Engine(EngineConfig(model=str(folders[name]), device="cuda", dtype=dtype, page_size=16, max_seqs=6,
                                     max_model_len=160, max_step_tokens=64, graphs=graphs, cache_tokens=960))
        rids = [engine.add(p, SamplingParams(temperature=0.0 if i % 2 else 0.7, seed=5, max_tokens=60 + 7 * i,
                                             ignore_eos=True)) for i, p in enumerate(prompts)]
        got = {r: [] for r in rids}
        while engine.has_work():
            for d in engine.step():
                got[d.rid].extend(d.token_ids)
        outs[graphs] = [got[r] for r in rids]
        engine.cache.check()
        if graphs:
            assert engine.runner.graph_replays > 20 and len(engine.runner.graphs) >= 3
        engine.close()
    assert outs[True] == outs[False]


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_kernels_alone_against_their_plain_forms(dtype):
    """Every operation the design brought or changed, on the GPU, against its plain form in torch."""
    import holon_amd.parts  # noqa: F401
    from holon_amd.kernels import load_hip
    from holon_amd.kernels.registry import kernel_op
    from holon_amd.parts.linear_attention import PIECE, gla_step_serves
    k, dev = load_hip(), "cuda"
    tol = 3e-6 if dtype == torch.float32 else 6e-3
    g = torch.Generator().manual_seed(0)

    def randn(*shape, to=dtype):
        return torch.randn(*shape, generator=g).to(dev).to(to)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)          # noqa: E731
    for dim in (96, 250, 1500, 2048, 3000, 8192, 9001):      # a result of two terms and a vector, normed, added; the next norm
        x, t1, t2, row = randn(7, dim, to=torch.float32), randn(7, dim), randn(7, dim), randn(dim, to=torch.float32)
        gain, w = randn(dim, to=torch.float32), 1 + 0.3 * randn(dim)
        for weight in (w, None):
            for mix in (None, (0.7, t2, -1.3, row), (1.0, t2, 0.5, None)):
                xa, xb = x.clone(), x.clone()
                a = k.stream_rms_post(xa, t1, gain, 1e-5, weight, 1e-6, dtype, mix)
                b = kernel_op("stream_rms_post").plain(xb, t1, gain, 1e-5, weight, 1e-6, dtype, mix)
                assert H.rel_rms(xa, xb) < 1e-6 and H.rel_rms(a, b) < tol, (dim, mix is None, weight is None)
        assert torch.equal(k.narrow_rows(x, dtype), x.to(dtype))
    # the embedding: rows that start and rows that continue, tokens that are still on the device, state kept by slot
    counts, starts, slots = [1, 9, 2, 5, 1, 3], [0, 0, 7, 3, 12, 2], [5, 0, 3, 1, 4, 2]
    qs = [0]
    for c in counts:
        qs.append(qs[-1] + c)
    token_row = i32([b for b, c in enumerate(counts) for _ in range(c)])
    for width, buckets, mul_prev, mul_cur in ((64, 37, 5, 3), (33, 1, 1, 1), (2048, 1009, (1 << 31) - 1, 1 << 30), (20, 50, 0, 7)):
        table, bigram = randn(90, width), randn(buckets + 1, width)
        ids = torch.randint(0, 90, (qs[-1],), generator=g, dtype=torch.int32).to(dev)
        prev = torch.randint(0, 90, (6,), generator=g, dtype=torch.int32).to(dev)
        take = (torch.full((qs[-1],), -1, dtype=torch.int32, device=dev), torch.randint(0, 90, (7,), generator=g, dtype=torch.int32).to(dev))
        take[0][0], take[0][qs[4]] = 5, 4
        for taken in (None, take):
            pa, pb = prev.clone(), prev.clone()
            args = (i32(slots), i32(starts), i32(qs), token_row, 6, mul_prev, mul_cur)
            a = k.bigram_embedding(ids, taken, table, bigram, pa, *args)
            b = kernel_op("bigram_embedding").plain(ids, taken, table, bigram, pb, *args)
            assert torch.equal(a, b) and torch.equal(pa, pb), (width, buckets)
            single = None if taken is None else (taken[0][:6].contiguous(), taken[1])
            args = (i32(slots), i32(starts), i32(list(range(7))), i32(list(range(6))), 6, mul_prev, mul_cur, True)
            a = k.bigram_embedding(ids[:6], single, table, bigram, pa, *args)
            b = kernel_op("bigram_embedding").plain(ids[:6], single, table, bigram, pb, *args)
            assert torch.equal(a, b) and torch.equal(pa, pb), (width, buckets, "single")
    # gated linear attention: columns of wider rows; single tokens, short rows, rows in pieces
    lens = [1, 300, 2, 64, 129, 530]
    at = [0]
    for c in lens:
        at.append(at[-1] + c)
    for heads, dim, vdim, rank, extra in ((3, 12, 20, 5, 7), (2, 64, 64, 16, 16), (1, 1, 1, 1, 3), (4, 32, 144, 16, 0),
                                          (2, 128, 128, 16, 8), (1, 200, 33, 40, 5), (2, 256, 256, 16, 8), (5, 24, 8, 3, 1),
                                          (1, 17, 300, 2, 2), (2, 48, 1000, 4, 8), (16, 128, 128, 16, 16)):
        c, n = heads * dim, heads * vdim
        wide = randn(at[-1], 2 * c + 2 * n + rank + extra)
        q, kk, v = wide[:, extra: extra + c], wide[:, extra + c: extra + 2 * c], wide[:, extra + 2 * c: extra + 2 * c + n]
        gate, a1 = wide[:, extra + 2 * c + n: extra + 2 * c + 2 * n], wide[:, extra + 2 * c + 2 * n:]
        w2t, bias = randn(rank, c) * rank ** -0.5, 2.0 * randn(c, to=torch.float32)
        bias[:: 7] = -20.0                                    # channels that forget at once, and some that never do
        bias[1:: 7] = 30.0
        S = randn(6, heads, dim, vdim, to=torch.float32)
        alpha = k.gla_decay(a1, w2t, bias, 4.0)
        assert H.rel_rms(alpha, kernel_op("gla_decay").plain(a1, w2t, bias, 4.0)) < 2e-6, (heads, dim)
        rows = (i32(slots), i32(starts), i32(at), 6, heads)
        npc = [-(-m // PIECE) for m in lens]
        pieces = (PIECE, max(npc), i32([sum(npc[:b]) for b in range(6)]), sum(npc))
        ref = kernel_op("gla_scan").plain(q, kk, v, dim ** -0.5, alpha, sb := S.clone(), *rows)
        for cut in (None, pieces):
            sa = S.clone()
            got = k.gla_scan(q, kk, v, dim ** -0.5, alpha, sa, *rows, cut)
            assert H.rel_rms(got, ref) < 4e-6 and H.rel_rms(sa, sb) < 4e-6, (heads, dim, vdim, cut is None)
            per = ((got - ref).square().mean(1).sqrt() / ref.square().mean().sqrt()).max().item()
            assert per < 4e-5, (heads, dim, vdim, per)
        assert gla_step_serves(dim, vdim) == bool(k.lib.holon_gla_step_supported(dim, vdim)), (dim, vdim)
        if gla_step_serves(dim, vdim):
            weight = 1 + 0.2 * randn(vdim)
            sa, sb = S.clone(), S.clone()
            cols = [x[:6] for x in (q, kk, v, gate, a1)]
            args = (dim ** -0.5, w2t, bias, 4.0, weight, 1e-5)
            a = k.gla_step(*cols, *args, sa, i32(slots), i32(starts), heads)
            b = kernel_op("gla_step").plain(*cols, *args, sb, i32(slots), i32(starts), heads)
            assert H.rel_rms(a, b) < max(tol, 8e-6) and H.rel_rms(sa, sb) < 4e-6, (heads, dim, vdim)
    # experts without gates, the gelu gate, alone and in the few-row product
    for experts, ff, shared, gated in ((6, 16, 24, 1), (5, 24, 0, 0), (3, 7, 9, 1), (10, 72, 136, 1), (1, 8, 8, 0)):
        up = randn(19, experts * ff + shared)
        weights = torch.rand(19, experts + gated, generator=g).to(dev)
        weights[:, :experts] *= (torch.rand(19, experts, generator=g) < 0.4).to(dev)
        a = k.moe_relu2(up, weights, ff, shared, shared_weight=bool(gated))
        assert H.rel_rms(a, kernel_op("moe_relu2").plain(up, weights, ff, shared, bool(gated))) < tol, (experts, ff)
    for rows_, f in ((1, 32), (9, 100), (40, 33), (300, 1024)):
        gu = 3.0 * randn(rows_, 2 * f)
        assert H.rel_rms(k.gelu_mul(gu), kernel_op("gelu_mul").plain(gu.double())) < tol, (rows_, f)
    if dtype == torch.bfloat16:
        for rows_, f, width in ((1, 256, 256), (8, 8192, 2048), (16, 512, 384), (5, 12288, 512)):
            x, w = randn(rows_, width), randn(2 * f, width) * width ** -0.5
            want = kernel_op("gelu_mul").plain((x.double() @ w.double().T))
            for tiled in (None, k.tile_weight(w)):
                got = k.linear_gelu_mul(x, w, tiled)
                assert got is not None and H.rel_rms(got, want) < tol, (rows_, f, width)


def _scattered(lens, page, columns, g):
    """A block table over scattered pages: (table, number of pages)."""
    n_pages = sum(-(-n // page) for n in lens) + 1
    table = torch.full((len(lens) + 1, columns), n_pages - 1, dtype=torch.int32)
    order, at = torch.randperm(n_pages - 1, generator=g).tolist(), 0
    for s_, n in enumerate(lens):
        for i in range(-(-n // page)):
            table[s_, i] = order[at]
            at += 1
    return table, n_pages


@pytest.mark.gpu
@pytest.mark.parametrize("dim", [64, 128, 256])
def test_chunks_in_the_attention_kernels(dim):
    """Attention inside chunks: in bfloat16 every prompt form of the matrix cores (short and long portions, stages through
    registers and copied directly, one and two tiles a wave, groups of heads of every size) and the decode kernel, in both
    types the general kernel; portions that start and end inside chunks beside decode rows at their edges, with a gate a
    head and without, with a cap; against float64."""
    import holon_amd.parts  # noqa: F401
    from holon_amd.kernels import load_hip
    from holon_amd.kernels.api import AttnRows
    from holon_amd.kernels.registry import kernel_op
    k, dev, page = load_hip(), "cuda", 16
    g = torch.Generator().manual_seed(dim + 3)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)          # noqa: E731
    twin, scale = TorchKernels(), 1.5 * dim ** -0.5
    lens, counts = [700, 75, 190, 3, 129, 1, 40, 360, 181, 641], [700, 1, 60, 3, 1, 1, 2, 1, 1, 290]
    table, n_pages = _scattered(lens, page, 48, g)
    table = table.to(dev)
    qstart = [0]
    for c in counts:
        qstart.append(qstart[-1] + c)
    decode = [b for b, c in enumerate(counts) if c == 1]
    chunk_rows = [b for b, c in enumerate(counts) if c > 1]
    rows = AttnRows(slots=i32(list(range(len(lens)))), lens=i32(lens), query_start=i32(qstart), decode_rows=i32(decode),
                    chunk_rows=i32(chunk_rows), n_decode=len(decode), n_chunk=len(chunk_rows),
                    max_decode_len=max(lens[b] for b in decode), max_chunk_query=max(counts),
                    max_chunk_len=max(lens[b] for b in chunk_rows))
    token_row = torch.cat([torch.full((c,), b, dtype=torch.int32) for b, c in enumerate(counts)]).to(dev)
    positions = torch.cat([torch.arange(n - c, n, dtype=torch.int32) for n, c in zip(lens, counts)]).to(dev)
    forms = [(1, 1), (0, 2), (0, 1)] if dim != 256 else [(1, 1)]            # (copies direct or not, two tiles a wave or not)
    for heads, groups, chunk in ((8, 2, 180), (4, 4, 64), (6, 1, 33), (40, 1, 150), (2, 2, 1000), (3, 3, 1)):
        pages = (torch.randn(n_pages, 2, groups, page * dim, generator=g) * 0.5).to(dev).bfloat16()
        q = torch.randn(qstart[-1], heads, dim, generator=g).to(dev).bfloat16()
        gates = (2.0 * torch.randn(qstart[-1], heads + 7, generator=g)).to(dev).bfloat16()[:, 3: 3 + heads]
        for gate, cap in ((gates, 0.0), (None, 0.0), (gates, 4.0)):
            want = twin.paged_attention(q.double(), pages.double(), table, rows, page, scale, -chunk, softcap=cap,
                                        head_gate=None if gate is None else gate.double())
            for direct, pair in forms:
                was = k.lib.holon_attention_prefill_copies(direct), k.lib.holon_attention_prefill_form(pair)
                got = k.paged_attention(q, pages, table, rows, page, scale, -chunk, softcap=cap, head_gate=gate)
                k.lib.holon_attention_prefill_copies(was[0]), k.lib.holon_attention_prefill_form(was[1])
                assert H.rel_rms(got, want) < 8e-3, (dim, heads, groups, chunk, direct, pair, cap)
                per = ((got.double() - want).square().mean((1, 2)).sqrt() / want.square().mean().sqrt()).max().item()
                assert per < 4e-2, (dim, heads, groups, chunk, direct, pair, cap, per)
            if gate is None:
                flat = pages.view(n_pages, -1)
                for dtype, tol in ((torch.bfloat16, 8e-3), (torch.float32, 2e-6)):
                    general = k.softmax_attention(q.to(dtype), flat.to(dtype), table, rows, token_row, positions, groups, dim,
                                                  page, None, scale, -chunk)
                    assert H.rel_rms(general.view(-1, heads, dim), want) < tol, (dim, heads, groups, chunk, dtype)
                plain_form = k.paged_attention(q.float(), pages.float(), table, rows, page, scale, -chunk)   # off the cores
                assert H.rel_rms(plain_form, want) < 2e-6, (dim, heads, groups, chunk)
    # decode rows alone, in order, of every length around a chunk's edges
    lens = [179, 180, 181, 359, 360, 361, 1, 33, 640]
    table, n_pages = _scattered(lens, page, 48, g)
    rows = AttnRows(slots=i32(list(range(9))), lens=i32(lens), query_start=i32(list(range(10))), decode_rows=i32(list(range(9))),
                    chunk_rows=i32([]), n_decode=9, n_chunk=0, max_decode_len=1024, max_chunk_query=0, max_chunk_len=0,
                    in_order=True)
    for heads, groups, chunk in ((8, 2, 180), (4, 4, 32), (16, 1, 360), (2, 2, 7)):
        pages = (torch.randn(n_pages, 2, groups, page * dim, generator=g) * 0.5).to(dev).bfloat16()
        q = torch.randn(9, heads, dim, generator=g).to(dev).bfloat16()
        gates = torch.randn(9, heads, generator=g).to(dev).bfloat16()
        got = k.paged_attention(q, pages, table.to(dev), rows, page, scale, -chunk, head_gate=gates)
        want = twin.paged_attention(q.double(), pages.double(), table.to(dev), rows, page, scale, -chunk, head_gate=gates.double())
        assert H.rel_rms(got, want) < 8e-3, (dim, heads, groups, chunk)
