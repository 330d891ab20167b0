"""Falisun through the engine against the plain model (`tests/plain/falisun.py`, written from the design's equations, no
cache, float64): every mechanism alone, every way of cutting a prompt, batches, reused pages and slots, far keys and keys
at page borders, the first tokens of a sequence, what a recurrent state still holds of them long after, rows that run in
pieces and the pieces' borders, layers that read another layer's latent, the router's choice, long decoding, sizes that
are 1 or equal, and greedy generation through the engine's own entry point. On the CPU the plain twins of the operations
stand in for the HIP kernels (this checks configuration, weights, cache, state and batching); the `gpu` cases run the HIP
kernels, each also alone against its twin."""
from __future__ import annotations

import functools
import json
import pathlib

import pytest
import torch

from tests import falisun_models as M
from tests import helpers as H
from tests.plain import falisun as plain
from tests.plain.ops import TorchKernels

DEVICES = [pytest.param("cpu", id="cpu-twin"), pytest.param("cuda", marks=pytest.mark.gpu, id="hip")]
DTYPES = ["float32", "bfloat16"]
MODELS = {"A": (M.CONFIG_A, 11, False, 8), "B": (M.CONFIG_B, 12, False, 16), "C": (M.CONFIG_C, 13, False, 4),
          "A-sharp": (M.CONFIG_A, 14, True, 16), "B-sharp": (M.CONFIG_B, 15, True, 8), "D-sharp": (M.CONFIG_D, 20, True, 16),
          "latent": (M.ONLY_LATENT, 16, True, 8), "mamba": (M.ONLY_MAMBA, 17, False, 8), "moe": (M.ONLY_MOE, 19, False, 8)}
LENGTHS = (40, 70, 33, 58, 50, 64, 21)
# bfloat16 engine against the float64 plain model, relative rms of the logits: what rounding alone gives on these
# models stays well below this; a lost key, state, gate or expert is far above it.
BF16_RMS = 0.08


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("falisun")
    return {name: M.make_folder(root / name, cfg, seed, sharp) for name, (cfg, seed, sharp, _) in MODELS.items()}


@functools.lru_cache(maxsize=None)
def _plain(folder: str) -> M.PlainFalisun:
    return M.PlainFalisun(folder)


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
        routed = sum(bool(layer.get("mlp")) for layer in config["layers"])
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
@pytest.mark.parametrize("name", ["A", "B-sharp", "C", "D-sharp", "mamba"])
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
    """The residual stream after each layer, float32, against the plain model's: the block's pending term, divided by
    its own root mean square and scaled, added to its rows."""
    from holon_amd.engine.batch import StepRow
    from holon_amd.parts.base import Stream
    folder = folders["A"]
    ids = H.random_ids(37, M.CONFIG_A["vocab"], 3)
    rep = _replayer(folder, device, "float32", 8, cache_tokens=40)
    slot = rep.cache.admit()
    rep.cache.reserve(slot, len(ids))
    step, _ = rep.runner.prepare([StepRow(slot, 0, ids, [])])
    model = rep.loaded.model
    stream = Stream(model.embed(step.token_ids, step.token_take))
    want = _plain(str(folder)).streams(ids)
    assert len(want) == len(model.sites) == 5
    for site, ref in zip(model.sites, want):
        stream = model.blocks[site.layer](stream, step, site)
        d = stream.delta
        x = stream.h.double() + plain.unit(d.term.double(), d.norm.eps) * d.gain.double()
        assert H.rel_rms(x.cpu(), ref) < 2e-5, f"layer {site.layer}"


def _needle(root, kind, dims, key_at, query_at, page):
    """One layer of latent attention (`shared`: behind one that adds nothing and whose latent it reads), no feed-forward.
    A pair of token ids (query token, key token) whose score, with the key at position `key_at` and the query at
    `query_at`, is the largest of all pairs', and a filler token whose scores with them and with itself are low; the
    query side is scaled until the pair's weight among hundreds of fillers is nearly all of it. Returns the folder and
    the three ids."""
    dim, rot, rank = dims
    layers = [M.latent(2, dim, rot, 16, rank, 0.25, base=30.0, scaling=M.SHORT_YARN)]
    if kind == "shared":
        layers.append(M.latent(2, dim, rot, 16, rank, 0.25, base=30.0, scaling=M.SHORT_YARN, kv_from=0))
    cfg = M.model(32, 40, layers)
    found = {}

    def edit(t):
        at = len(layers) - 1
        if kind == "shared":
            t["l0.mix.o"] = torch.zeros_like(t["l0.mix.o"])
        p = {k: v.double() for k, v in t.items()}
        m = layers[at]["mixer"]
        kept_in = plain.unit(p["embed"], 1e-6) * p["l0.norm1"]
        a_in = plain.unit(p["embed"], 1e-6) * p[f"l{at}.norm1"]
        n = a_in.shape[0]
        q = (a_in @ p[f"l{at}.mix.q"].T).view(n, 2, dim + rot)[:, 0]
        both = kept_in @ p["l0.mix.dkv"].T
        c, r = plain.unit(both[:, :rank], 1e-6) * p["l0.mix.dkv.norm"], both[:, rank:]
        k = c @ p[f"l{at}.mix.uk"].view(2, dim, rank)[0].T
        places = query_at + 1
        q_at = plain.turn(q[None, :, dim:].expand(places, n, rot), m["rot"])[query_at]
        r_at = plain.turn(r[None].expand(places, n, rot), m["rot"])                                # [place, token, rot]
        score = ((q[:, :dim] @ k.T)[:, :, None] + torch.einsum("ad,pbd->abp", q_at, r_at)) * m["scale"]
        a, b = divmod(int(score[:, :, key_at].argmax()), n)
        worst = score[a].amax(-1)                       # a token's highest score with the query, wherever it stands
        worst[a] = worst[b] = float("inf")
        filler = int(worst.argmin())
        gain = 12.0 / max(float(score[a, b, key_at] - worst[filler]), 1e-3)      # the pair stands e^12 above any filler
        t[f"l{at}.mix.q"] = (p[f"l{at}.mix.q"] * gain).bfloat16()
        t[f"l{at}.mix.g"] = (p[f"l{at}.mix.g"] * 0.0).bfloat16()                 # every value passes by half
        found.update(a=a, b=b, filler=filler)
    folder = M.make_folder(root, cfg, 77, edit=edit)
    return folder, found["a"], found["b"], found["filler"]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,dims,page,key_at", [("own", (12, 4, 20), 8, 7), ("own", (16, 32, 96), 16, 16),
                                                   ("shared", (16, 32, 96), 16, 35), ("shared", (8, 8, 24), 8, 8),
                                                   ("own", (16, 64, 128), 16, 15)])
def test_a_far_key_at_a_page_border(tmp_path, kind, dims, page, key_at, dtype, device):
    """One key 300 tokens behind the query, the last of a page, the first of one or inside one, whose score stands out
    among hundreds: it carries the result in a whole prompt, in a prompt cut into portions (down to two tokens, the
    query in one of them), and when the query is decoded alone; without it the logits are far away."""
    query_at = key_at + 300
    folder, a, b, filler = _needle(tmp_path / "needle", kind, dims, key_at, query_at, page)
    plain_model = M.PlainFalisun(folder)
    ids = [filler] * key_at + [b] + [filler] * (query_at - key_at - 1) + [a, filler]
    without = [filler] * query_at + [a, filler]
    gap = H.rel_rms(plain_model.logits(ids)[query_at], plain_model.logits(without)[query_at])
    assert gap > 0.1, f"the far key does not show: {gap}"
    rep = _replayer(folder, device, dtype, page, cache_tokens=-(-len(ids) // page) * page, max_model_len=352)
    tol = gap / 8
    got = H.run_trace(rep, H.trace_whole({"f": ids}))
    _check(folder, dtype, {"f": ids}, got, "far key, whole")
    assert H.rel_rms(got[("f", query_at)], plain_model.logits(ids)[query_at]) < tol
    got = H.run_trace(rep, H.trace_chunks("f", ids, [150, 2, 97, query_at - 249 - 1, 2]))
    assert H.rel_rms(got[("f", query_at)], plain_model.logits(ids)[query_at]) < tol, "a portion of two"
    got = H.run_trace(rep, H.trace_decode_tail("f", ids, 3))
    _check(folder, dtype, {"f": ids}, got, "far key, decoded")
    assert H.rel_rms(got[("f", query_at)], plain_model.logits(ids)[query_at]) < tol, "decoded alone"
    got = H.run_trace(rep, H.trace_whole({"g": without}))
    assert H.rel_rms(got[("g", query_at)], plain_model.logits(without)[query_at]) < tol
    rep.cache.check()


def _long_memory(root):
    """One mamba2 layer whose decays are near one: what the first token wrote is read hundreds of tokens later."""
    cfg = M.model(32, 40, [M.mamba2(2, 16, 24, 1, 2, conv=3)])

    def edit(t):
        t["l0.mix.dt_bias"] = torch.full((2,), -1.0).bfloat16()
        t["l0.mix.A_log"] = torch.full((2,), -8.0).bfloat16()
        t["l0.mix.in"][-2:] = (4.0 * t["l0.mix.in"][-2:].float()).bfloat16()        # step sizes differ from token to token
    return M.make_folder(root, cfg, 5, edit=edit)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_a_state_that_reaches_far_and_the_pieces_borders(tmp_path, dtype, device):
    """A first token that still shows 560 tokens later; rows of that length run in pieces of 256 tokens, and portions end
    just before, at and just behind a piece's and a tile's border, so that a state is handed on at every kind of place;
    then single tokens across the same positions."""
    folder = _long_memory(tmp_path / "m")
    base = M.PlainFalisun(folder)
    ids = H.random_ids(560, 40, 9)
    other = [(ids[0] + 7) % 40] + ids[1:]
    gap = H.rel_rms(base.logits(other)[-1], base.logits(ids)[-1])
    assert gap > 3e-3, f"the first token does not show: {gap}"
    rep = _replayer(folder, device, dtype, 16, cache_tokens=560, max_model_len=560)
    for sizes in ([560], [255, 2, 303], [256, 256, 48], [257, 255, 48], [64, 63, 2, 1, 257, 173], [2, 558], [16, 15, 17, 512]):
        got = H.run_trace(rep, H.trace_chunks("x", ids, sizes))
        _check(folder, dtype, {"x": ids}, got, f"portions {sizes}")
        if dtype == "float32":
            assert H.rel_rms(got[("x", 559)], base.logits(ids)[559]) < gap / 30
    got = H.run_trace(rep, H.trace_chunks("x", ids, [250] + [1] * 12 + [298]))
    _check(folder, dtype, {"x": ids}, got, "single tokens across a piece's border")
    ids2 = H.random_ids(300, 40, 10)
    rep = _replayer(folder, device, dtype, 16, cache_tokens=1040, max_model_len=560)
    got = {}
    got.update(_steps(rep, [[("a", ids[:300]), ("b", ids2[:1])], [("a", ids[300:301]), ("b", ids2[1:290])],
                            [("b", ids2[290:291]), ("a", ids[301:])], [("b", ids2[291:])]]))
    _check(folder, dtype, {"a": ids, "b": ids2}, got, "two long rows side by side")


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


@pytest.mark.parametrize("device", DEVICES)
def test_each_mechanism_shows(folders, tmp_path, device):
    """The gate, the latent's norm, the learned scales, the norms behind the sublayers, the filter's bias, D, step sizes
    and decays, the gate and norm behind the recurrence, YaRN, the groups of the router each move the plain model's
    logits far more than the engine differs from it: a mechanism left out or mistaken would not pass the other tests."""
    ids = H.random_ids(60, 90, 4)
    flip = lambda t: t.flip(-1)                    # noqa: E731
    cases = [("latent", "l0.mix.g", lambda t: -t), ("latent", "l0.mix.dkv.norm", flip), ("latent", "l1.ls1", flip),
             ("latent", "l1.norm1b", flip), ("latent", "l1.mix.uk", lambda t: t.flip(0)), ("latent", "l2.mix.uv", lambda t: t.flip(0)),
             ("mamba", "l0.mix.conv.b", lambda t: t * 0.0), ("mamba", "l0.mix.D", lambda t: t * 0.0),
             ("mamba", "l0.mix.dt_bias", flip), ("mamba", "l1.mix.A_log", flip), ("mamba", "l0.mix.norm", flip),
             ("mamba", "l1.mix.conv", flip), ("moe", "l0.mlp.router", lambda t: t.flip(0)), ("moe", "l0.ls2", flip)]
    for name, key, change in cases:
        base = _plain(str(folders[name]))
        cfg, seed, sharp, page = MODELS[name]

        def edit(t, key=key, change=change):
            t[key] = change(t[key].float()).bfloat16()
        other = M.PlainFalisun(M.make_folder(tmp_path / f"{name}-{key}", cfg, seed, sharp, edit=edit))
        gap = H.rel_rms(other.logits(ids), base.logits(ids))
        rep = _replayer(folders[name], device, "float32", page, cache_tokens=64)
        got = H.run_trace(rep, H.trace_chunks("x", ids, [23, 2, 9]))
        g, w = H.gather({"x": base.logits(ids)}, got)
        assert gap > 5e-3 and H.rel_rms(g, w) < gap / 100, f"{name} {key}: gap {gap}"
    for name, layers, path, value in (("latent", (0, 1), ("mixer", "rot", "scaling"), None),
                                      ("latent", (0, 1), ("mixer", "rot", "scaling", "factor"), 1.5),
                                      ("latent", (1,), ("mixer", "kv_from"), None), ("mamba", (0,), ("mixer", "norm_groups"), 1),
                                      ("moe", (0,), ("mlp", "router", "groups"), None),
                                      ("moe", (0,), ("mlp", "router", "groups", "keep"), 2)):
        changed = M.variant(MODELS[name][0])
        for layer in layers:
            where = changed["layers"][layer]
            for key in path[:-1]:
                where = where[key]
            where[path[-1]] = value
        other = M.PlainFalisun(M.make_folder(tmp_path / f"{name}-{'-'.join(path)}-{value}", changed, MODELS[name][1],
                                             MODELS[name][2]))
        for key, tensor in _plain(str(folders[name])).tensors.items():         # the same weights, one key changed
            other.tensors[key] = tensor
        assert H.rel_rms(other.logits(ids), _plain(str(folders[name])).logits(ids)) > 5e-3, (name, path)


@pytest.mark.parametrize("device", DEVICES)
def test_the_router_chooses_as_the_plain_model(device):
    """The router's weights on their own: the best groups by their largest logit, the largest logits among those, equal
    ones to the lower index, weights the chosen scores divided by their sum."""
    import holon_amd.parts  # noqa: F401
    from holon_amd.kernels.registry import kernel_op
    if device == "cuda":
        from holon_amd.kernels import load_hip
        router_top = load_hip().moe_router_top
    else:
        router_top = kernel_op("moe_router_top").plain
    g = torch.Generator().manual_seed(3)
    for experts, top, width, groups, keep in ((8, 3, 64, 4, 2), (12, 4, 250, 3, 2), (6, 6, 32, 2, 2), (16, 1, 100, 16, 1),
                                              (1, 1, 8, 1, 1), (64, 6, 512, 8, 3), (130, 9, 48, 13, 2), (96, 5, 33, 1, 1)):
        x = torch.randn(50, width, generator=g).to(device)
        router = (2.0 * torch.randn(experts, width, generator=g) * width ** -0.5).to(device)
        if experts > 1:
            router[1] = router[0]                  # two experts with equal logits
        got = router_top(x, router, None, experts, top, groups, keep).cpu().double()
        z = x.double().cpu() @ router.double().cpu().T
        for t in range(50):
            chosen = plain.route(z[t], {"top": top, "groups": {"count": groups, "keep": keep}})
            want = torch.zeros(experts, dtype=torch.float64)
            for e, weight in chosen:
                want[e] = weight
            near = sorted(z[t].tolist())
            if experts > 2 and min((b - a for a, b in zip(near, near[1:]) if b != a), default=1.0) < 1e-5:
                continue                           # a call that float32 cannot make
            assert torch.allclose(got[t], want, atol=2e-6), (experts, top, t)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(folders, dtype, device):
    """180 tokens one by one after a prompt of 5, over many pages, through states and layers that read another's cache."""
    folder, page = folders["A-sharp"], 8
    ids = H.random_ids(185, M.CONFIG_A["vocab"], 21)
    rep = _replayer(folder, device, dtype, page, cache_tokens=192)
    trace = H.trace_decode_tail("d", ids, 180)
    trace.steps[-1]["end"] = []
    got = H.run_trace(rep, trace)
    _check(folder, dtype, {"d": ids}, got, f"long decoding {dtype}")
    kept = [[d.name for d in decls] for decls in rep.loaded.model.state_decls()]
    assert kept == [["conv", "S"], ["latent"], [], ["conv", "S"], []]           # two layers keep nothing of their own
    assert rep.cache.groups[0].decl.elems == 48                                 # an entry once: 40 + 8 values a token
    rep.cache.check()
    rep.step([], ["d"])
    assert all(g.pool.free == g.pool.usable for g in rep.cache.groups)


def test_configuration_and_weights_are_checked(tmp_path):
    from holon_amd.config.model import ConfigError
    from holon_amd.registry import resolve
    from holon_amd.weights.loader import WeightError
    cfg, spec = resolve(M.CONFIG_A)
    assert [(r.layer, r.reads) for r in spec.order] == [(0, None), (1, None), (2, 1), (3, None), (4, 1)]
    assert cfg.to_dict()["layers"] == M.CONFIG_A["layers"]

    def changed(layer, path, value):
        c = M.variant(M.CONFIG_A)
        where = c["layers"][layer]
        for key in path[:-1]:
            where = where[key]
        where[path[-1]] = value
        return c
    for bad in ({k: v for k, v in M.CONFIG_A.items() if k != "norm"}, M.variant(M.CONFIG_A, layers=[]),
                M.variant(M.CONFIG_A, layers=[{"type": "conv", "mixer": {}, "mlp": None}]),
                changed(2, ("mixer", "kv_from"), 3), changed(2, ("mixer", "kv_from"), 0), changed(4, ("mixer", "kv_from"), 2),
                changed(2, ("mixer", "kv_rank"), 32), changed(2, ("mixer", "rot", "base"), 50.0),
                changed(1, ("mixer", "rot", "dims"), 7), changed(1, ("mixer", "rot", "scaling", "factor"), 0),
                changed(0, ("mixer", "groups"), 4), changed(0, ("mixer", "norm_groups"), 5), changed(0, ("mixer", "state"), 0),
                changed(1, ("mlp", "router", "top"), 7), changed(1, ("mlp", "router", "groups", "count"), 5),
                changed(0, ("mlp", "kind"), "dense")):
        with pytest.raises(ConfigError):
            resolve(bad)

    def drop(t):
        del t["l1.mix.g"]
        t["l0.mix.conv.b"] = torch.zeros(5).bfloat16()
        t["l2.mix.dkv"] = torch.zeros(48, 64).bfloat16()         # a layer that reads another's latent has none
    folder = M.make_folder(tmp_path / "bad", M.CONFIG_A, 1, edit=drop)
    from holon_amd.engine.loading import load_model
    with pytest.raises(WeightError) as e:
        load_model(folder, device="cpu", dtype="float32", kernels=TorchKernels(), max_model_len=32, max_seqs=2)
    assert "l1.mix.g" in str(e.value) and "l0.mix.conv.b" in str(e.value) and "l2.mix.dkv" in str(e.value)

    def idle(t):                                                 # a layer without feed-forward may still list its norms
        t.update({name: torch.ones(64).bfloat16() for name in ("l2.norm2", "l2.norm2b", "l2.ls2")})
    load_model(M.make_folder(tmp_path / "idle", M.CONFIG_A, 1, edit=idle), device="cpu", dtype="float32",
               kernels=TorchKernels(), max_model_len=32, max_seqs=2)


@pytest.mark.parametrize("device", DEVICES)
def test_random_weights_from_the_command_line_replay(tmp_path, device):
    """`holon_amd random` writes a Falisun folder, and the engine and the plain model agree on it."""
    from holon_amd.cli import main
    (tmp_path / "c.json").write_text(json.dumps(M.CONFIG_A))
    assert main(["random", "--config", str(tmp_path / "c.json"), "--seed", "4", "--out", str(tmp_path / "m")]) == 0
    ids = H.random_ids(30, M.CONFIG_A["vocab"], 2)
    rep = _replayer(tmp_path / "m", device, "float32", 8, cache_tokens=32)
    got = H.run_trace(rep, H.trace_chunks("a", ids, [4, 9]))
    _check(tmp_path / "m", "float32", {"a": ids}, got, "random folder")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_engine(folders, dtype, device):
    """The engine's own entry point and scheduler: prompts of unequal length generated side by side, with prompt
    portions riding beside decode rows, follow the plain model's most likely token wherever that is clear."""
    from holon_amd.config import EngineConfig, SamplingParams
    from holon_amd.engine.engine import Engine
    folder = folders["B-sharp"]
    plain_model = _plain(str(folder))
    prompts = [H.random_ids(n, M.CONFIG_B["vocab"], 50 + n) for n in (5, 37, 18, 1)]
    cfg = EngineConfig(model=str(folder), device=device, dtype=dtype, page_size=8, max_seqs=3, max_model_len=96,
                       max_step_tokens=40, chunk_with_decode=16, cache_tokens=192)
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
    from holon_amd.parts.mamba2 import PIECE
    from holon_amd.parts.positions import rope_table
    k, dev = load_hip(), "cuda"
    tol = 3e-6 if dtype == torch.float32 else 6e-3
    g = torch.Generator().manual_seed(0)

    def randn(*shape, to=dtype):
        return torch.randn(*shape, generator=g).to(dev).to(to)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)          # noqa: E731
    for dim in (96, 250, 1500, 2048, 3000, 8192, 9001):      # the norm behind a sublayer, the add, the norm in front of one
        for wide in (False, True):
            x, term, w = randn(7, dim, to=torch.float32), randn(7, dim), 1 + 0.3 * randn(dim, to=torch.float32 if wide else dtype)
            gain = randn(dim, to=torch.float32)
            xa, xb = x.clone(), x.clone()
            a = k.stream_rms_post(xa, term, gain, 1e-5, w, 1e-6, dtype)
            b = kernel_op("stream_rms_post").plain(xb, term, gain, 1e-5, w, 1e-6, dtype)
            assert H.rel_rms(xa, xb) < 1e-6 and H.rel_rms(a, b) < tol, dim
    # the filter: columns of wider rows, a bias, the last inputs as a ring; rows that start and rows that continue
    counts, starts, slots = [1, 9, 2, 5, 1, 3], [0, 0, 7, 3, 12, 2], [5, 0, 3, 1, 4, 2]
    qs = [0]
    for c in counts:
        qs.append(qs[-1] + c)
    token_row = i32([b for b, c in enumerate(counts) for _ in range(c)])
    for channels, taps, extra in ((40, 4, 24), (37, 3, 11), (64, 1, 0), (24, 2, 8), (16, 7, 16)):
        wide = randn(qs[-1], channels + extra)
        x = wide[:, extra // 2: extra // 2 + channels]
        w, bias = randn(channels, taps), randn(channels)
        for ring in (False, True):
            held = randn(6, taps if ring else taps - 1, channels)
            ha, hb = held.clone(), held.clone()
            args = (i32(slots), i32(starts), i32(qs), token_row, len(counts), False, True, False, bias, ring)
            a = k.causal_conv(x, w, ha, *args)
            b = kernel_op("causal_conv").plain(x, w, hb, *args)
            assert H.rel_rms(a, b) < tol and torch.equal(ha, hb), (channels, taps, ring)
            one = (i32(slots), i32(starts), i32(list(range(7))), i32(list(range(6))), 6, False, True, True, bias, ring)
            a = k.causal_conv(x[:6], w, ha, *one)                        # single tokens: one kernel does both
            b = kernel_op("causal_conv").plain(x[:6], w, hb, *one)
            assert H.rel_rms(a, b) < tol and torch.equal(ha, hb), (channels, taps, ring, "single")
    # the recurrence: single tokens from the raw projection, and rows of every length in pieces
    for heads, groups, n, vdim, taps, pad in ((4, 2, 16, 12, 4, 3), (6, 3, 24, 8, 3, 0), (2, 1, 128, 64, 4, 14), (1, 1, 1, 1, 1, 0),
                                              (3, 1, 40, 100, 2, 5), (2, 2, 256, 160, 4, 0), (4, 1, 72, 33, 4, 1)):
        inner, channels = heads * vdim, heads * vdim + 2 * groups * n
        dt_bias, a_log, d = randn(heads, to=torch.float32) - 1, randn(heads, to=torch.float32), randn(heads, to=torch.float32)
        proj = randn(6, inner + channels + heads + pad)
        w, bias = randn(channels, taps) * 0.5, randn(channels) * 0.3
        held, S = randn(6, taps, channels), randn(6, heads, n, vdim, to=torch.float32)
        ha, hb, sa, sb = held.clone(), held.clone(), S.clone(), S.clone()
        args = (i32(slots), i32(starts), heads, groups, n, vdim)
        a = k.ssd_step(proj, w, bias, ha, dt_bias, a_log, d, sa, *args)
        b = kernel_op("ssd_step").plain(proj, w, bias, hb, dt_bias, a_log, d, sb, *args)
        assert H.rel_rms(a, b) < tol and H.rel_rms(sa, sb) < tol and torch.equal(ha, hb), (heads, groups, n, vdim)
        lens = [1, 300, 2, 64, 65, 530]
        at = [0]
        for c in lens:
            at.append(at[-1] + c)
        xbc, dts = randn(at[-1], channels), randn(at[-1], heads + 5)[:, 2: 2 + heads]
        npc = [-(-c // PIECE) for c in lens]
        base = i32([sum(npc[:b]) for b in range(len(npc))])
        rows = (i32(slots), i32(starts), i32(at), len(lens), heads, groups, n, vdim)
        sa, sb = S.clone(), S.clone()
        a = k.ssd_scan(xbc, dts, dt_bias, a_log, d, sa, *rows, (PIECE, max(npc), base, sum(npc)))
        b = kernel_op("ssd_scan").plain(xbc, dts, dt_bias, a_log, d, sb, *rows)
        assert H.rel_rms(a, b) < 3e-6 and H.rel_rms(sa, sb) < 3e-6, (heads, groups, n, vdim)
        per = ((a - b).square().mean(1).sqrt() / b.square().mean().sqrt()).max().item()
        assert per < 3e-5, (heads, groups, n, vdim, per)
    for dim, parts, extra in ((96, 2, 16), (250, 5, 3), (4096, 1, 8), (6000, 2, 0), (1500, 1500, 1), (33, 1, 2)):
        y, wide, w = randn(9, dim, to=torch.float32), randn(9, dim + extra), 1 + 0.2 * randn(dim)
        gate = wide[:, extra // 2: extra // 2 + dim]
        a = k.gated_parts_norm(y, gate, w, parts, 1e-5, dtype)
        assert H.rel_rms(a, kernel_op("gated_parts_norm").plain(y, gate, w, parts, 1e-5, dtype)) < tol, (dim, parts)
    for experts, top, width, groups, keep in ((8, 3, 256, 4, 2), (12, 4, 250, 3, 3), (64, 6, 2048, 8, 4), (100, 7, 320, 10, 3),
                                              (300, 2, 96, 2, 1), (17, 17, 1024, 1, 1)):
        x, router = randn(19, width), randn(experts, width, to=torch.float32) * 0.2
        got = k.moe_router_top(x, router, None, experts, top, groups, keep)
        want = kernel_op("moe_router_top").plain(x, router, None, experts, top, groups, keep)
        close = ((got != 0) != (want != 0)).any(1)            # rows whose choice fell the other way on a close call
        assert close.sum() <= 1 and torch.allclose(got[~close], want[~close], atol=2e-5), (experts, width)
    for heads, a_, b_, extra, t in ((4, 24, 40, 7, 9), (3, 128, 64, 0, 16), (16, 64, 128, 16, 1), (5, 20, 12, 3, 60), (2, 96, 64, 8, 200)):
        x, w, wide = randn(t, heads, a_), randn(heads, b_, a_) * a_ ** -0.5, randn(t, heads * b_ + extra)
        gate = wide[:, extra: extra + heads * b_]
        got = k.head_linear(x, w, gate=gate)
        want = kernel_op("head_linear").plain(x.double(), w.double(), None, gate)
        assert H.rel_rms(got, want) < tol, (heads, a_, b_, t)
        place = randn(t, heads, b_ + 5)
        full = place.clone()
        k.head_linear(x, w, out=full[..., :b_])
        assert H.rel_rms(full[..., :b_], kernel_op("head_linear").plain(x.double(), w.double())) < tol
        assert torch.equal(full[..., b_:], place[..., b_:])
    # a paged cache of three rows over scattered pages
    page, n_pages = 16, 40
    lens = [70, 33, 150]
    table = torch.full((4, 12), n_pages - 1, dtype=torch.int32)
    order, at = torch.randperm(n_pages - 1, generator=g).tolist(), 0
    for s, n in enumerate(lens):
        for i in range(-(-n // page)):
            table[s, i] = order[at]
            at += 1
    table = table.to(dev)
    token_row = torch.cat([torch.full((n,), i, dtype=torch.int32) for i, n in enumerate(lens)]).to(dev)
    positions = torch.cat([torch.arange(n, dtype=torch.int32) for n in lens]).to(dev)
    write_page = table[token_row.long(), (positions // page).long()].contiguous()
    write_off = (positions % page).to(torch.int32)
    for heads, dim, rot, rank, extra in ((4, 16, 8, 40, 16), (3, 8, 4, 24, 0), (1, 1, 2, 1, 5), (16, 128, 64, 192, 32)):
        width, both = rank + rot, randn(sum(lens), heads * (dim + rot) + rank + rot + extra)
        tab, cw = rope_table(256, rot, 1000.0).to(dev), 1 + 0.2 * randn(rank)
        for copies in (1, 2):
            pa = torch.zeros(n_pages, copies * page * width, device=dev, dtype=dtype)
            pb = pa.clone()
            args = (heads, dim, rot, rank, cw, 1e-6, tab, positions)
            a = k.latent_rope_prepare(both, *args, pa, write_page, write_off, page, copies=copies)
            b = kernel_op("latent_rope_prepare").plain(both, *args, pb, write_page, write_off, page, copies=copies)
            assert H.rel_rms(pa, pb) < tol and torch.equal(a[0], b[0]) and H.rel_rms(a[1][..., rank:], b[1][..., rank:]) < tol
        only_q = both[:, : heads * (dim + rot)].contiguous()
        c = k.latent_rope_prepare(only_q, heads, dim, rot, rank, None, 0.0, tab, positions, None, None, None, page)
        assert torch.equal(c[0], a[0]) and torch.equal(c[1][..., rank:], a[1][..., rank:]), "queries alone"


@pytest.mark.gpu
@pytest.mark.parametrize("rank,rot", [(128, 16), (96, 32), (512, 64), (192, 64), (40, 24), (256, 64), (60, 4), (384, 64)])
def test_latent_entries_on_the_gpu(rank, rot):
    """Attention over entries kept once: in bfloat16 the matrix-core prompt and decode kernels, in both types the general
    kernel, prompt portions beside decode rows over scattered pages, head counts that fill tiles of 16 and that do not, a
    row of every length around a tile's border, with and without a sink, against float64."""
    import holon_amd.parts  # noqa: F401
    from holon_amd.kernels import load_hip
    from holon_amd.kernels.api import AttnRows
    from holon_amd.kernels.registry import kernel_op
    from holon_amd.parts.softmax_attention import latent_on_cores
    k, dev, width = load_hip(), "cuda", rank + rot
    assert latent_on_cores(width, rank) == bool(k.lib.holon_latent_cores_supported(width, rank))
    g = torch.Generator().manual_seed(rank)
    lens, counts = [300, 75, 190, 3, 129, 1, 40, 64, 65, 700, 31], [300, 1, 60, 3, 1, 1, 2, 1, 1, 1, 31]
    qstart = [0]
    for c in counts:
        qstart.append(qstart[-1] + c)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)          # noqa: E731
    decode = [b for b, c in enumerate(counts) if c == 1]
    chunk = [b for b, c in enumerate(counts) if c > 1]
    rows = AttnRows(slots=i32(list(range(len(lens)))), lens=i32(lens), query_start=i32(qstart), decode_rows=i32(decode),
                    chunk_rows=i32(chunk), n_decode=len(decode), n_chunk=len(chunk),
                    max_decode_len=max(lens[b] for b in decode), max_chunk_query=max(counts),
                    max_chunk_len=max(lens[b] for b in chunk))
    token_row = torch.cat([torch.full((c,), b, dtype=torch.int32) for b, c in enumerate(counts)]).to(dev)
    positions = torch.cat([torch.arange(n - c, n, dtype=torch.int32) for n, c in zip(lens, counts)]).to(dev)
    op = kernel_op("latent_attention").plain
    for heads, page in ((16, 16), (3, 16), (20, 32), (1, 8), (8, 64)):
        n_pages = sum(-(-n // page) for n in lens) + 1
        table = torch.full((len(lens) + 1, 96), n_pages - 1, dtype=torch.int32)
        order, at = torch.randperm(n_pages - 1, generator=g).tolist(), 0
        for s_, n in enumerate(lens):
            for i in range(-(-n // page)):
                table[s_, i] = order[at]
                at += 1
        table = table.to(dev)
        pages = torch.randn(n_pages, page * width, generator=g).to(dev).bfloat16()
        for s_, n in enumerate(lens):              # what lies behind a row's last token in its page must not be read
            if n % page:
                pages.view(n_pages, page, width)[int(table[s_, n // page]), n % page:] = float("nan")
        pages.view(n_pages, page, width)[n_pages - 1] = float("nan")
        q = (torch.randn(qstart[-1], heads, width, generator=g) * 2.5 * width ** -0.5).to(dev).bfloat16()
        sinks = [None, torch.randn(heads, generator=g).to(dev)]
        for sink in sinks[: 2 if heads in (3, 16) else 1]:
            args = (table, rows, token_row, positions, rank, page)
            want = op(q.double(), pages.double(), *args, None if sink is None else sink.double(), 0.9, 0)
            for what, got, tol in (("cores", k.latent_attention(q, pages, *args, sink, 0.9, 0), 6e-3),
                                   ("general", k.latent_attention(q, pages, *args, sink, 0.9, 4096), 6e-3),
                                   ("float32", k.latent_attention(q.float(), pages.float(), *args, sink, 0.9, 0), 2e-6)):
                assert torch.isfinite(got).all(), (heads, page, what)
                assert H.rel_rms(got, want) < tol, (heads, page, what)
                per = ((got.double() - want).square().mean((1, 2)).sqrt() / want.square().mean((1, 2)).sqrt()).max().item()
                assert per < 5 * tol, (heads, page, what, per)
    window = 33                                    # a window: the general kernel
    got = k.latent_attention(q, pages, table, rows, token_row, positions, rank, page, None, 0.9, window)
    assert H.rel_rms(got, op(q.double(), pages.double(), table, rows, token_row, positions, rank, page, None, 0.9, window)) < 6e-3
