"""Nuzinex on the GPU against the plain float64 implementation (plain_nuzinex): every mechanism alone (kernels and one-layer
models), whole prompts against token-by-token decoding and against portions down to two tokens, batches of unequal requests
against each alone with pages and slots that are used again, a key made to stand out far back, at page borders and just
inside and just outside every window (its own layer's and a reader's of its cache), in prompts and in decoding, memories that do not
fade, the first tokens, long decoding, and greedy generation through the engine."""

import json
import math
from pathlib import Path

import numpy as np
import pytest
import torch

import bitwise_amd as bw
import plain_nuzinex as pn

pytestmark = pytest.mark.gpu

# float32: 32-bit sums against float64 ones, a few 1e-6 of a row.  bfloat16: activations rounded where the products and the
# cache take them, carried through the layers; a row whose sublayer nearly cancels is blown up by the norm behind it, its
# roundings with it, so in that mode the 90th percentile carries the tight bound.
TOL = {"float32": 2e-5, "bfloat16": 0.06}
MOST = {"float32": 1.0, "bfloat16": 0.9}
TYPICAL = {"float32": 3e-6, "bfloat16": 3e-2}
SIGMA = 0.15


def att(heads, kv_heads, dim, vdim, scale, dims, base=1000.0, window=None, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": dims}}
    if window is not None:
        m["mask"] = {"size": window}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def attention(*args, ff=None, **kw):
    return {"type": "attention", "mixer": att(*args, **kw), "mlp": ff and {"kind": "dense", "ff": ff}}


def parallel(left, heads, kv_heads, dim, vdim, conv, scales=(0.6, 0.9), ff=None):
    return {"type": "parallel", "mlp": ff and {"kind": "dense", "ff": ff},
            "mixer": {"left": left, "right": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv},
                      "left_scale": scales[0], "right_scale": scales[1]}}


def lightning(heads, dim, vdim, decay=None, ff=None):
    decay = decay or [1.0 - 0.5 ** (1 + 7 * (h + 1) / heads) for h in range(heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}, "mlp": ff and {"kind": "dense", "ff": ff}}


def config(width, vocab, eps, side, layers, max_positions=1024):
    return {"architecture": "Nuzinex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "token_side": {"dim": side},
            "layers": layers, "max_positions": max_positions}


CONFIGS = {
    # one mechanism each
    "only_attention": config(48, 61, 1e-5, 8, [attention(4, 2, 16, 16, 0.3, 16, window=21)]),
    "only_parallel": config(48, 61, 1e-5, 8, [parallel(att(4, 2, 16, 16, 0.3, 8), 4, 2, 16, 24, 4)]),
    "only_lightning": config(48, 61, 1e-5, 8, [lightning(4, 16, 24)]),
    "only_dense": config(48, 61, 1e-5, 8, [lightning(1, 8, 8, ff=72)]),
    "only_side": config(48, 61, 1e-5, 40, [lightning(1, 8, 8), lightning(2, 8, 8)]),
    # caches shared between layers: readers with narrower, wider and no windows, two readers of one cache
    "shared": config(56, 67, 1e-5, 16, [
        attention(4, 2, 16, 8, 0.4, 8, window=13), attention(2, 2, 16, 8, 0.3, 8, window=29, kv_from=0),
        attention(3, 1, 8, 24, 0.3, 8, window=18), attention(6, 2, 16, 8, 0.5, 8, window=5, kv_from=0),
        attention(5, 1, 8, 24, 0.2, 8, kv_from=2)]),
    # sizes that are no multiples of 8 anywhere: every product stays on the 32-bit kernels in bfloat16 mode too; one value
    # channel a head, odd heads, nothing rotated, a convolution over one token (no state of its own) and over eight, a side
    # input of one column, heads that all share one key and that share none, decays of 0 and 1
    "odd": config(44, 53, 1e-5, 1, [
        attention(3, 3, 10, 5, 0.3, 6, window=7, base=77.0, ff=37), parallel(att(5, 1, 7, 9, 0.3, 0), 6, 3, 70, 1, 1, (1.0, -0.5), ff=13),
        lightning(3, 9, 7, [0.0, 1.0, 0.9]), parallel(att(2, 2, 6, 11, 0.4, 2), 5, 5, 9, 13, 8, (0.3, 1.7)),
        attention(6, 3, 10, 5, 0.4, 6, window=12, base=77.0, kv_from=0)]),
    # everything together, sizes all different from layer to layer: windows that are no multiple of a page, one key head and as
    # many as query heads, wholly and partly rotated heads, values wider and narrower than keys, a window on the left branch
    "mixed": config(64, 131, 1e-6, 24, [
        attention(6, 2, 24, 16, 0.25, 24, base=1e4, window=37, ff=88),
        parallel(att(4, 4, 12, 20, 0.3, 8, base=2e5), 6, 2, 16, 40, 4, (0.7, 0.4), ff=56),
        lightning(5, 16, 8),
        attention(4, 2, 24, 16, 0.3, 24, base=1e4, window=50, kv_from=0),
        parallel(att(6, 1, 32, 32, 0.2, 32, base=500.0, window=45), 2, 2, 40, 24, 2, (0.5, 1.2)),
        lightning(2, 40, 48, ff=120),
        attention(8, 8, 8, 8, 0.4, 4, window=16, ff=40),
    ]),
    # heads of the sizes real models have (64, 128, 256), windows longer than a block of keys, inner sizes beyond one step of the
    # products, four query heads a key
    "wide": config(136, 77, 1e-5, 64, [
        attention(4, 1, 128, 128, 0.09, 128, base=5e5, window=140, ff=264),
        parallel(att(4, 2, 64, 128, 0.12, 32, base=8e4), 4, 2, 128, 64, 4, ff=136),
        lightning(2, 128, 256),
        parallel(att(2, 1, 128, 64, 0.1, 64), 3, 1, 256, 128, 3, (1.0, 1.0)),
    ]),
}
SEEDS = {name: 131 + i for i, name in enumerate(CONFIGS)}


@pytest.fixture(scope="module")
def folders(tmp_path_factory, gpu):
    tmp = tmp_path_factory.mktemp("nuzinex")
    return {name: bw.write_random_model(tmp / name, cfg, SEEDS[name], SIGMA) for name, cfg in CONFIGS.items()}


def weights(folder):
    from safetensors.torch import load_file
    return pn.to64(load_file(str(Path(folder) / "model.safetensors")))


def tokens_for(name, n, seed=0):
    g = torch.Generator().manual_seed(6000 + seed)
    return torch.randint(0, CONFIGS[name]["vocab"], (n,), generator=g).tolist()


_plain = {}


def plain(folder, toks):
    key = (str(folder), tuple(toks))
    if key not in _plain:
        _plain[key] = pn.forward(json.loads((Path(folder) / "config.json").read_text()), weights(folder), toks).numpy()
    return _plain[key]


def close(got, want, dtype):
    worst, most, typical = (pn.logits_error(got, want, q) for q in (1.0, MOST[dtype], 0.5))
    print(f"{dtype}: worst row {worst:.2e}, most {most:.2e}, median {typical:.2e}")
    return worst < 0.6 and most < TOL[dtype] and typical < TYPICAL[dtype]


def replayer(folder, dtype, max_tokens, **kw):
    from bitwise_amd.replay import Replayer
    return Replayer(str(folder), dtype, max_tokens, max_live=4, **kw)


def run_cut(rp, rid, toks, cuts):
    """One request through a replayer in portions of the given sizes (the rest one by one); logits at every position."""
    out, at = [], 0
    for n in list(cuts) + [1] * (len(toks) - sum(cuts)):
        out.append(rp.step([{"id": rid, "tokens": toks[at:at + n], "want": list(range(n))}]))
        at += n
    rp.step([], [rid])
    return np.concatenate(out)


# ----------------------------------------------------------------------------- the model against the plain one

@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompts_equal_plain(folders, name, dtype):
    model = bw.Model.load(folders[name], dtype)
    for n, seed in ((1, 0), (2, 1), (37, 2), (130, 3)):
        toks = tokens_for(name, n, seed)
        assert close(model.logits(toks), plain(folders[name], toks), dtype), (name, n)
    assert model.weight_bytes > 0 and model.config.width == CONFIGS[name]["width"]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["shared", "mixed", "odd", "wide"])
def test_decoding_and_portions_equal_the_whole_prompt(folders, name, dtype):
    """Token by token from the first token on, a prompt then single tokens, and portions down to two tokens whose edges
    fall inside pages and inside windows: every position stays what the plain model says, with graphs and without, and
    all ways of cutting leave the same bits."""
    toks = tokens_for(name, 83, 5)
    want = plain(folders[name], toks)
    cuttings = ([83], [], [51], [2, 2, 3, 16, 17, 2, 30, 5], [15, 1, 1, 33, 2], [64, 2])
    first = None
    for graphs in (True, False):
        rp = replayer(folders[name], dtype, 256, use_graphs=graphs, poison_freed_pages=True)
        for k, cuts in enumerate(cuttings):
            got = run_cut(rp, f"r{k}", toks, cuts)
            assert close(got, want, dtype), (name, graphs, cuts)
            first = got if first is None else first
            assert np.array_equal(got, first), (name, graphs, cuts, pn.logits_error(got, first))
        assert rp.manager.all_free()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_portions_in_parallel_passes(folders, dtype):
    """With the engine's leave to let logits depend on the cut in their last bits, portions of 96 rows and more run the
    memories that fade in three passes over chunks (delta memories walk on): the same values to rounding, alone and beside
    short portions."""
    name = "mixed"
    toks, other = tokens_for(name, 230, 6), tokens_for(name, 40, 8)
    want, want_other = plain(folders[name], toks), plain(folders[name], other)
    rp = replayer(folders[name], dtype, 512, exact_cuts=False)
    assert close(run_cut(rp, "a", toks, [230]), want, dtype)
    assert close(run_cut(rp, "b", toks, [100, 3, 127]), want, dtype)
    lg = rp.step([{"id": "c", "tokens": toks[:200], "want": list(range(200))}, {"id": "d", "tokens": other, "want": list(range(40))}])
    assert close(lg[:200], want[:200], dtype) and close(lg[200:], want_other, dtype)
    lg = rp.step([{"id": "c", "tokens": toks[200:], "want": list(range(30))}], ["c", "d"])
    assert close(lg, want[200:], dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_requests_together_equal_each_alone(folders, dtype):
    """Four live requests of different lengths, portions beside single tokens, requests that pause, end and are followed
    by others in the same slots and pages (freed pages are filled with NaN at once): every position as alone, bit for
    bit, so also what the slots keep between steps (the convolutions' inputs, both kinds of memory) and what windows keep."""
    name = "mixed"
    lengths = {"a": 70, "b": 9, "c": 33, "d": 1, "e": 48, "f": 21}
    toks = {r: tokens_for(name, n, 20 + i) for i, (r, n) in enumerate(lengths.items())}
    rp = replayer(folders[name], dtype, 64 * 4, poison_freed_pages=True)
    plan = [
        [("a", 17), ("b", 2), ("c", 5), ("d", 1)],
        [("a", 1), ("b", 1), ("c", 16)],
        [("a", 30), ("b", 6), ("e", 2)],             # d has ended: e takes its slot; c pauses
        [("a", 1), ("c", 12), ("e", 31), ("f", 3)],  # b has ended
        [("a", 21), ("e", 1), ("f", 18)],
        [("e", 14)],
    ]
    at = {r: 0 for r in toks}
    got = {r: [] for r in toks}
    slots_used = {}
    for step in plan:
        entries, ends = [], []
        for r, n in step:
            entries.append({"id": r, "tokens": toks[r][at[r]:at[r] + n], "want": list(range(n))})
            at[r] += n
            if at[r] == lengths[r]:
                ends.append(r)
        lg = rp.step(entries, [])
        for r in (e["id"] for e in entries):
            slots_used[r] = rp.live[r].slot
        row = 0
        for r, n in step:
            got[r].append(lg[row:row + n])
            row += n
        rp.step([], ends)
    assert at == lengths and rp.manager.all_free()
    assert len(set(slots_used.values())) < len(slots_used), "slots were meant to be used again"
    solo = replayer(folders[name], dtype, 128)
    for r in toks:
        assert close(np.concatenate(got[r]), plain(folders[name], toks[r]), dtype), r
        assert np.array_equal(np.concatenate(got[r]), run_cut(solo, r, toks[r], [lengths[r]])), r


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(folders, dtype):
    """250 tokens one by one behind a short prompt, across many pages and windows, then most of it as one portion: the
    kernels of prompt portions and those of single tokens leave the same bits."""
    name = "wide"
    toks = tokens_for(name, 280, 7)
    rp = replayer(folders[name], dtype, 320)
    got = run_cut(rp, "x", toks, [30])
    assert close(got, plain(folders[name], toks), dtype)
    assert np.array_equal(run_cut(rp, "y", toks, [250]), got)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine(folders, dtype):
    """bw.generate with the engine's scheduler, a small token budget and a small page pool: the tokens of the plain
    implementation, which recomputes the whole sequence for every token; crowded and alone give the same tokens."""
    name = "mixed"
    cfg, w = CONFIGS[name], weights(folders[name])
    model = bw.Model.load(folders[name], dtype)
    prompts = [tokens_for(name, n, 40 + n) for n in (1, 6, 19, 40)]
    sp = bw.SamplingParams(max_new_tokens=10, ignore_eos=True)
    results = bw.generate(model, prompts, sp, bw.EngineConfig(num_blocks=16, max_batched_tokens=24, max_num_seqs=3, dtype=dtype))
    for p, r in zip(prompts, results):
        assert r.finished and len(r.tokens) == 10
        if dtype == "float32":
            assert r.tokens == pn.generate_greedy(cfg, w, p, 10)
        solo = bw.generate(model, [p], sp, bw.EngineConfig(num_blocks=16, max_num_seqs=1, dtype=dtype, use_graphs=False))[0]
        assert solo.tokens == r.tokens and solo.logits_fingerprint == r.logits_fingerprint


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decode_phases_leave_the_same_tokens(folders, dtype):
    """The decode products held back to run as phases of one launch: nothing of this design overtakes what waits."""
    model = bw.Model.load(folders["mixed"], dtype)
    prompts = [tokens_for("mixed", n, 60 + n) for n in (3, 21)]
    sp = bw.SamplingParams(max_new_tokens=12, ignore_eos=True)
    a, b = (bw.generate(model, prompts, sp, bw.EngineConfig(num_blocks=24, max_num_seqs=2, dtype=dtype, decode_phases=f)) for f in (False, True))
    assert [r.tokens for r in a] == [r.tokens for r in b] and [r.logits_fingerprint for r in a] == [r.logits_fingerprint for r in b]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_randomized_scenarios(gpu, dtype):
    """The scenario simulator on the architecture's tiny model: every request against its solo run, no page or slot
    lost; preemption happens on the way and restarts from a cleared slot."""
    from bitwise_amd.registry import ARCHITECTURES
    from bitwise_amd.sim import Simulator

    model = bw.Model.random(ARCHITECTURES["Nuzinex"].tiny_config, 47, dtype, sigma=0.08)
    tally = Simulator(model, dtype).run(12, seed=3)
    print(tally.line(dtype))
    assert tally.violations() == 0, "\n".join(tally.notes[:10])
    assert tally.requests_compared > 30 and tally.prefix_hit_tokens == 0


# ----------------------------------------------------------------------------- one key made to stand out

A, B, FILLER = 7, 11, 3


def needle_model(tmp, windows, tag, on_left=False):
    """Layers of attention whose token rows are unit vectors: token A alone makes a key and a value, token B alone a query, in
    elements that are not rotated, with a scale that makes their score large: what a B sees of an A decides its logits.
    ``windows``: of the layer that owns the cache and, if there are two, of the layer that reads it (the first one's output
    and every feed-forward and side input are zero then).  ``on_left``: the left branch of a parallel layer instead."""
    from safetensors.torch import load_file, save_file
    width, vocab, heads, dim = 64, 40, 2, 16
    m = lambda w, **kw: att(heads, 1, dim, dim, 1.0, 8, window=w, **kw)
    if on_left:
        layers = [parallel(m(windows[0]), 2, 1, 8, 8, 3, (1.0, 0.0))]
    else:
        layers = [attention(heads, 1, dim, dim, 1.0, 8, window=w, kv_from=None if i == 0 else 0) for i, w in enumerate(windows)]
    for L in layers:
        (L["mixer"]["left"] if on_left else L["mixer"])["scale"] = 14.0 / math.sqrt(dim * heads * dim)
    cfg = config(width, vocab, 1e-6, 8, layers, max_positions=2048)
    folder = bw.write_random_model(Path(tmp) / f"needle_{tag}", cfg, 77, 0.3)
    w = load_file(str(Path(folder) / "model.safetensors"))
    w["embed"] = torch.eye(vocab, width).to(torch.bfloat16)
    direction = torch.zeros(dim)
    direction[8:] = torch.randn(8, generator=torch.Generator().manual_seed(5))
    direction = (direction / direction.norm()).to(torch.bfloat16)
    for i in range(len(layers)):
        mix = f"l{i}.mix." + ("left." if on_left else "")
        for n in list(w):
            if n.startswith(mix) and n.endswith(".b"):
                w[n] = torch.zeros_like(w[n])
        w[f"l{i}.side.proj"] = torch.zeros_like(w[f"l{i}.side.proj"])
        w[mix + "q.norm"] = torch.ones_like(w[mix + "q.norm"])
        w[mix + "q"] = torch.zeros_like(w[mix + "q"])
        for h in range(heads):
            w[mix + "q"][dim * h:dim * h + dim, B] = direction
        if i == 0:
            w[mix + "k.norm"] = torch.ones_like(w[mix + "k.norm"])
            w[mix + "k"] = torch.zeros_like(w[mix + "k"])
            w[mix + "k"][:, A] = direction
            v = torch.zeros_like(w[mix + "v"])
            v[:, A] = torch.randn(dim, generator=torch.Generator().manual_seed(6)).to(torch.bfloat16)
            v[:, FILLER] = 0.05
            w[mix + "v"] = v
        if i + 1 < len(layers):
            w[mix + "o"] = torch.zeros_like(w[mix + "o"])
    save_file(w, str(Path(folder) / "model.safetensors"))
    return folder, cfg


# a window in one block of keys, one that ends at a page, one of several blocks, one longer than the sequence; a reader that
# looks further back, and less far, than the layer whose cache it reads, and one without a window; the left branch, which
# sees everything
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("windows,on_left", [((37,), False), ((48,), False), ((129,), False), ((300,), False), ((40, 70), False),
                                             ((70, 33), False), ((20, None), False), ((None,), True), ((50,), True)])
def test_a_key_that_stands_out(tmp_path_factory, gpu, dtype, windows, on_left):
    """One key answers a later query with a large score: far back, at page borders (pages of 16), at blocks of 64 and 128
    keys, as the first token, and just inside and just outside the query's window, in a prompt and in decoding.  The
    test first makes sure, with the plain model, that seeing the key or not moves the logits by far more than the tolerance."""
    folder, cfg = needle_model(tmp_path_factory.mktemp("needle"), windows, f"{windows}_{on_left}".replace(" ", ""), on_left)
    w = weights(folder)
    n = 300
    W = windows[-1] or n
    # (key position, query position): far back, around page and block borders, the first token, around the window's edge
    cases = [(0, n - 1), (0, W - 1), (0, W), (1, W), (1, W + 1), (15, 15 + W - 1), (16, 16 + W - 1), (16, 16 + W), (17, 17 + W),
             (200 - W, 199), (200 - W, 200), (250, 250 + W - 1), (250, 250 + W), (239, 240), (127, 128), (127, 127 + W - 1), (128, 128 + W - 1),
             (128, 128 + W), (63, 64), (3, 290)]
    cases = sorted({(k, q) for k, q in cases if 0 <= k < q < n})
    seen = unseen = 0
    rp = replayer(folder, dtype, 320, poison_freed_pages=True)
    for i, (kpos, qpos) in enumerate(cases):
        toks = [FILLER] * n
        toks[kpos], toks[qpos] = A, B
        want = pn.forward(cfg, w, toks[:qpos + 1]).numpy()
        base = [FILLER] * (qpos + 1)
        base[qpos] = B
        without = pn.forward(cfg, w, base).numpy()
        sees = qpos - kpos < W
        moved = pn.logits_error(want[qpos:], without[qpos:])
        assert (moved > 0.2) == sees, (kpos, qpos, moved)
        seen, unseen = seen + sees, unseen + (not sees)
        # as a prompt, and with the query (and what lies behind the key) decoded token by token
        for cuts in ([n], [kpos + 1], [max(qpos - 3, 1), 2]):
            got = run_cut(rp, f"n{i}", toks, cuts)
            assert pn.logits_error(got[:qpos + 1], want, 1.0) < TOL[dtype], (kpos, qpos, cuts)
    assert seen >= 5 and (unseen >= 4 or W >= n)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["delta", "lightning"])
def test_memories_that_do_not_fade(tmp_path_factory, gpu, dtype, kind):
    """Decays pushed to 1 (and, for the delta memory, small step sizes, so that later writes do not overwrite): the first
    token still moves the logits 250 tokens later (the plain model says so), through prompts, portions and decoding."""
    from safetensors.torch import load_file, save_file
    if kind == "delta":
        cfg = config(48, 61, 1e-5, 8, [parallel(att(2, 1, 16, 16, 1.0, 8, window=3), 4, 2, 24, 16, 4, (0.0, 1.0))])
    else:
        cfg = config(48, 61, 1e-5, 8, [lightning(3, 24, 16, [1.0, 1.0, 0.9999])])
    folder = bw.write_random_model(tmp_path_factory.mktemp("memory") / kind, cfg, 5, 0.3)
    w = load_file(str(Path(folder) / "model.safetensors"))
    if kind == "delta":
        w["l0.mix.right.A_log"] = torch.full_like(w["l0.mix.right.A_log"], -14.0)          # exp(-exp(-14) softplus) is 1 - 8e-7 softplus
        w["l0.mix.right.b"] = w["l0.mix.right.b"] * 0 - 0.05
    save_file(w, str(Path(folder) / "model.safetensors"))
    w64 = pn.to64(w)
    n = 260
    toks = tokens_for("only_parallel", n, 3)
    other = [(toks[0] + 1) % 61] + toks[1:]
    want, want_other = pn.forward(cfg, w64, toks).numpy(), pn.forward(cfg, w64, other).numpy()
    assert pn.logits_error(want[-5:], want_other[-5:], 0.0) > 5e-4, "the first token was meant to matter at the end"
    rp = replayer(folder, dtype, 320)
    for cuts in ([n], [1], [200, 2, 50], [17, 100]):
        assert close(run_cut(rp, "m", toks, cuts), want, dtype), cuts
    rp = replayer(folder, dtype, 320, exact_cuts=False)
    assert close(run_cut(rp, "m", toks, [n]), want, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_side_input_and_scale_matter(folders, dtype):
    """Two tokens with one embedding row and different side rows end in different logits; the engine follows (a side table
    that is read at the wrong columns, or left out, would not)."""
    from safetensors.torch import load_file, save_file
    name = "only_side"
    folder = Path(folders[name]).parent / "side_probe"
    folder.mkdir(exist_ok=True)
    (folder / "config.json").write_text((Path(folders[name]) / "config.json").read_text())
    w = load_file(str(Path(folders[name]) / "model.safetensors"))
    w["embed"][9] = w["embed"][4]
    w["side.embed"][9, :40] = w["side.embed"][4, :40]               # alike for the first layer, different for the second
    save_file(w, str(folder / "model.safetensors"))
    w64 = pn.to64(w)
    a, b = [1, 4, 2, 4], [1, 9, 2, 4]
    want_a, want_b = pn.forward(CONFIGS[name], w64, a).numpy(), pn.forward(CONFIGS[name], w64, b).numpy()
    assert pn.logits_error(want_b[1:2], want_a[1:2]) > 0.1
    model = bw.Model.load(folder, dtype)
    for t, want in ((a, want_a), (b, want_b)):
        assert close(model.logits(t), want, dtype)


# ----------------------------------------------------------------------------- kernels alone

def _dev(gpu):
    return lambda x: torch.tensor(x, dtype=torch.int32, device=gpu)


@pytest.mark.parametrize("key_heads,heads,dim,vdim,taps", [(2, 4, 16, 24, 4), (1, 3, 70, 9, 2), (3, 3, 128, 64, 8), (2, 2, 200, 5, 3), (5, 5, 7, 1, 1)])
def test_what_a_delta_memory_reads_against_plain(gpu, key_heads, heads, dim, vdim, taps):
    """Convolution with SiLU, unit queries and keys, step sizes and decays in one launch, through portions and slots that
    change hands; the bits do not depend on the cut."""
    from bitwise_amd.csrc import ops
    g = torch.Generator().manual_seed(dim)
    dev = _dev(gpu)
    qk, n = key_heads * dim, 40
    channels = 2 * qk + heads * vdim
    wc, rate, bias = torch.randn(channels, taps, generator=g), torch.rand(heads, generator=g) * 2, torch.randn(heads, generator=g)
    seqs = [torch.randn(n, channels + 2 * heads, generator=g) for _ in range(3)]
    want = []
    for s in seqs:
        u = pn.silu(pn.causal_convolution(s[:, :channels].double(), wc.double()))
        q, k = (pn.unit(t.view(n, key_heads, dim)) for t in (u[:, :qk], u[:, qk:2 * qk]))
        u = torch.cat([(q * dim ** -0.5).reshape(n, qk), k.reshape(n, qk), u[:, 2 * qk:]], 1)
        beta = torch.sigmoid(s[:, channels + heads:].double())
        decay = torch.exp(-rate.double() * pn.softplus(s[:, channels:channels + heads].double() + bias.double()))
        want.append((u, torch.cat([beta, decay, (q * k).sum(-1) * dim ** -0.5], 1)))

    def run(steps):
        state = torch.full((2, max(1, (taps - 1) * channels) + 3), float("nan"), device=gpu)
        at, slot_of, got = [0, 0, 0], {0: 0, 1: 1, 2: 0}, [[], [], []]
        for step in steps:
            x, pos, seq_rows, slots = [], [], [], []
            for r, m in step:
                if at[r] == 0:
                    state[slot_of[r]].zero_()
                seq_rows += [len(pos), m]
                x.append(torch.cat([torch.zeros(m, 2), seqs[r][at[r]:at[r] + m]], 1))
                pos += list(range(at[r], at[r] + m))
                slots.append(slot_of[r])
            xd = torch.cat(x).to(gpu)[:, 2:]
            out, gates = torch.zeros(len(pos), channels, device=gpu), torch.zeros(len(pos), 2 * heads + key_heads, device=gpu)
            ops.conv_heads(xd, wc.to(gpu), state[:, 3:] if taps > 1 else None, xd, channels, channels + heads, bias.to(gpu), rate.to(gpu),
                           key_heads, dim, dev(seq_rows), dev(slots), dev(pos), len(step), max(m for _, m in step), out, gates, dim ** -0.5, 1e-6)
            o = 0
            for r, m in step:
                got[r].append(torch.cat([out[o:o + m], gates[o:o + m]], 1).cpu())
                o += m
                at[r] += m
        assert at == [n, n, n]
        return [torch.cat(t) for t in got]

    a = run([[(0, 5), (1, 1)], [(1, 2), (0, 1)], [(0, 34), (1, 1)], [(1, 36), (2, 3)], [(2, 1)], [(2, 36)]])
    b = run([[(0, n)], [(1, n), (2, n)]])
    for r in range(3):
        assert torch.equal(a[r], b[r]), r
        assert (a[r].double() - torch.cat(want[r], 1)).abs().max() < 2e-5, r


@pytest.mark.parametrize("heads,key_heads,dim,vdim", [(4, 2, 16, 16), (6, 2, 20, 12), (2, 1, 64, 128), (3, 3, 128, 64), (2, 2, 200, 24), (5, 1, 9, 1)])
def test_delta_recurrence_against_plain(gpu, heads, key_heads, dim, vdim):
    """The memory alone, with step sizes near 1 on keys that come again (so that replacing and adding differ): whole
    sequences and portions that continue from the slot (bit for bit alike)."""
    from bitwise_amd.csrc import ops
    g = torch.Generator().manual_seed(heads * 100 + dim)
    T, hv, qk = 150, heads * vdim, key_heads * dim
    keys = pn.unit(torch.randn(5, key_heads, dim, generator=g).double()).float()
    k = keys[torch.randint(0, 5, (T,), generator=g)].reshape(T, qk) + 0.01 * torch.randn(T, qk, generator=g)
    q, v = torch.randn(T, qk, generator=g), torch.randn(T, hv, generator=g)
    beta, decay = torch.rand(T, heads, generator=g), 0.9 + 0.1 * torch.rand(T, heads, generator=g)
    want = pn.delta_recurrence(q.double().view(T, key_heads, dim), k.double().view(T, key_heads, dim), v.double().view(T, heads, vdim),
                               decay.double(), beta.double())
    dev = _dev(gpu)
    kq = (k.double() * q.double()).view(T, key_heads, dim).sum(-1).float()
    u, gates = torch.cat([q, k, v], 1).to(gpu), torch.cat([beta, decay, kq], 1).to(gpu)
    positions = dev(list(range(T)))

    def run(cuts):
        state = torch.zeros(2, heads * dim * vdim + 3, device=gpu)[:, 3:]           # (a column slice, as a shared slot gives it)
        out, at = torch.zeros(T, hv, device=gpu), 0
        for n in cuts:
            rows = slice(at, at + n)
            o = torch.zeros(n, hv, device=gpu)
            ops.linear_recurrence(ops.RECUR_DELTA, u[rows], 0, qk, 2 * qk, gates[rows], 0, heads, None, None, 0.0, 1.0, state, o, dev([0, n]),
                                  dev([1]), positions[rows].contiguous(), 1, heads, dim, vdim, heads_per_key=heads // key_heads,
                                  few_rows=n <= 2)
            out[rows] = o
            at += n
        return out

    whole = run([T])
    assert (whole.cpu().double().view(T, heads, vdim) - want).abs().max() / want.abs().max() < 3e-5
    for cuts in ([1] * T, [7, 64, 2, 77]):
        assert torch.equal(run(cuts), whole), cuts
    with pytest.raises(ValueError):
        ops.linear_recurrence(ops.RECUR_DELTA, u, 0, qk, 2 * qk, gates, 0, heads, None, None, 0.0, 1.0, torch.zeros(2, heads * dim * vdim, device=gpu),
                              torch.zeros(T, hv, device=gpu), dev([0, 0]), dev([1]), positions, 0, heads, dim, vdim,
                              heads_per_key=heads // key_heads, scan=(None,) * 6)


@pytest.mark.parametrize("heads,dim,vdim", [(4, 16, 24), (3, 20, 7), (2, 128, 64), (2, 200, 130)])
def test_fading_recurrence_with_silu_against_plain(gpu, heads, dim, vdim):
    """Constant decays, SiLU where the operands are loaded or by a launch in front: the same bits, whole, in portions, and to
    rounding in the three passes."""
    from bitwise_amd.csrc import ops
    g = torch.Generator().manual_seed(dim + vdim)
    T, hd, hv = 150, heads * dim, heads * vdim
    y = torch.randn(T, 2 * hd + hv + 3, generator=g)
    decay = [0.5 + 0.5 * h / max(heads - 1, 1) for h in range(heads)]
    act = pn.silu(y[:, :2 * hd + hv].double())
    want = pn.fading_recurrence(act[:, :hd].view(T, heads, dim), act[:, hd:2 * hd].view(T, heads, dim), act[:, 2 * hd:].view(T, heads, vdim), decay)
    dev = _dev(gpu)
    positions, dd = dev(list(range(T))), torch.tensor(decay, device=gpu)

    def run(cuts, staged, scan_from=None):
        state = torch.zeros(1, heads * dim * vdim, device=gpu)
        yd = y.to(gpu)
        if not staged:
            ops.silu_rows(yd[:, :2 * hd + hv], T)
            assert torch.equal(yd[:, 2 * hd + hv:].cpu(), y[:, 2 * hd + hv:])
        out, at = torch.zeros(T, hv, device=gpu), 0
        for n in cuts:
            rows = slice(at, at + n)
            o = torch.zeros(n, hv, device=gpu)
            scan, seq_rows, nseq = None, dev([0, n]), 1
            if scan_from is not None and n >= scan_from:
                chunks = [(c0, min(32, n - c0), 0, int(c0 + 32 >= n)) for c0 in range(0, n, 32)]
                rec = heads * ops.recurrence_record(dim, vdim)
                scan = (dev(sum(chunks, ())), len(chunks), dev([0, 0, len(chunks)]), 1,
                        torch.zeros(len(chunks) * rec, device=gpu), torch.zeros(len(chunks) * rec, device=gpu))
                seq_rows, nseq = dev([0, 0]), 0
            ops.linear_recurrence(ops.RECUR_FIXED_DECAY, yd[rows], 0, hd, 2 * hd, None, 0, 0, dd, None, 0.0, 1.0, state, o, seq_rows, dev([0]),
                                  positions[rows].contiguous(), nseq, heads, dim, vdim, scan=scan, silu=staged, few_rows=n <= 2)
            out[rows] = o
            at += n
        return out

    err = lambda o: (o.cpu().double().view(T, heads, vdim) - want).abs().max() / want.abs().max()
    whole = run([T], True)
    assert err(whole) < 2e-5
    for cuts, staged in (([T], False), ([1] * T, True), ([7, 64, 2, 77], False)):
        assert torch.equal(run(cuts, staged), whole), (cuts, staged)
    for staged in (True, False):
        assert err(run([20, 130], staged, scan_from=96)) < 2e-5


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-6), (torch.bfloat16, 2 ** -8)])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,hd,rot", [(6, 2, 16, 16, 16, 16), (3, 1, 10, 5, 16, 6), (5, 5, 7, 9, 16, 0), (32, 8, 128, 128, 128, 64), (40, 20, 96, 128, 128, 96)])
def test_norm_over_whole_projections_with_bias_and_rotation(gpu, heads, kv_heads, dim, vdim, hd, rot, dtype, tol):
    """Queries and keys with biases, normed over all heads at once, rotated by either pairing, padded, and written to their
    page slots with the values; also without a cache write (a layer that reads another's)."""
    from bitwise_amd.csrc import ops
    from bitwise_amd.parts.rope import HalfRotaryTable, PairRotaryTable
    from bitwise_amd.runtime import Runtime
    g = torch.Generator().manual_seed(heads * dim)
    rows, page, qn, kn = 5, 16, heads * dim, kv_heads * dim
    n = qn + kn + kv_heads * vdim
    src, bias = torch.randn(rows, n + 3, generator=g), torch.randn(n, generator=g)
    qw, kw = torch.randn(qn, generator=g), torch.randn(kn, generator=g)
    table, pos = torch.tensor([[3, 1]], dtype=torch.int32, device=gpu), [14, 15, 16, 17, -1]
    dev = _dev(gpu)
    for cls, pairs in ((PairRotaryTable, True), (HalfRotaryTable, False)):
        cos, sin = cls({"base": 300.0, "dims": rot, "max_positions": 64}, Runtime("float32", gpu)).tables()
        for with_bias in (True, False):
            z = src[:4, :n].double() + (bias.double() if with_bias else 0)
            spin = lambda x, w: pn.rotate(pn.rms_norm(x, w.double(), 1e-4).view(4, -1, dim), 14, {"base": 300.0, "dims": rot}, pairs)
            want_q, want_k, want_v = spin(z[:, :qn], qw), spin(z[:, qn:qn + kn], kw), z[:, qn + kn:].view(4, kv_heads, vdim)
            for write in (True, False):
                kc, vc = (torch.full((4, kv_heads * page * hd), 9.0, dtype=dtype, device=gpu) for _ in range(2))
                q = torch.full((rows, heads * hd), 9.0, dtype=dtype, device=gpu)
                b = None if not with_bias else (bias if write else bias[:qn]).contiguous().to(gpu)
                ops.whole_norm_kv(src.to(gpu)[:, :n if write else qn], dev(pos), dev([0] * rows), table, qw.to(gpu), kw.to(gpu) if write else qw.to(gpu),
                                  1e-4, q, kc, vc, rows, heads, kv_heads, dim, vdim, hd, page, write, bias=b, cos=cos, sin=sin, rot=rot, halves=not pairs)
                q = q.cpu().double().view(rows, heads, hd)
                near = lambda x, y: ((x - y).abs() <= tol * (1 + y.abs())).all()
                assert near(q[:4, :, :dim], want_q) and (q[:4, :, dim:] == 0).all() and (q[4] == 9).all(), (pairs, with_bias, write)
                if not write:
                    assert (kc == 9).all() and (vc == 9).all()
                    continue
                kc = kc.cpu().double().view(4, kv_heads, page, hd)
                vc = vc.cpu().double().view(4, kv_heads, hd, page).transpose(2, 3) if dtype == torch.bfloat16 else vc.cpu().double().view(4, kv_heads, page, hd)
                for r, p in enumerate(pos[:4]):
                    pg, sl = int(table[0, p // page]), p % page
                    assert near(kc[pg, :, sl, :dim], want_k[r]) and (kc[pg, :, sl, dim:] == 0).all(), r
                    assert near(vc[pg, :, sl, :vdim], want_v[r]) and (vc[pg, :, sl, vdim:] == 0).all(), r


def test_sums_of_branches_side_gate_and_gated_norms(gpu):
    from bitwise_amd.csrc import ops
    g = torch.Generator().manual_seed(4)
    rows = 5
    for width in (37, 512, 2048, 4096, 5000):
        for n in (1, 2, 4):
            ys = [torch.randn(rows + 1, width + 2, generator=g) for _ in range(n)]
            scales = [0.6, -1.5, 2.0, 0.25][:n]
            z = sum(s * y[:, 2:].double() for s, y in zip(scales, ys))
            dev = [y.to(gpu)[:, 2:] for y in ys]
            out = torch.zeros(rows, width, device=gpu)
            ops.scaled_sum(dev, scales, out, rows)
            assert (out.cpu().double() - z[:rows]).abs().max() < 1e-5
            w, x = torch.randn(width, generator=g), torch.randn(rows, width, generator=g)
            xa, xb = x.to(gpu), x.to(gpu)
            ra, rb = (torch.zeros(rows, width, dtype=torch.bfloat16, device=gpu) for _ in range(2))
            ops.scaled_sum_norm_add(dev, scales, w.to(gpu), 1e-3, 1.0, xa, rows, ra)
            ops.norm_add(out, w.to(gpu), xb, rows, 1e-3, rb)
            assert torch.equal(xa, xb) and torch.equal(ra, rb) and torch.equal(ra, xa.to(torch.bfloat16)), (width, n)
            assert (xa.cpu().double() - (x.double() + pn.rms_norm(z[:rows], w.double(), 1e-3))).abs().max() < 2e-5, (width, n)
        # the norm in front of the gate, whole rows and parts, SiLU and sigmoid
        for parts in (1, width // 512 or 1):
            if width % parts:
                continue
            o, zg, w = torch.randn(rows, width, generator=g), torch.randn(rows, width + 5, generator=g) * 3, torch.randn(width, generator=g)
            pos = _dev(gpu)([0] * (rows - 1) + [-1])
            normed = pn.rms_norm(o.double().view(rows, parts, -1), 1.0, 1e-3).reshape(rows, width) * w.double()
            for gate, fn in ((ops.GATE_SIGMOID, torch.sigmoid), (ops.GATE_SILU, pn.silu)):
                want = normed * fn(zg[:, :width].double())
                for dt, tol in ((torch.float32, 1e-5), (torch.bfloat16, 2 ** -8)):
                    out = torch.full((rows, width), 7.0, dtype=dt, device=gpu)
                    ops.gated_part_norm(o.to(gpu), zg.to(gpu)[:, :width], w.to(gpu), out, pos, rows, parts, 1e-3, gate=gate, behind=True)
                    assert ((out[:-1].cpu().double() - want[:-1]).abs() <= tol * (1 + want[:-1].abs())).all() and bool((out[-1] == 7).all())
    # a token's own columns of the side table: a given token, one the step before sampled, padding
    table = torch.randn(29, 60, generator=g)
    z = torch.randn(4, 24, generator=g) * 2
    tokens, feedback = _dev(gpu)([5, -2, -1, 28]), _dev(gpu)([0, 17, 3, 0])
    want = pn.gelu_tanh(z[:, :20].double()) * torch.stack([table[5, 30:50], table[17, 30:50], torch.zeros(20), table[28, 30:50]]).double()
    for tt in (torch.float32, torch.bfloat16):
        for dt, tol in ((torch.float32, 1e-2 if tt == torch.bfloat16 else 1e-6), (torch.bfloat16, 1.2e-2)):
            out = torch.full((4, 20), 7.0, dtype=dt, device=gpu)
            ops.side_gate(z.to(gpu), tokens, feedback, table.to(tt).to(gpu)[:, 30:50], out, 4)
            assert ((out.cpu().double() - want).abs() <= tol * (1 + want.abs())).all(), (tt, dt)
    av = torch.randn(3, 6 * 16, generator=g).to(gpu)
    out = torch.zeros(3, 6 * 10, device=gpu)
    ops.gate_mul(av, 16, None, out, 3, 6, 10)
    assert torch.equal(out.view(3, 6, 10), av.view(3, 6, 16)[:, :, :10])


@pytest.mark.parametrize("N,K", [(256, 2048), (4096, 4104), (2048, 4096), (5120, 2048), (1040, 8192), (4096, 256), (17408, 2048)])
def test_stores_and_gelu_of_products_do_not_depend_on_the_rows(gpu, N, K):
    """A 32-bit store whose segments of K have waves or workgroups of their own: the bits of the plain store, of the residual
    add onto zeros and of every row alone; the exact GELU as the product's epilogue: the bits of the activation behind it."""
    from bitwise_amd.csrc import ops
    torch.manual_seed(N + K)
    w = (torch.randn(N, K, device=gpu) * K ** -0.5).to(torch.bfloat16)
    x = torch.randn(600, K, device=gpu).to(torch.bfloat16)
    first = None
    for rows in (600, 300, 128, 100, 64, 33, 17, 16, 8, 1):
        floats, counters = ops.gemm_add_scratch(rows, N, K)
        scratch = (torch.zeros(max(floats, 1), device=gpu), torch.zeros(max(counters, 1), dtype=torch.int32, device=gpu))
        plain, split, added = (torch.zeros(rows, N, device=gpu) for _ in range(3))
        ops.gemm_bf16(x, w, plain, rows, ops.EPI_F32)
        for again in range(2):                          # (the counters are zero again behind a launch)
            split.fill_(5.0)
            ops.gemm_bf16(x, w, split, rows, ops.EPI_F32, scratch=scratch)
            assert torch.equal(plain, split), (rows, again)
        ops.gemm_bf16(x, w, added, rows, ops.EPI_ADD_F32, scratch=scratch)
        assert torch.equal(plain, added), rows
        first = plain if first is None else first
        assert torch.equal(plain, first[:rows]), rows
        act, ref = (torch.zeros(rows, N, dtype=torch.bfloat16, device=gpu) for _ in range(2))
        ops.gemm_bf16(x, w, act, rows, ops.EPI_GELU_BF16)
        ops.activate(plain, ref, rows, ops.PLAIN_GELU_ERF)
        assert torch.equal(act, ref), rows
    want = x[:40].double() @ w.double().T
    assert (first[:40].double() - want).abs().max() < 1e-4
    gelu = pn.gelu_erf(want.cpu())
    assert ((act[:1].cpu().double() - gelu[:1]).abs() <= 2 ** -7 * gelu[:1].abs() + 1e-5).all()


@pytest.mark.parametrize("N,K", [(16, 64), (256, 2048), (40, 4096), (256, 8192), (1000, 1024), (7, 12288)])
def test_side_gate_in_the_product_of_few_rows(gpu, N, K):
    """The gate of the side input as the product's epilogue: the bits of the product followed by the gate's launch, with given
    tokens, tokens the step before sampled, and padding."""
    from bitwise_amd.csrc import ops
    torch.manual_seed(N + K)
    w, x = (torch.randn(N, K, device=gpu) * K ** -0.5).to(torch.bfloat16), torch.randn(16, K, device=gpu).to(torch.bfloat16)
    table = torch.randn(37, N + 24, device=gpu).to(torch.bfloat16)[:, 8:8 + N]
    tokens = torch.randint(0, 37, (16,)).tolist()
    feedback = torch.randint(0, 37, (16,), dtype=torch.int32, device=gpu)
    for rows in (1, 5, 8, 16):
        given = list(tokens)
        given[rows - 1] = -2
        if rows > 3:
            given[2] = -1
        given = _dev(gpu)(given)
        z, want, got = torch.zeros(16, N, device=gpu), *(torch.full((16, N), 3.0, dtype=torch.bfloat16, device=gpu) for _ in range(2))
        ops.gemm_bf16(x, w, z, rows, ops.EPI_F32)
        ops.side_gate(z, given, feedback, table, want, rows)
        ops.gemm_side_bf16(x, w, given, feedback, table, got, rows)
        assert torch.equal(got, want), rows
    assert (got[2] == 0).all() and not (got[0] == 0).all()
    with pytest.raises(ValueError):
        ops.gemm_side_bf16(torch.zeros(17, K, dtype=torch.bfloat16, device=gpu), w, torch.zeros(17, dtype=torch.int32, device=gpu), None, table,
                           torch.zeros(17, N, dtype=torch.bfloat16, device=gpu), 17)


def test_exact_gelu_against_plain(gpu):
    from bitwise_amd.csrc import ops
    x = torch.cat([torch.randn(7, 300, generator=torch.Generator().manual_seed(1)) * 4, torch.tensor([0.0, -1e-6, 1e-6, -80.0, 80.0]).repeat(7, 1)], 1)
    want = pn.gelu_erf(x.double())
    for dt, rel in ((torch.float32, 1e-6), (torch.bfloat16, 2 ** -8)):
        out = torch.zeros(7, 305, dtype=dt, device=gpu)
        ops.activate(x.to(gpu), out, 7, ops.PLAIN_GELU_ERF)
        assert ((out.cpu().double() - want).abs() <= rel * want.abs() + 3e-7 * x.double().abs() + 1e-9).all(), dt
