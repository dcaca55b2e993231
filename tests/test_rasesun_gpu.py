"""Rasesun on the GPU against the plain float64 implementation (plain_rasesun): every mechanism alone (kernels and
one-layer models), whole prompts against token-by-token decoding and against portions down to two tokens, batches of
unequal requests against each alone with pages and slots that are used again, a key made to stand out far back, at page
borders and just inside and outside the window (in prompts and in decoding), memories whose decay is pushed to 1, the
first tokens, long decoding, and greedy generation through the engine."""

import json
import math
from pathlib import Path

import numpy as np
import pytest
import torch

import bitwise_amd as bw
import plain_rasesun as pr

pytestmark = pytest.mark.gpu

# float32: 32-bit sums against float64 ones, a few 1e-6 of a row.  bfloat16: activations rounded where the products and the
# cache take them, carried through the layers and the loop's passes.  A row whose sublayer nearly cancels out is blown up
# by the norm behind it, its roundings with it (the plain model with rounded activations has such rows too: one in a
# hundred moves by a tenth or more of its size), so in that mode the 90th percentile carries the tight bound.
TOL = {"float32": 5e-5, "bfloat16": 0.08}
MOST = {"float32": 1.0, "bfloat16": 0.9}
TYPICAL = {"float32": 1e-5, "bfloat16": 2.5e-2}
SIGMA = 0.15


def mamba(heads, vdim, state, groups, conv, norm_groups, mlp=None):
    return {"type": "mamba2", "mlp": mlp, "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                                    "norm_groups": norm_groups}}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, window, base=1000.0, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                      "scale": scale, "mask": {"size": window}, "rot": {"base": base, "dims": rot_dim}}}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def config(width, vocab, eps, scale, cap, loop, layers, max_positions=1024):
    out = {"architecture": "Rasesun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "logit_softcap": cap, "layers": layers, "max_positions": max_positions}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


CONFIGS = {
    # one mechanism each
    "only_mamba": config(48, 61, 1e-5, 1.0, 15.0, None, [mamba(4, 16, 24, 2, 4, 2)]),
    "only_latent": config(48, 61, 1e-5, 2.0, 15.0, None, [latent(4, 16, 8, 16, 24, 32, 0.3, 21)]),
    "only_dense": config(48, 61, 1e-5, 1.0, 9.0, None, [mamba(1, 16, 8, 1, 2, 1, dense(72))]),
    "only_moe": config(48, 61, 1e-5, 3.0, 30.0, None, [mamba(1, 16, 8, 1, 2, 1, moe(7, 3, 24))]),
    # a span of layers that runs three times, from the second layer on
    "looped": config(40, 53, 1e-5, 1.5, 20.0, (1, 3, 3), [
        mamba(2, 8, 16, 1, 3, 2, moe(5, 2, 16)), latent(2, 8, 4, 8, 8, 16, 0.5, 9, 100.0), mamba(3, 8, 8, 3, 2, 1, moe(4, 1, 8)),
        latent(3, 16, 4, 8, 16, 8, 0.4, 12, mlp=dense(32))]),
    # sizes that are no multiples of 8 anywhere: every product stays on the 32-bit kernels in bfloat16 mode too; a convolution
    # over one token (no state of its own), one value channel a head, a state larger than a wave's lanes
    "odd": config(44, 53, 1e-5, 0.7, 5.0, (0, 2, 2), [
        latent(3, 10, 6, 5, 11, 13, 0.3, 7, 77.0, moe(6, 4, 13)), mamba(6, 1, 70, 3, 1, 3, dense(37)), mamba(5, 7, 9, 5, 7, 7, moe(3, 3, 11))]),
    # everything together, sizes all different from layer to layer: windows that are no multiple of a page, heads that
    # fill no group, one expert a token and all of them, one group of the memory and as many as heads, the norm in one part
    # and in many, a layer without feed-forward, the loop in the middle
    "mixed": config(64, 131, 1e-6, 2.0, 25.0, (1, 4, 2), [
        latent(6, 12, 8, 20, 40, 48, 0.3, 37, 1e4, dense(88)),
        mamba(6, 24, 16, 2, 4, 2, moe(9, 1, 40)),
        latent(3, 32, 16, 8, 24, 64, 0.2, 50, 500.0, moe(5, 5, 16)),
        mamba(4, 40, 33, 4, 5, 5, None),
        latent(18, 8, 8, 16, 56, 24, 0.4, 16, 2e5, moe(12, 3, 24)),
        mamba(2, 64, 128, 1, 4, 1, dense(48)),
    ]),
    # heads of the sizes real models have, a latent of 512, more experts than a wave has lanes, inner sizes beyond one step of
    # the products, windows longer than a block of keys
    "wide": config(136, 77, 1e-5, 4.0, 30.0, (0, 2, 2), [
        latent(2, 128, 64, 128, 96, 512, 0.07, 200, 5e5, moe(72, 6, 48)),
        mamba(4, 64, 128, 2, 4, 2, dense(264)),
        latent(17, 64, 32, 64, 72, 256, 0.1, 140, 8e4, None),
    ]),
}
SEEDS = {name: 91 + i for i, name in enumerate(CONFIGS)}


@pytest.fixture(scope="module")
def folders(tmp_path_factory, gpu):
    tmp = tmp_path_factory.mktemp("rasesun")
    return {name: bw.write_random_model(tmp / name, cfg, SEEDS[name], SIGMA) for name, cfg in CONFIGS.items()}


def weights(folder):
    from safetensors.torch import load_file
    return pr.to64(load_file(str(Path(folder) / "model.safetensors")))


def tokens_for(name, n, seed=0):
    g = torch.Generator().manual_seed(5000 + seed)
    return torch.randint(0, CONFIGS[name]["vocab"], (n,), generator=g).tolist()


_plain = {}


def plain(folder, toks):
    key = (str(folder), tuple(toks))
    if key not in _plain:
        _plain[key] = pr.forward(json.loads((Path(folder) / "config.json").read_text()), weights(folder), toks).numpy()
    return _plain[key]


def close(got, want, dtype):
    worst, most, typical = (pr.logits_error(got, want, q) for q in (1.0, MOST[dtype], 0.5))
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
@pytest.mark.parametrize("name", ["mixed", "odd", "wide"])
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
            assert np.array_equal(got, first), (name, graphs, cuts, pr.logits_error(got, first))
        assert rp.manager.all_free()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_portions_in_parallel_passes(folders, dtype):
    """With the engine's leave to let logits depend on the cut in their last bits, portions of 96 rows and more run
    their recurrences in three passes over chunks: the same values to rounding, alone and beside short portions."""
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
    bit, so also what the slots keep between steps (the convolution's inputs, the memories) and what the windows keep."""
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
            assert r.tokens == pr.generate_greedy(cfg, w, p, 10)
        solo = bw.generate(model, [p], sp, bw.EngineConfig(num_blocks=16, max_num_seqs=1, dtype=dtype, use_graphs=False))[0]
        assert solo.tokens == r.tokens and solo.logits_fingerprint == r.logits_fingerprint


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_randomized_scenarios(gpu, dtype):
    """The scenario simulator on the architecture's tiny model: every request against its solo run, no page or slot
    lost; preemption happens on the way and restarts from a cleared slot."""
    from bitwise_amd.registry import ARCHITECTURES
    from bitwise_amd.sim import Simulator

    model = bw.Model.random(ARCHITECTURES["Rasesun"].tiny_config, 43, dtype, sigma=0.08)
    tally = Simulator(model, dtype).run(12, seed=2)
    print(tally.line(dtype))
    assert tally.violations() == 0, "\n".join(tally.notes[:10])
    assert tally.requests_compared > 30 and tally.prefix_hit_tokens == 0


# ----------------------------------------------------------------------------- one key made to stand out

def needle_model(tmp, window, kv_rank=32, rot_dim=8, tag=""):
    """One layer of attention, no feed-forward, token rows that are unit vectors, a latent of token A that lies across every
    other token's and that alone makes a key, a query latent of token B that alone makes a query, with a scale that makes
    that one score large: what a B sees of an A decides its logits.  Returns (folder, config, A, B, filler)."""
    from safetensors.torch import load_file, save_file
    width, vocab = 64, 40
    a, b, filler = 7, 11, 3
    cfg = config(width, vocab, 1e-6, 1.0, 30.0, None, [latent(2, 16, rot_dim, 16, 24, kv_rank, 1.0, window)], max_positions=2048)
    folder = bw.write_random_model(Path(tmp) / f"needle_{window}_{kv_rank}_{tag}", cfg, 77, 0.3)
    w = load_file(str(Path(folder) / "model.safetensors"))
    w["embed"] = torch.eye(vocab, width).to(torch.bfloat16)
    for n in ("l0.norm1", "l0.norm1b", "l0.mix.dq.norm", "l0.mix.dkv.norm", "final.norm"):
        w[n] = torch.ones_like(w[n])
    for n in ("l0.mix.g", "l0.mix.dq", "l0.mix.dkv", "l0.mix.uq", "l0.mix.uk"):
        w[n] = torch.zeros_like(w[n])                       # (every gate is 1/2; rotated parts stay out of it)
    g = torch.Generator().manual_seed(5)
    direction = torch.randn(16, generator=g)
    direction = direction / direction.norm()
    # latents: A's is the first unit vector, every other token's the second; the same for the queries' and token B
    w["l0.mix.dkv"][1, :] = 1.0
    w["l0.mix.dkv"][:2, a] = torch.tensor([1.0, 0.0]).to(torch.bfloat16)
    w["l0.mix.dq"][1, :] = 1.0
    w["l0.mix.dq"][:2, b] = torch.tensor([1.0, 0.0]).to(torch.bfloat16)
    for h in range(2):
        w["l0.mix.uk"][16 * h:16 * h + 16, 0] = direction.to(torch.bfloat16)
        w["l0.mix.uq"][(16 + rot_dim) * h:(16 + rot_dim) * h + 16, 0] = direction.to(torch.bfloat16)
    # (the latents' lengths are sqrt(kv_rank) and sqrt(q_rank): a score of about 14)
    cfg["layers"][0]["mixer"]["scale"] = 14.0 / math.sqrt(kv_rank * 24)
    (Path(folder) / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(Path(folder) / "model.safetensors"))
    return folder, cfg, a, b, filler


# a window in one block of keys, one that ends at a page, one of several blocks, one longer than the sequence; a latent whose
# key vectors are no multiple of 8 (the 32-bit kernel in either mode)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window,kv_rank,rot_dim", [(37, 32, 8), (48, 264, 8), (129, 512, 64), (300, 32, 8), (64, 30, 6)])
def test_a_key_that_stands_out(tmp_path_factory, gpu, dtype, window, kv_rank, rot_dim):
    """One key answers a later query with a large score: far back, at page borders (pages of 16), at blocks of 64 and 128
    keys, as the first token, and just inside and just outside the query's window, in a prompt and in decoding.  The
    test first makes sure, with the plain model, that seeing the key or not moves the logits by far more than the tolerance."""
    folder, cfg, a, b, filler = needle_model(tmp_path_factory.mktemp("needle"), window, kv_rank, rot_dim)
    w = weights(folder)
    n, W = 300, window
    # (key position, query position): far back, around page and block borders, the first token, around the window's edge
    cases = [(0, n - 1), (0, W - 1), (0, W), (1, W), (1, W + 1), (15, 15 + W - 1), (16, 16 + W - 1), (16, 16 + W), (17, 17 + W),
             (200 - W, 199), (200 - W, 200), (250, 250 + W - 1), (250, 250 + W), (239, 240), (127, 128), (127, 127 + W - 1), (128, 128 + W - 1),
             (128, 128 + W), (63, 64), (3, 290)]
    cases = sorted({(k, q) for k, q in cases if 0 <= k < q < n})
    seen = unseen = 0
    rp = replayer(folder, dtype, 320)
    for i, (kpos, qpos) in enumerate(cases):
        toks = [filler] * n
        toks[kpos], toks[qpos] = a, b
        # (the other tokens' rows are alike in every case; the plain model is asked for what lies around the query)
        want = pr.forward(cfg, w, toks[:qpos + 1]).numpy()
        base = [filler] * (qpos + 1)
        base[qpos] = b
        without = pr.forward(cfg, w, base).numpy()
        sees = qpos - kpos < W
        moved = pr.logits_error(want[qpos:], without[qpos:])
        assert (moved > 0.2) == sees, (kpos, qpos, moved)
        seen, unseen = seen + sees, unseen + (not sees)
        # as a prompt, and with the query (and what lies behind the key) decoded token by token
        for cuts in ([n], [kpos + 1], [max(qpos - 3, 1), 2]):
            got = run_cut(rp, f"n{i}", toks, cuts)
            assert pr.logits_error(got[:qpos + 1], want, 1.0) < TOL[dtype], (kpos, qpos, cuts)
    assert seen >= 5 and (unseen >= 4 or window >= n)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_memories_that_do_not_fade(tmp_path_factory, gpu, dtype):
    """Decays pushed to 1: the first token still moves the logits 250 tokens later (the plain model says so), through
    prompts, portions and decoding; with the usual decays it would be long gone."""
    from safetensors.torch import load_file, save_file
    cfg = config(48, 61, 1e-5, 1.0, 15.0, None, [mamba(4, 16, 24, 2, 4, 2)])
    folder = bw.write_random_model(tmp_path_factory.mktemp("memory") / "m", cfg, 5, 0.3)
    w = load_file(str(Path(folder) / "model.safetensors"))
    w["l0.mix.A_log"] = torch.full_like(w["l0.mix.A_log"], -14.0)          # exp(-exp(-14) delta) is 1 - 8e-7 delta
    save_file(w, str(Path(folder) / "model.safetensors"))
    w64 = pr.to64(w)
    n = 260
    toks = tokens_for("only_mamba", n, 3)
    other = [(toks[0] + 1) % 61] + toks[1:]
    want, want_other = pr.forward(cfg, w64, toks).numpy(), pr.forward(cfg, w64, other).numpy()
    # (one token among 260 that are all remembered alike: some 1/260 of a row, many times the 32-bit tolerance)
    assert pr.logits_error(want[-5:], want_other[-5:], 0.0) > 1e-3, "the first token was meant to matter at the end"
    rp = replayer(folder, dtype, 320)
    for cuts in ([n], [1], [200, 2, 50], [17, 100]):
        assert close(run_cut(rp, "m", toks, cuts), want, dtype), cuts
    rp = replayer(folder, dtype, 320, exact_cuts=False)
    assert close(run_cut(rp, "m", toks, [n]), want, dtype)


# ----------------------------------------------------------------------------- kernels alone

def _dev(gpu):
    return lambda x: torch.tensor(x, dtype=torch.int32, device=gpu)


def test_convolution_with_silu_through_portions_and_slots(gpu):
    from bitwise_amd.csrc import ops
    g = torch.Generator().manual_seed(1)
    dev = _dev(gpu)
    for channels, taps in ((24, 4), (300, 2), (5, 8), (7, 1)):
        wc, bc = torch.randn(channels, taps, generator=g), torch.randn(channels, generator=g)
        seqs = [torch.randn(40, channels, generator=g) for _ in range(3)]
        want = [pr.silu(pr.causal_convolution(s.double(), wc.double(), bc.double())) for s in seqs]
        state = torch.zeros(2, max(1, (taps - 1) * channels) + 3, device=gpu)
        at, slot_of = [0, 0, 0], {0: 0, 1: 1, 2: 0}
        for step in [[(0, 5), (1, 1)], [(1, 2), (0, 1)], [(0, 34), (1, 1)], [(1, 36), (2, 3)], [(2, 1)], [(2, 36)]]:
            x, pos, seq_rows, slots = [], [], [], []
            for r, n in step:
                if at[r] == 0:
                    state[slot_of[r]].zero_()
                seq_rows += [len(pos), n]
                x.append(torch.cat([torch.zeros(n, 2), seqs[r][at[r]:at[r] + n]], 1))
                pos += list(range(at[r], at[r] + n))
                slots.append(slot_of[r])
            out = torch.zeros(len(pos), channels, device=gpu)
            ops.causal_conv(torch.cat(x).to(gpu)[:, 2:], wc.to(gpu), bc.to(gpu), state, dev(seq_rows), dev(slots), dev(pos), len(step),
                            max(n for _, n in step), out, silu=True)
            o = 0
            for r, n in step:
                assert (out[o:o + n].cpu().double() - want[r][at[r]:at[r] + n]).abs().max() < 1e-5, (channels, taps, r, at[r])
                o += n
                at[r] += n
        assert at == [40, 40, 40]


@pytest.mark.parametrize("heads,groups,dim,vdim", [(4, 2, 16, 16), (6, 2, 20, 12), (2, 1, 64, 128), (3, 3, 128, 64), (2, 2, 200, 24), (5, 1, 9, 1)])
def test_recurrence_with_step_sizes_against_plain(gpu, heads, groups, dim, vdim):
    """The memory alone: whole sequences, portions that continue from the slot (bit for bit alike), and the three passes."""
    from bitwise_amd.csrc import ops
    g = torch.Generator().manual_seed(heads * 100 + dim)
    T, hv, gn = 150, heads * vdim, groups * dim
    u = torch.randn(T, hv + 2 * gn, generator=g)
    z = torch.randn(T, heads + 3, generator=g)
    bias, alog, skip = torch.randn(heads, generator=g), torch.randn(heads, generator=g), torch.randn(heads, generator=g)
    want = pr.ssd_recurrence(u[:, :hv].double().view(T, heads, vdim), u[:, hv:hv + gn].double().view(T, groups, dim),
                             u[:, hv + gn:].double().view(T, groups, dim), pr.softplus(z[:, 3:].double() + bias.double()), alog.double(), skip.double())
    dev = _dev(gpu)
    ud, zd = u.to(gpu), z.to(gpu)
    positions = dev(list(range(T)))
    rate = alog.double().exp().float().to(gpu)

    def run(cuts, scan_from=None):
        state = torch.zeros(2, heads * dim * vdim + 3, device=gpu)[:, 3:]           # (a column slice, as a shared slot gives it)
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
            ops.linear_recurrence(ops.RECUR_STEP_DECAY, ud[rows].contiguous(), hv + gn, hv, 0, zd[rows], 3, 0, bias.to(gpu), rate, 0.0, 1.0,
                                  state, o, seq_rows, dev([1]), positions[rows].contiguous(), nseq, heads, dim, vdim, scan=scan,
                                  heads_per_key=heads // groups, skip=skip.to(gpu))
            out[rows] = o
            at += n
        return out

    scale = want.abs().max()
    err = lambda o: (o.cpu().double().view(T, heads, vdim) - want).abs().max() / scale
    whole = run([T])
    assert err(whole) < 2e-5
    for cuts in ([1] * T, [7, 64, 2, 77]):
        assert torch.equal(run(cuts), whole), cuts
    assert err(run([T], scan_from=96)) < 2e-5 and err(run([20, 130], scan_from=96)) < 2e-5


def test_gated_norm_in_parts_and_activations(gpu):
    from bitwise_amd.csrc import ops
    g = torch.Generator().manual_seed(2)
    rows = 7
    for width, parts in ((48, 1), (48, 3), (37, 37), (600, 2), (4096, 1), (5000, 2)):
        o, z, w = torch.randn(rows, width, generator=g), torch.randn(rows, width + 5, generator=g) * 3, torch.randn(width, generator=g)
        want = pr.gated_part_norm(o.double(), z[:, :width].double(), w.double(), parts, 1e-3)
        pos = _dev(gpu)([0] * (rows - 1) + [-1])
        for dt, tol in ((torch.float32, 1e-5), (torch.bfloat16, 2 ** -8)):
            out = torch.full((rows, width), 7.0, dtype=dt, device=gpu)
            ops.gated_part_norm(o.to(gpu), z.to(gpu)[:, :width], w.to(gpu), out, pos, rows, parts, 1e-3)
            assert ((out[:-1].cpu().double() - want[:-1]).abs() <= tol * (1 + want[:-1].abs())).all() and bool((out[-1] == 7).all()), (width, parts, dt)
    x = torch.cat([torch.randn(rows, 300, generator=g) * 4, torch.tensor([0.0, -1e-6, 1e-6, -80.0]).repeat(rows, 1)], 1)
    for act, want, coeff in ((ops.PLAIN_RELU2, pr.squared_relu(x.double()), (0.0, 0.0)),
                             (ops.PLAIN_XIELU, pr.xielu(x.double(), torch.tensor([0.4, -0.7], dtype=pr.F)),
                              tuple(float(pr.softplus(torch.tensor(v, dtype=pr.F))) for v in (0.4, -0.7)))):
        for dt, rel in ((torch.float32, 1e-6), (torch.bfloat16, 2 ** -8)):
            out = torch.zeros(rows, 304, dtype=dt, device=gpu)
            ops.activate(x.to(gpu), out, rows, act, *coeff)
            assert ((out.cpu().double() - want).abs() <= rel * want.abs() + 1e-6 * x.double().abs() + 1e-9).all(), (act, dt)


@pytest.mark.parametrize("rows", [1, 5, 40, 700])
@pytest.mark.parametrize("top,experts", [(1, 3), (3, 12), (4, 4), (5, 100), (2, 1024)])
def test_experts_by_table_against_plain(gpu, rows, top, experts):
    """Choices, weights and plan from the token ids (also one that the step before sampled, and padding rows, which take the
    first row's experts), then the products of experts without a gate, in 32-bit and on the matrix cores."""
    from bitwise_amd.csrc import ops
    g = torch.Generator().manual_seed(rows * 10 + top)
    vocab, width, ff = 29, 40, (72 if experts < 1000 else 8)
    table = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(vocab)]).to(torch.int32)
    tokens = torch.randint(0, vocab, (rows,), generator=g)
    given, feedback = tokens.clone(), torch.zeros(rows, dtype=torch.int64)
    if rows > 3:
        given[2], feedback[2] = -2, tokens[2]
        given[3] = -1
        tokens[3] = tokens[0]
    slots = rows * top
    dev = lambda t: t.to(torch.int32).to(gpu)
    ids, wts = torch.full((rows, top), -1, dtype=torch.int32, device=gpu), torch.zeros(rows, top, device=gpu)
    srt, place = (torch.full((slots,), -1, dtype=torch.int32, device=gpu) for _ in range(2))
    tiles, meta = torch.zeros(4 * ops.moe_max_tiles(slots, experts), dtype=torch.int32, device=gpu), torch.zeros(4, dtype=torch.int32, device=gpu)
    ops.moe_table_plan(dev(given), dev(feedback), rows, dev(table), experts, 1.0 / top, ids, wts, srt, place, tiles, meta)
    assert torch.equal(ids.cpu(), table[tokens]) and torch.allclose(wts.cpu(), torch.full((rows, top), 1.0 / top))
    flat = ids.cpu().reshape(-1)
    assert torch.equal(srt.cpu().long(), torch.argsort(flat, stable=True)) and torch.equal(place.cpu()[srt.cpu().long()].long(), torch.arange(slots))
    up, down = torch.randn(experts, ff, width, generator=g) * 0.2, torch.randn(experts, width, ff, generator=g) * 0.2
    x = torch.randn(rows, width, generator=g)
    for dt, tol in ((torch.float32, 1e-5), (torch.bfloat16, 0.03)):
        xr, wu, wd = x.to(dt), up.to(dt), down.to(dt)
        w = {f"e{e}.up": wu[e].double() for e in range(experts)} | {f"e{e}.down": wd[e].double() for e in range(experts)} | {"table": table}
        want = pr.table_moe(xr.double(), tokens.tolist(), w, "", {"router": {"experts": experts, "top": top}})
        act = torch.zeros(slots, ff, dtype=dt, device=gpu)
        ops.moe_experts(xr.to(gpu), wu.to(gpu), act, srt, tiles, meta, slots, top, ops.MOE_PLAIN)
        y = torch.zeros(slots, width, device=gpu)
        ops.moe_experts(act, wd.to(gpu), y, srt, tiles, meta, slots, top, ops.MOE_DOWN)
        out = torch.zeros(rows, width, device=gpu)
        ops.moe_combine(y, place, wts, top, out, rows, False)
        assert (out.cpu().double() - want).abs().max() / want.abs().max() < tol, dt


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows", [1, 9, 40, 130])
def test_products_per_head_with_rotation_and_gate(gpu, rows, dtype):
    """A product per head into a wider row, with the rotation of neighbours beside it, and one with a gate per head: by
    32-bit chains and on the matrix cores (whose rows do not depend on how many come together)."""
    from bitwise_amd.csrc import ops
    from bitwise_amd.parts.rope import PairRotaryTable
    from bitwise_amd.runtime import Runtime
    g = torch.Generator().manual_seed(rows)
    for heads, dim, rot, rank in ((3, 16, 8, 40), (2, 128, 64, 512), (5, 10, 6, 7), (2, 264, 8, 30)):
        per, wide = dim + rot, rank + rot
        x, wk = torch.randn(rows, heads * per, generator=g), (torch.randn(heads, dim, rank, generator=g) * 0.1).to(torch.bfloat16)
        table = PairRotaryTable({"base": 300.0, "dims": rot, "max_positions": 300}, Runtime("float32", gpu))
        cos, sin = table.tables()
        pos = torch.arange(60, 60 + rows).to(torch.int32).to(gpu)
        gate = torch.randn(rows, heads + 2, generator=g)
        xv = x.double().view(rows, heads, per)
        turned = pr.rotate_pairs(xv[..., dim:], 60, {"base": 300.0, "dims": rot})
        for cores in ([False, True] if ops.headwise_mfma_ok(wk, dim, heads * per, per) else [False]):
            wd = (wk.transpose(1, 2) if cores else wk).contiguous().to(gpu)
            xin = pr.round_bf16(xv[..., :dim]) if cores else xv[..., :dim]
            product = torch.einsum("rhi,hio->rho", xin, wk.double())
            tol = 1e-5 if dtype == torch.float32 else 0.02
            run = lambda n, ld, **kw: ops.headwise_linear(x[:n].to(gpu), 0, per, wd, out, 0, ld, n, matrix_cores=cores, **kw)
            out = torch.zeros(rows, heads * wide, dtype=dtype, device=gpu)
            run(rows, wide, rotate=(rot, rot, True, dim, rank, cos, sin, pos))
            want = torch.cat([product, turned], -1).reshape(rows, -1)
            assert (out.cpu().double() - want).abs().max() / want.abs().max() < tol, (heads, cores)
            whole, out = out, torch.zeros(1, heads * wide, dtype=dtype, device=gpu)
            run(1, wide, rotate=(rot, rot, True, dim, rank, cos, sin, pos))
            assert torch.equal(out[0], whole[0])
            out = torch.zeros(rows, heads * rank, dtype=dtype, device=gpu)
            run(rows, rank, gate=gate.to(gpu)[:, 2:])
            want = (product * torch.sigmoid(gate[:, 2:].double())[..., None]).reshape(rows, -1)
            assert (out.cpu().double() - want).abs().max() / want.abs().max() < tol, (heads, cores)
            if cores:
                out = torch.zeros(rows, heads * rank, dtype=dtype, device=gpu)
                ops.headwise_linear(x.to(torch.bfloat16).to(gpu), 0, per, wd, out, 0, rank, rows, matrix_cores=True)
                want = product.reshape(rows, -1)
                assert (out.cpu().double() - want).abs().max() / want.abs().max() < tol, heads
