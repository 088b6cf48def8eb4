"""Fikupel through the engine against the plain implementation (tests/plain/fikupel_plain.py): each mechanism alone, every way
of cutting the work, windows' edges, kept first tokens and the first that are not, far tokens, long decoding, pages used again,
other sizes, generation through the scheduler.  Backend "host" runs the engine's own code on the CPU with the kernels' plain
references in their place; backend "gpu" runs the HIP kernels."""
import copy
import json
import math
import os

import pytest
import torch

import replay_util as U
from conftest import seeded_tokens
from plain import fikupel_plain as plain


# ----------------------------------------------------------------------------------------------------------------
# configurations: each differs from the others in every size
# ----------------------------------------------------------------------------------------------------------------
def scaling(factor=4.0, original=64, low=1.0, high=4.0):
    return dict(factor=factor, original=original, low=low, high=high)


def attention(heads=4, kv_heads=2, dim=16, vdim=8, dims=8, base=10000.0, scale=None, window=20, keep=5, scaled=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale if scale is not None else 0.9 * dim ** -0.5,
             rot=dict(base=base, dims=dims))
    if scaled:
        m["rot"]["scaling"] = scaled
    if window:
        m["mask"] = dict(size=window)
        if keep is not None:
            m["mask"]["keep_first"] = keep
    return dict(type="attention", mixer=m)


def latent(heads=3, dim=8, vdim=12, kv_rank=16, q_rank=12, scale=None, window=20):
    m = dict(heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale if scale is not None else dim ** -0.5)
    if window:
        m["mask"] = dict(size=window)
    return dict(type="latent_attention", mixer=m)


def dense(ff=40):
    return dict(kind="dense", ff=ff)


def moe(ff=24, experts=6, top=2):
    return dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))


def config(layers, width=32, vocab=97, eps=1e-5, streams=3):
    c = dict(architecture="Fikupel", vocab=vocab, width=width, norm=dict(eps=eps), layers=layers)
    if streams:
        c["streams"] = streams
    return c


def with_mlp(layer, mlp):
    return dict(layer, mlp=mlp)


# both mixers and both feed-forwards; grouped key heads; part of a head turned, stretched; windows that are no multiple of a
# page; first tokens that are no multiple of one; a layer without a feed-forward
CFG_P = config([with_mlp(attention(4, 2, 16, 8, dims=8, window=23, keep=5, scaled=scaling(4.0, 64, 1.0, 4.0)), dense(40)),
                with_mlp(latent(3, 8, 12, 16, 12, window=37), moe(24, 6, 2)),
                with_mlp(attention(2, 1, 24, 40, dims=24, window=9, keep=33, base=500.0), None),
                with_mlp(latent(5, 12, 6, 24, 20, window=11), dense(24))], width=32, vocab=97, streams=3)
# other sizes: one copy of the stream; one key head; values wider than keys; a head size that no 16 divides; nothing turned in
# the keys; a window of one, one shorter than a page, one that never closes; kept tokens that fill whole pages, none, and more
# than the window; one expert of four; another order of layers
CFG_Q = config([with_mlp(latent(2, 12, 5, 20, 7, window=5), moe(16, 4, 1)),
                with_mlp(attention(3, 1, 24, 40, dims=0, base=300.0, scale=0.31, window=1, keep=16), dense(20)),
                with_mlp(attention(2, 2, 8, 4, dims=2, window=0), moe(40, 3, 3)),
                with_mlp(attention(5, 5, 10, 6, dims=4, window=16, keep=0, scaled=scaling(8.0, 16, 0.5, 2.0)), None),
                with_mlp(latent(4, 6, 16, 8, 33, window=0), dense(56))], width=48, vocab=131, eps=1e-6, streams=1)
# sizes that are multiples of nothing, and a stream without copies
CFG_R = config([with_mlp(attention(2, 1, 10, 6, dims=4, window=9, keep=3, scaled=scaling(2.0, 32, 1.0, 1.0)), moe(12, 9, 3)),
                with_mlp(latent(5, 6, 10, 7, 5, window=50), dense(9)),
                with_mlp(latent(1, 3, 1, 9, 6, window=2), moe(7, 2, 2))], width=36, vocab=61, streams=0)
# sizes nearer a small model's
CFG_S = config([with_mlp(latent(4, 48, 32, 80, 64, window=100), dense(352)),
                with_mlp(attention(6, 3, 64, 48, dims=48, base=100000.0, window=130, keep=40, scaled=scaling(3.0, 128, 1.0, 8.0)), moe(48, 12, 4)),
                with_mlp(attention(4, 1, 96, 96, dims=64, base=20000.0, window=65, keep=2), moe(64, 5, 2))], width=192, vocab=300, streams=5)
CONFIGS = {"P": (CFG_P, 31), "Q": (CFG_Q, 32), "R": (CFG_R, 33), "S": (CFG_S, 34)}


def louder_mixers(tensors):
    """Drawn weights leave a mixer's result small beside a feed-forward's: its values are made larger, so that what the
    attention does shows in the logits."""
    for name in tensors:
        if name.endswith((".mix.v", ".mix.uv")):
            tensors[name] = tensors[name] * (20.0 if name.endswith(".v") else 4.0)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    from denno_beta_amd.weights import write_model_folder
    made = {}

    def get(name, dtype="float32", cfg=None, seed=None, change=louder_mixers):
        key = (name, dtype)
        if key not in made:
            c, s = CONFIGS[name] if cfg is None else (cfg, seed)
            d = str(tmp_path_factory.mktemp(f"fikupel{name}_{dtype}"))
            write_model_folder(d, c, s, dtype)
            from safetensors.torch import load_file, save_file
            path = os.path.join(d, "model.safetensors")
            stored = load_file(path)
            tensors = {k: v.float() for k, v in stored.items()}
            change(tensors)
            save_file({k: v.to(stored[k].dtype).contiguous() for k, v in tensors.items()}, path)
            made[key] = d
        return made[key]
    return get


def runner_for(folder, dtype, device, cache_tokens, max_live=4, page_size=16, graphs=True):
    from denno_beta_amd.config import EngineOptions
    from denno_beta_amd.engine import ModelRunner
    return ModelRunner.from_folder(folder, EngineOptions(dtype=dtype, device=device, page_size=page_size,
                                                         cache_tokens=cache_tokens, max_live=max_live, use_graphs=graphs))


_plain = {}


def plain_model(folder):
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    return cfg, {k: v.double() for k, v in load_file(os.path.join(folder, "model.safetensors")).items()}


def plain_logits(folder, seq, layers=None):
    key = (folder, tuple(seq))
    if key not in _plain or layers is not None:
        cfg, w = plain_model(folder)
        logits, streams = plain.forward(seq, cfg, w, return_layers=True)
        if layers is not None:
            layers.extend(streams)
        _plain[key] = logits
    return _plain[key]


def row_errors(got, want):
    """Per position: the root mean square of the difference (its mean taken off) over the spread of the wanted row."""
    d = got.double() - want.double()
    d = d - d.mean(dim=1, keepdim=True)
    return torch.sqrt((d * d).mean(dim=1)) / want.double().std(dim=1)


# bfloat16, in models 32 to 48 wide: a typical row is off by 0.01 of its spread, and one in twenty may be off by more than the
# bound, none by more than two and a half times; a fault moves rows by 0.2 and more
BOUND = {"float32": 2e-5, "bfloat16": 0.06}
BF16_OVER, BF16_WORST = 0.05, 0.15
# bfloat16: a router's choice between two experts whose logits are close may fall the other way under rounding, which
# moves that row, and through keys later rows, by as much as a fault would.  The bfloat16 models of these tests therefore let
# every token use all its experts (`all_experts`): the same kernels run, no choice can turn, and every row keeps the bound.  The
# choice itself is tested in 32-bit.


def assert_rows(got, want, dtype, what, bound=None, worst=BF16_WORST):
    e = row_errors(got, want)
    b = bound or BOUND[dtype]
    if dtype == "bfloat16" and bound is None:
        over = int((e > b).sum())
        assert over <= max(1, BF16_OVER * len(e)) and e.max() <= worst, (
            f"{what}: {over} of {len(e)} positions are off by more than {b} of their row's spread, the worst (position "
            f"{int(e.argmax())}) by {e.max().item():.3g}")
        return
    assert bool((e <= b).all()), f"{what}: position {int(e.argmax())} is off by {e.max().item():.3g} of its row's spread (bound {b})"


def seqs_for(cfg, lengths, seed=3):
    return [seeded_tokens(seed + i, n, cfg["vocab"]) for i, n in enumerate(lengths)]


def all_experts(cfg):
    cfg = copy.deepcopy(cfg)
    for layer in cfg["layers"]:
        if layer.get("mlp") and layer["mlp"]["kind"] == "moe":
            layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return cfg


# ----------------------------------------------------------------------------------------------------------------
# the plain implementation against itself, and the engine's own constants against it
# ----------------------------------------------------------------------------------------------------------------
def test_plain_pieces():
    g = torch.Generator().manual_seed(0)
    randn = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)      # noqa: E731
    # a window of n: the row itself and the n - 1 before it, and the first tokens
    seen = plain.seen_keys(8, 3, 2)
    assert seen[7].tolist() == [True, True, False, False, False, True, True, True]
    assert seen[1].tolist() == [True, True] + [False] * 6 and seen[3].tolist() == [True] * 4 + [False] * 4
    assert plain.seen_keys(5, None, None)[4].all() and plain.seen_keys(6, 1, 0)[5].tolist() == [False] * 5 + [True]
    # the sink takes its share of the weight and gives nothing; a sink far below is none
    seen = plain.seen_keys(4, None, None)
    p = plain.sink_softmax(torch.zeros(2, 4, 4, dtype=torch.float64), seen, torch.tensor([math.log(2.0), -60.0], dtype=torch.float64))
    assert torch.allclose(p[0][3], torch.full((4,), 1 / 6, dtype=torch.float64)) and torch.allclose(p[1].sum(-1), torch.ones(4, dtype=torch.float64))
    # the stretched encoding: pairs of many turns stay, of few are slowed down by the factor, between the two a blend
    f0 = plain.stretched_frequencies(16, 10000.0, None)
    assert torch.allclose(f0, plain.stretched_frequencies(16, 10000.0, scaling(1.0, 64, 1.0, 4.0)))
    f4 = plain.stretched_frequencies(16, 10000.0, scaling(4.0, 64, 1.0, 4.0))
    assert float(f4[0]) == float(f0[0]) and abs(float(f4[-1]) - float(f0[-1]) / 4) < 1e-18
    assert bool((f4 <= f0 + 1e-18).all()) and bool((f4 >= f0 / 4 - 1e-18).all())
    mid = [i for i in range(8) if 1.0 < 64 * float(f0[i]) / (2 * math.pi) < 4.0]
    assert mid and all(float(f0[i]) / 4 < float(f4[i]) < float(f0[i]) for i in mid)
    # a turn keeps a pair's length and is undone by its reverse; the rest of the vector passes
    v = randn(3, 2, 8)
    pos, freq = torch.tensor([0, 7, 1000]), plain.stretched_frequencies(4, 100.0, None)
    t = plain.turn_pairs(v, pos, freq)
    assert torch.allclose(t[0], v[0]) and torch.allclose(t[..., 4:], v[..., 4:]) and not torch.allclose(t[1], v[1])
    assert torch.allclose(plain.turn_pairs(t, pos, freq, -1.0), v)
    # the polynomial: with one number alone it is that power, normed; with the last alone a constant
    z = randn(5, 12)
    rms = lambda x: torch.sqrt((x * x).mean(-1))      # noqa: E731
    for i, power in enumerate((1, 2, 3)):
        y = plain.poly_norm(z, [2.0 if k == i else 0.0 for k in range(4)], 0.0)
        assert torch.allclose(rms(y), torch.full((5,), 2.0, dtype=torch.float64)) and torch.allclose(y / y[:, :1], z ** power / z[:, :1] ** power)
    assert torch.equal(plain.poly_norm(z, [0.0, 0.0, 0.0, 3.0], 1e-5), torch.full((5, 12), 3.0, dtype=torch.float64))
    # copies of the stream: the mix is indexed [from, to], and all copies are made from the old ones
    w = {"in": torch.tensor([0.5, 2.0], dtype=torch.float64), "out": torch.tensor([1.0, -1.0], dtype=torch.float64),
         "mix": torch.tensor([[1.0, 10.0], [100.0, 1000.0]], dtype=torch.float64)}
    xs = torch.stack([torch.full((1, 1), 1.0), torch.full((1, 1), 2.0)]).double()
    seen = []
    out = plain.sublayer(xs, w.__getitem__, lambda u: (seen.append(float(u)), u * 0 + 7.0)[1])
    assert seen == [4.5] and out.flatten().tolist() == [1 + 200 + 7, 10 + 2000 - 7]
    # the experts' weights are the softmax over the chosen logits alone, the bias among them
    W, E = 3, 4
    pw = {"router": torch.zeros(E, W, dtype=torch.float64), "router.b": torch.tensor([0.0, 3.0, -1.0, 3.0 + math.log(3.0)], dtype=torch.float64)}
    for e in range(E):
        pw[f"e{e}.gate"], pw[f"e{e}.up"], pw[f"e{e}.down"] = randn(2, W), randn(2, W), randn(W, 2)
    h = randn(2, W)
    ex = lambda e: plain.expert(h, pw[f"e{e}.gate"], pw[f"e{e}.up"], pw[f"e{e}.down"])      # noqa: E731
    assert torch.allclose(plain.moe_ff(h, pw.__getitem__, moe(2, E, 2)), 0.25 * ex(1) + 0.75 * ex(3))


@pytest.mark.parametrize("dims,base,sc", [(8, 10000.0, scaling(4.0, 64, 1.0, 4.0)), (4, 5000.0, scaling(2.0, 32, 0.5, 8.0)), (24, 300.0, None),
                                          (16, 250000.0, scaling(1.0, 128, 2.0, 3.0)), (2, 10.0, scaling(8.0, 16, 1.0, 1.0)),
                                          (64, 1e6, scaling(8.0, 8192, 1.0, 4.0)), (0, 100.0, None)])
def test_frequencies_of_the_stretched_encoding(dims, base, sc):
    from denno_beta_amd.parts.positions import RotaryPairs
    part = RotaryPairs(dims=dims, base=base, head_dim=max(dims, 2), scaling=sc)
    assert torch.allclose(part.frequencies(), plain.stretched_frequencies(dims, base, sc), rtol=1e-14, atol=0) and part.mag == 1.0


# ----------------------------------------------------------------------------------------------------------------
# each mechanism alone
# ----------------------------------------------------------------------------------------------------------------
ALONE = {
    "attention": [with_mlp(attention(4, 2, 8, 8, dims=8, window=0), None)],
    "attention_window": [with_mlp(attention(2, 2, 8, 8, dims=4, window=7, keep=None), None)],
    "attention_first_kept": [with_mlp(attention(2, 1, 8, 8, dims=4, window=4, keep=6), None)],
    "attention_stretched": [with_mlp(attention(2, 1, 12, 20, dims=6, window=0, scaled=scaling(4.0, 16, 0.5, 3.0)), None)],
    "attention_keys_not_turned": [with_mlp(attention(3, 3, 16, 8, dims=0, window=11, keep=2), None)],
    "attention_wide_values": [with_mlp(attention(1, 1, 4, 36, dims=2, window=9, keep=1), None)],
    "latent": [with_mlp(latent(2, 8, 8, 8, 6, window=0), None)],
    "latent_of_one_number": [with_mlp(latent(2, 3, 1, 1, 1, window=8), None)],      # (normed, it is a sign)
    "latent_window": [with_mlp(latent(3, 6, 10, 5, 9, window=6), None)],
    # a latent too wide for one key of the attention kernels: every head's own keys and values are kept instead
    "latent_kept_by_heads": [with_mlp(latent(2, 8, 12, 262, 10, window=9), None)],
    "dense": [with_mlp(latent(1, 4, 4, 4, 4, window=3), dense(28))],
    "dense_wide": [with_mlp(latent(1, 4, 4, 4, 4, window=3), dense(1100))],
    "experts": [with_mlp(latent(1, 4, 4, 4, 4, window=3), moe(12, 6, 3))],
    "one_expert": [with_mlp(latent(1, 4, 4, 4, 4, window=3), moe(10, 1, 1))],
}


# (every number of copies with three of the mechanisms, two with all)
@pytest.mark.parametrize("what,streams", [(w, n) for w in sorted(ALONE) for n in (0, 2)]
                         + [(w, n) for w in ("attention_first_kept", "experts", "dense") for n in (1, 4, 7)])
def test_each_mechanism_alone(backend, folders, what, streams):
    cfg = config(ALONE[what], width=24, vocab=53, streams=streams)
    folder = folders(f"alone_{what}_{streams}", "float32", cfg, 5)
    seq = seqs_for(cfg, [29])[0]
    want = plain_logits(folder, seq)
    r = runner_for(folder, "float32", backend, 64)
    assert_rows(U.replay(r, U.whole_trace([seq]))["r0"], want, "float32", what)
    r = runner_for(folder, "float32", backend, 64)
    assert_rows(U.replay(r, U.chunk_trace([seq], sizes=(2, 5, 1, 9, 3)))["r0"], want, "float32", what + " in portions")


def test_what_the_model_fixes_matters(folders):
    """The constants and tensors that the plain model is built from change its logits: a test against it would see them."""
    cfg0 = CFG_P
    folder = folders("P", "float32")
    _, W = plain_model(folder)
    seq = seqs_for(cfg0, [60])[0]
    want = plain_logits(folder, seq)

    def cfg_change(*path, value=None, delete=False):
        c = copy.deepcopy(cfg0)
        d = c
        for key in path[:-1]:
            d = d[key]
        if delete:
            del d[path[-1]]
        else:
            d[path[-1]] = value
        return c, W
    zero = lambda name: (cfg0, dict(W, **{name: torch.zeros_like(W[name])}))      # noqa: E731
    ones = lambda name: (cfg0, dict(W, **{name: torch.ones_like(W[name])}))       # noqa: E731
    swapped = dict(W, **{"l1.hc1.mix": W["l1.hc1.mix"].t().contiguous()})
    changes = {"window": cfg_change("layers", 0, "mixer", "mask", "size", value=24), "latent window": cfg_change("layers", 1, "mixer", "mask", "size", value=36),
               "keep_first": cfg_change("layers", 0, "mixer", "mask", "keep_first", value=4),
               "scaling": cfg_change("layers", 0, "mixer", "rot", "scaling", delete=True), "base": cfg_change("layers", 2, "mixer", "rot", "base", value=600.0),
               "scale": cfg_change("layers", 1, "mixer", "scale", value=0.5), "eps": cfg_change("norm", "eps", value=1e-2),
               "gate": zero("l0.mix.g"), "sink": zero("l0.mix.sink"), "latent sink": zero("l1.mix.sink"), "temp": ones("l2.mix.temp"),
               "q norm": ones("l0.mix.q.norm"), "k norm": ones("l2.mix.k.norm"), "dq norm": ones("l1.mix.dq.norm"), "dkv norm": ones("l3.mix.dkv.norm"),
               "act": zero("l0.mlp.act"), "router bias": zero("l1.mlp.router.b"), "in": ones("l0.hc2.in"), "out": ones("l3.hc2.out"),
               "mix": (cfg0, swapped), "norm1": ones("l1.norm1"), "norm2": ones("l0.norm2"), "final norm": ones("final.norm")}
    for name, (c, w) in changes.items():
        assert row_errors(plain.forward(seq, c, w), want).max() > 1e-3, name


# ----------------------------------------------------------------------------------------------------------------
# every way of cutting the work
# ----------------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name,dtype", [(n, d) for d in ("float32", "bfloat16") for n in "PQRS"])
def test_every_cutting_matches_the_plain_implementation(backend, folders, name, dtype):
    cfg = CONFIGS[name][0]
    lengths = ((1, 2, 37, 70, 23) if name != "S" else (2, 40)) if backend == "cpu" else (1, 2, 37, 150, 23, 301)
    if dtype == "bfloat16":
        cfg = all_experts(cfg)
    folder = folders(name, dtype, cfg, CONFIGS[name][1])
    seqs = seqs_for(cfg, lengths)
    want = [plain_logits(folder, s) for s in seqs]
    traces = {"whole": U.whole_trace(seqs), "tail": U.tail_decode_trace(seqs, 20),
              "chunks": U.chunk_trace(seqs, sizes=(2, 3, 5, 17, 2, 16, 7, 32, 2, 31)), "mixed": U.mixed_trace(seqs, seed=5, max_live=3)}
    results = {}
    for kind, steps in traces.items():
        tokens = U.max_live_tokens(steps)
        r = runner_for(folder, dtype, backend, cache_tokens=tokens, max_live=3)
        got = U.replay(r, steps)
        r.cache.manager.check()
        assert r.cache.manager.live() == 0
        if kind == "mixed":
            assert max(r.cache.manager.reuse_count(g) for g in r.cache.paged_groups()) > 0, "the pool was too large: no page was used again"
        for i in range(len(seqs)):
            assert_rows(got[f"r{i}"], want[i], dtype, f"{name} {dtype} {kind} request {i}")
        results[kind] = got
    for kind in ("tail", "chunks", "mixed"):
        for i in range(len(seqs)):
            a, b = results["whole"][f"r{i}"], results[kind][f"r{i}"]
            assert_rows(b, a, dtype, f"{name} {dtype} {kind} against whole, request {i}", 1e-5 if dtype == "float32" else None)


def test_the_stream_after_every_layer(backend, folders):
    """Layer by layer: the sum of the stream's copies behind each layer, read from the engine's own rows."""
    from denno_beta_amd.parts.blocks import MultiStreamBlock
    cfg = CONFIGS["P"][0]
    folder = folders("P", "float32")
    seq = seqs_for(cfg, [47], seed=11)[0]
    streams = []
    plain_logits(folder, seq, streams)
    r = runner_for(folder, "float32", backend, 64)
    seen = []
    real = MultiStreamBlock.forward

    def spy(self, xs, ctx, caches, runtime):
        real(self, xs, ctx, caches, runtime)
        seen.append(xs.detach().sum(dim=0).cpu())
    MultiStreamBlock.forward = spy
    try:
        U.replay(r, U.whole_trace([seq]))
    finally:
        MultiStreamBlock.forward = real
    assert len(seen) == len(cfg["layers"])
    for i, want in enumerate(streams):
        d = (seen[i].double() - want).abs().max() / want.abs().max()
        assert d < 2e-5, f"the stream behind layer {i} differs by {d:.3g} of its largest entry"


# ----------------------------------------------------------------------------------------------------------------
# far tokens, windows' edges and kept first tokens: weights made so that losing one token, or seeing one too many, shows
# ----------------------------------------------------------------------------------------------------------------
MARKER = 7      # the token that the crafted layers look for
WINDOW, KEEP = 40, 19
NEEDLE_DIM, LATENT_DIM, LATENT_RANK = 16, 8, 24


def _directions(tensors, seed):
    """Every token's row becomes a random vector of length about 1 plus 0.7 along a common direction u; the marker's row
    alone has a part along m (at right angles to u and to every other row).  The copies of the stream are read as their mean and
    written as they are."""
    g = torch.Generator().manual_seed(seed)
    V, W = tensors["embed"].shape
    unit = lambda n: torch.nn.functional.normalize(torch.randn(n, generator=g), dim=0)   # noqa: E731
    u, m = unit(W), unit(W)
    m = torch.nn.functional.normalize(m - (m @ u) * u, dim=0)
    e = torch.randn(V, W, generator=g) / W ** 0.5
    e = e - torch.outer(e @ m, m) - torch.outer(e @ u, u)
    tensors["embed"] = e + 0.7 * u
    tensors["embed"][MARKER] += 2.0 * m
    tensors["l0.norm1"] = torch.ones_like(tensors["l0.norm1"])
    n = tensors["l0.hc1.in"].shape[0]
    tensors["l0.hc1.in"], tensors["l0.hc1.out"], tensors["l0.hc1.mix"] = torch.full((n,), 1.0 / n), torch.ones(n), torch.eye(n)
    return u, m


def needle(tensors):
    """An attention whose first head looks for one token wherever it may see it: every query points along d (made from the
    common direction u), the marker's key alone has a part along d (made from m), and every key of that key head has the same part
    along c, at right angles to d; d lies in the pair of dimensions that the position turns slowest, c in the fastest.  Behind
    the norm of q and k the marker's score is large, the others' zero.  A key that is lost, misplaced, read from a wrong page or
    seen from outside changes a row as much as one head can."""
    u, m = _directions(tensors, 1)
    q, k = tensors["l0.mix.q"], tensors["l0.mix.k"]
    dk = NEEDLE_DIM      # (the first query head and the only key head)
    d, c = torch.zeros(dk), torch.zeros(dk)
    d[-2:] = torch.tensor([0.6, 0.8])
    c[:2] = torch.tensor([0.8, -0.6])
    q[:dk] = 8.0 * torch.outer(d, u)
    k[:dk] = 4.0 * torch.outer(d, m) + 4.0 * torch.outer(c, u)
    for name in ("q.norm", "k.norm", "temp"):
        tensors["l0.mix." + name] = torch.ones_like(tensors["l0.mix." + name])
    tensors["l0.mix.v"] = tensors["l0.mix.v"] * 20.0
    tensors["l0.mix.g"] = torch.zeros_like(tensors["l0.mix.g"])       # (every gate at one half)


def latent_needle(tensors):
    """The same in a latent attention: every query of the first head points along d, the marker's latent alone has an entry
    that the first head's keys are made from."""
    u, m = _directions(tensors, 4)
    d = torch.zeros(LATENT_DIM)
    d[-2:] = torch.tensor([0.6, 0.8])
    tensors["l0.mix.dq"][0] = 4.0 * u
    tensors["l0.mix.dkv"] = tensors["l0.mix.dkv"] * 8.0      # (so that a rounded row's small part along m stays small behind the norm)
    tensors["l0.mix.dkv"][0] = 3.0 * m
    for name in ("dq.norm", "dkv.norm"):
        tensors["l0.mix." + name] = torch.ones_like(tensors["l0.mix." + name])
    uq, uk = tensors["l0.mix.uq"], tensors["l0.mix.uk"]
    uq[:LATENT_DIM] = 0.0
    uq[:LATENT_DIM, 0] = d
    uk[:LATENT_DIM] = 0.0
    uk[:LATENT_DIM, 0] = d
    tensors["l0.mix.uv"] = tensors["l0.mix.uv"] * 4.0


CRAFTED = {"attention": (config([with_mlp(attention(2, 1, NEEDLE_DIM, 16, dims=16, base=1e6, scale=1.0, window=WINDOW, keep=KEEP), None)],
                                width=32, vocab=71, streams=3), needle),
           "latent": (config([with_mlp(latent(2, LATENT_DIM, 16, LATENT_RANK, 20, scale=0.3, window=WINDOW), None)],
                             width=32, vocab=71, streams=2), latent_needle)}


@pytest.mark.parametrize("what", ["attention", "latent"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_edge_of_a_window(backend, folders, what, dtype):
    """One layer, so that a row sees the marked token through the attention alone: the row `window - 1` behind it must; the
    row `window` behind it must not, unless the token is one of the first that are kept, which every row sees.  In a prompt, in
    portions cut at, before and behind the edge, and in decoded tokens."""
    cfg, change = CRAFTED[what]
    folder = folders(f"crafted_{what}", dtype, cfg, 9, change)
    n = 110
    ordinary = [t if t != MARKER else MARKER + 1 for t in seqs_for(cfg, [n], seed=40)[0]]
    # the first place, a page's last and first place, the last kept token and the first that is not, the middle of a page
    for at in (0, 15, 16, KEEP - 1, KEEP, 29):
        kept = what == "attention" and at < KEEP
        seq = list(ordinary)
        seq[at] = MARKER
        want, without = plain_logits(folder, seq), plain_logits(folder, ordinary)
        inside, outside = at + WINDOW - 1, at + WINDOW
        # the test's own check: rows that see the marker depend on it, the others do not at all
        e = row_errors(without, want)
        assert e[at + 1:inside + 1].min() > 0.15, "the crafted weights do not show the window's edge"
        assert (e[outside:].min() > 0.15) if kept else (e[outside:].max() < 1e-9)
        cuts = {"whole": U.whole_trace([seq]), "tail": U.tail_decode_trace([seq], n - at - 3),
                "at_the_edge": U.chunk_trace([seq], sizes=(inside, 1, 1, 1000)),
                "around": U.chunk_trace([seq], sizes=(outside, 2, 1000) if at else (inside - 1, 3, 2, 1000)),
                "pages": U.chunk_trace([seq], sizes=(16, 16, 32, 1, 15, 48))}
        for kind, steps in cuts.items():
            if backend == "cpu" and at not in (0, KEEP) and kind in ("around", "pages", "tail"):
                continue          # (the host backend is slow)
            r = runner_for(folder, dtype, backend, U.max_live_tokens(steps))
            got = U.replay(r, steps)["r0"]
            assert_rows(got, want, dtype, f"window {what} {dtype} {kind}, the marker at {at}", 1e-4 if dtype == "float32" else None)
            # sharper at the two rows: each is far nearer to the model with the right window than to one that is off by one
            right = row_errors(got[[inside, outside]], want[[inside, outside]])
            assert right[0] < 0.05 and right[1] < 0.05, (kind, at, right)
            assert row_errors(got[[inside]], without[[inside]])[0] > 0.1, f"{kind}: the row at the window's edge lost the marked token"
            if kept:
                assert row_errors(got[outside:], without[outside:]).min() > 0.1, f"{kind}: a row behind the window lost a kept token"


def test_kept_tokens_far_behind_in_a_small_pool(backend, folders):
    """A kept token seen from hundreds of positions on, while the pages between it and the window are used again: by the same
    request and by its neighbour, in a pool that holds the kept pages and a few windows."""
    cfg, change = CRAFTED["attention"]
    folder = folders("crafted_attention", "float32", cfg, 9, change)
    n = 150 if backend == "cpu" else 700
    seqs = [[t if t != MARKER else MARKER + 1 for t in s] for s in seqs_for(cfg, [n, n // 2], seed=44)]
    seqs[0][KEEP - 1] = seqs[1][3] = MARKER
    steps = U.mixed_trace(seqs, seed=2, max_live=2, sizes=(1, 1, 2, 7, 19))
    r = runner_for(folder, "float32", backend, cache_tokens=16 * 16, max_live=2)
    if n > 16 * 16:
        assert n + n // 2 > r.options.cache_tokens
    got = U.replay(r, steps)
    r.cache.manager.check()
    assert min(r.cache.manager.reuse_count(g) for g in r.cache.paged_groups()) > (0 if backend == "cpu" else 20)
    for i, s in enumerate(seqs):
        want = plain_logits(folder, s)
        assert_rows(got[f"r{i}"], want, "float32", f"request {i} in a pool of a few windows", 1e-4)
        lost = plain_logits(folder, [t if t != MARKER else MARKER + 1 for t in s])
        assert row_errors(lost[60:], want[60:]).min() > 0.15


def test_pages_behind_a_window_are_given_back(backend, folders):
    """Two kinds of windows side by side: a group that keeps first tokens and one that does not, in a pool of a few windows."""
    cfg = config([with_mlp(attention(2, 1, 8, 8, dims=4, window=9, keep=17), None), with_mlp(latent(2, 8, 8, 8, 8, window=20), dense(16))],
                 width=24, vocab=53, streams=2)
    folder = folders("windows_only", "float32", cfg, 17)
    n = 150 if backend == "cpu" else 400
    seqs = seqs_for(cfg, [n, n // 2], seed=70)
    steps = U.mixed_trace(seqs, seed=2, max_live=2, sizes=(1, 1, 2, 7, 19))
    r = runner_for(folder, "float32", backend, cache_tokens=10 * 16, max_live=2)       # far fewer than the requests' tokens
    got = U.replay(r, steps)
    r.cache.manager.check()
    assert min(r.cache.manager.reuse_count(g) for g in r.cache.paged_groups()) > 0
    for i, s in enumerate(seqs):
        assert_rows(got[f"r{i}"], plain_logits(folder, s), "float32", f"request {i} in a pool of a few windows")


# ----------------------------------------------------------------------------------------------------------------
# the first tokens; a request beside others; long decoding
# ----------------------------------------------------------------------------------------------------------------
def test_first_tokens_one_by_one(backend, folders):
    for name, seed in (("R", 77), ("Q", 78), ("P", 79)):
        cfg = CONFIGS[name][0]
        folder = folders(name, "float32")
        seq = seqs_for(cfg, [12], seed=seed)[0]
        want = plain_logits(folder, seq)
        r = runner_for(folder, "float32", backend, 64)
        assert_rows(U.replay(r, U.tail_decode_trace([seq], 12))["r0"], want, "float32", f"{name}: token by token from the first")
        r = runner_for(folder, "float32", backend, 64)
        assert_rows(U.replay(r, U.chunk_trace([seq], sizes=(1, 2, 1, 3, 2, 1)))["r0"], want, "float32", f"{name}: the first tokens in portions")


def test_pages_of_a_request_that_ended_are_used_again(backend, folders):
    cfg = CONFIGS["P"][0]
    folder = folders("P", "float32")
    a, b, c = seqs_for(cfg, [63, 41, 58], seed=90)
    r = runner_for(folder, "float32", backend, 64, max_live=1)
    steps = U.whole_trace([a]) + [dict(s, step=1 + i) for i, s in enumerate(U.chunk_trace([b], sizes=(5, 2, 9)))]
    for i, s in enumerate(steps[1:]):      # (other names than the first request's)
        s["entries"][0]["id"], s["end"] = "second", (["second"] if s["end"] else [])
    got = U.replay(r, steps)
    assert_rows(got["second"], plain_logits(folder, b), "float32", "the second request in the first one's pages")
    got = U.replay(r, [dict(U.whole_trace([c])[0], step=99)])
    assert_rows(got["r0"], plain_logits(folder, c), "float32", "the third")
    r.cache.manager.check()


def test_unequal_requests_together_equal_each_alone(backend, folders):
    for name in ("Q", "P"):
        cfg = CONFIGS[name][0]
        folder = folders(name, "float32")
        seqs = seqs_for(cfg, [5, 40, 1, 17], seed=123)
        r = runner_for(folder, "float32", backend, 4 * 64)
        together = U.replay(r, [{"step": 0, "entries": [{"id": f"r{i}", "tokens": s, "want": list(range(len(s)))} for i, s in enumerate(seqs)],
                                 "end": [f"r{i}" for i in range(len(seqs))]}])
        alone = U.replay(runner_for(folder, "float32", backend, 64), U.whole_trace(seqs))
        for i in range(len(seqs)):
            if backend == "cpu":     # (the host's library products sum in an order that depends on the batch)
                assert_rows(together[f"r{i}"], alone[f"r{i}"], "float32", f"{name} request {i} beside the others", 1e-5)
            else:                    # every kernel sums a row in one order whatever else the step holds
                assert torch.equal(together[f"r{i}"], alone[f"r{i}"]), f"{name} request {i}: 32-bit logits depend on the batch"


def test_two_hundred_decoded_tokens(backend, folders):
    """A short prompt, then token after token for long: pages fill, windows pass on, first tokens stay."""
    cfg = CONFIGS["P"][0]
    folder = folders("P", "float32")
    n = 60 if backend == "cpu" else 230
    seq = seqs_for(cfg, [n], seed=600)[0]
    steps = U.tail_decode_trace([seq], n - 4)
    r = runner_for(folder, "float32", backend, U.max_live_tokens(steps))
    assert_rows(U.replay(r, steps)["r0"], plain_logits(folder, seq), "float32", "long decoding")


@pytest.mark.gpu
def test_decoded_tokens_of_a_batch_from_graphs(folders):
    """Steps of single tokens of four requests replayed from graphs, across pages, windows' and kept tokens' edges, with prompts
    between them, against the same steps kernel by kernel: the same bits, and the plain implementation's logits."""
    for name in ("P", "S"):
        cfg = all_experts(CONFIGS[name][0])
        for dtype in ("float32", "bfloat16"):
            folder = folders(name + "_graphs", dtype, cfg, CONFIGS[name][1])
            seqs = seqs_for(cfg, [150, 61, 97, 24], seed=700)
            steps, at = [], [6, 20, 50, 1]
            steps.append({"step": 0, "entries": [{"id": f"r{i}", "tokens": s[:at[i]], "want": list(range(at[i]))} for i, s in enumerate(seqs)], "end": []})
            while any(a < len(s) for a, s in zip(at, seqs)):
                live = [i for i in range(4) if at[i] < len(seqs[i])]
                n = 3 if len(steps) % 17 == 0 else 1        # (now and then a step of portions between the replays)
                entries = [{"id": f"r{i}", "tokens": seqs[i][at[i]:at[i] + n], "want": list(range(len(seqs[i][at[i]:at[i] + n])))} for i in live]
                for i in live:
                    at[i] += len(seqs[i][at[i]:at[i] + n])
                steps.append({"step": len(steps), "entries": entries, "end": [f"r{i}" for i in live if at[i] >= len(seqs[i])]})
            tokens = U.max_live_tokens(steps)
            got = U.replay(runner_for(folder, dtype, "cuda:0", tokens), steps)
            apart = U.replay(runner_for(folder, dtype, "cuda:0", tokens, graphs=False), steps)
            for i, s in enumerate(seqs):
                assert_rows(got[f"r{i}"], plain_logits(folder, s), dtype, f"{name} {dtype} request {i} from graphs")
                assert_rows(got[f"r{i}"], apart[f"r{i}"], dtype, f"{name} {dtype} request {i}: graphs against kernel by kernel", 1e-5 if dtype == "float32" else 0.04)


# ----------------------------------------------------------------------------------------------------------------
# generation through the engine's own entry point and scheduler
# ----------------------------------------------------------------------------------------------------------------
def test_greedy_generation_through_the_scheduler(backend, folders):
    from denno_beta_amd.config import EngineOptions
    from denno_beta_amd.engine import Engine, SamplingParams
    cfg = CONFIGS["P"][0]
    folder = folders("P", "float32")
    prompts = seqs_for(cfg, [3, 29, 11], seed=300)
    n_new = 10
    eng = Engine.from_folder(folder, EngineOptions(dtype="float32", device=backend, cache_tokens=4 * 64, max_live=2,
                                                   prefill_chunk=7, max_batch_tokens=16))
    got = eng.generate(prompts, SamplingParams(max_tokens=n_new, temperature=0.0))
    for p, g in zip(prompts, got):
        seq = list(p)
        for n, tok in enumerate(g):
            row = plain_logits(folder, seq)[-1]
            top = row.topk(2)
            if tok != int(top.indices[0]):
                assert float(top.values[0] - top.values[1]) < 1e-4 * float(row.std()), f"token {n} of {g}: the plain model says {int(top.indices[0])}"
            seq.append(tok)
        assert len(g) == n_new


# ----------------------------------------------------------------------------------------------------------------
# configuration and weights
# ----------------------------------------------------------------------------------------------------------------
def test_config_is_read_with_errors_that_name_the_key(folders):
    from denno_beta_amd.config import ConfigError, resolve_architecture
    from denno_beta_amd.models.fikupel import FikupelConfig, build_fikupel
    assert resolve_architecture({"architecture": "Fikupel"}).config_cls is FikupelConfig
    for path, match in ((("layers", 0, "mixer", "kv_heads"), "kv_heads"), (("layers", 1, "mixer", "q_rank"), "q_rank"), (("norm",), "norm"),
                        (("layers", 1, "mixer", "kv_rank"), "kv_rank"), (("layers", 0, "mixer", "scale"), "scale"),
                        (("layers", 1, "mlp", "router"), "router"), (("layers", 0, "mixer", "rot", "scaling", "high"), "high"),
                        (("layers", 0, "mixer", "mask", "size"), "size"), (("layers", 0, "mixer", "rot", "base"), "base"), (("layers", 0, "mlp", "ff"), "ff"),
                        (("vocab",), "vocab"), (("layers",), "layers")):
        bad = copy.deepcopy(CFG_P)
        d = bad
        for key in path[:-1]:
            d = d[key]
        del d[path[-1]]
        with pytest.raises(ConfigError, match=match):
            FikupelConfig.from_dict(bad)
    for path, value, match in ((("layers", 0, "type"), "something", "type"), (("layers", 0, "mixer", "rot", "dims"), 18, "rot.dims"),
                               (("layers", 0, "mixer", "rot", "dims"), 3, "rot.dims"), (("layers", 0, "mixer", "vdim"), 7, "vdim"),
                               (("layers", 0, "mixer", "kv_heads"), 3, "kv_heads"), (("layers", 1, "mlp", "router", "top"), 7, "router"),
                               (("layers", 0, "mixer", "rot", "scaling", "high"), 0.5, "high"), (("streams",), 0, "streams"),
                               (("layers", 1, "mixer", "mask", "keep_first"), 4, "keep_first"), (("layers", 1, "mlp", "kind"), "sparse", "kind")):
        bad = copy.deepcopy(CFG_P)
        d = bad
        for key in path[:-1]:
            d = d[key]
        d[path[-1]] = value
        with pytest.raises(ConfigError, match=match):
            FikupelConfig.from_dict(bad)
    # what config.json may leave out: copies of the stream, windows, kept tokens, stretching
    spec = build_fikupel(FikupelConfig.from_dict(CFG_R))
    assert spec.streams == 0 and spec.layers[0].arrangement == "pre_norm_plain" and spec.head_weight is None
    spec = build_fikupel(FikupelConfig.from_dict(CFG_Q))
    assert spec.streams == 1 and spec.layers[2].parts["mixer"][1]["window"] == 0 and spec.layers[4].parts["mixer"][1]["window"] == 0
    # caches: windows that keep first tokens are a kind of their own
    m = build_fikupel(FikupelConfig.from_dict(CFG_P)).instantiate()
    assert [(cs.window, cs.keep_first) for cs in m.cache_specs] == [(23, 5), (37, 0), (9, 33), (11, 0)]


def test_a_checkpoint_that_does_not_fit_is_reported_whole(folders, tmp_path):
    from safetensors.torch import load_file, save_file
    from denno_beta_amd.config import EngineOptions
    from denno_beta_amd.engine import ModelRunner
    from denno_beta_amd.weights import CheckpointError
    import shutil
    d = str(tmp_path / "m")
    shutil.copytree(folders("R", "float32"), d)
    tensors = load_file(os.path.join(d, "model.safetensors"))
    del tensors["l0.mlp.e1.gate"]
    tensors["l0.mix.temp"] = tensors["l0.mix.temp"][:1].contiguous()
    tensors["stray"] = torch.zeros(3)
    save_file(tensors, os.path.join(d, "model.safetensors"))
    with pytest.raises(CheckpointError) as e:
        ModelRunner.from_folder(d, EngineOptions(dtype="float32", device="cpu", cache_tokens=64, max_live=1))
    assert "l0.mlp.e1.gate" in e.value.missing and "stray" in e.value.unexpected and e.value.wrong_shape[0][0] == "l0.mix.temp"


# ----------------------------------------------------------------------------------------------------------------
# the command line and the trace runner as child processes
# ----------------------------------------------------------------------------------------------------------------
def plain_greedy(folder, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(plain_logits(folder, seq)[-1].argmax()))
    return seq[len(prompt):]


@pytest.mark.gpu
def test_command_line_generates_what_the_plain_model_does(folders):
    import subprocess
    import sys
    from conftest import ROOT
    folder = folders("R", "float32")
    prompt = seqs_for(CONFIGS["R"][0], [7], seed=410)[0]
    want = plain_greedy(folder, prompt, 6)
    out = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "denno"), "generate", folder, "--prompt-ids",
                          ",".join(map(str, prompt)), "--max-tokens", "6", "--temperature", "0", "--quant", "fp32", "--raw",
                          "--cache-tokens", "128"], capture_output=True, text=True, timeout=300)
    assert out.returncode == 0, out.stderr
    assert [int(t) for t in out.stdout.strip().split(",")] == want


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_as_a_child_process(folders, tmp_path, dtype):
    """bin/trace_run on a mixed trace with four requests alive: the files it writes against the plain implementation."""
    import subprocess
    from conftest import ROOT
    cfg = CONFIGS["P"][0] if dtype == "float32" else all_experts(CONFIGS["P"][0])
    folder = folders("P", dtype, cfg, CONFIGS["P"][1])
    seqs = seqs_for(cfg, [90, 3, 41, 17, 64, 29, 5], seed=500)
    steps = U.mixed_trace(seqs, seed=3, max_live=4)
    out = str(tmp_path / "out")
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", out, "--max-tokens",
                        str(U.max_live_tokens(steps))], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done ")] == [f"done {s['step']}" for s in steps]
    got = U.collect_files(out, steps, cfg["vocab"])
    for i, s in enumerate(seqs):
        assert_rows(got[f"r{i}"], plain_logits(folder, s), dtype, f"trace_run {dtype} request {i}")
