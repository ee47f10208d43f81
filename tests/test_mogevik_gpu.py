"""Mogevik on the engine against the plain implementation (tests/plain_mogevik.py): each mechanism alone through its
kernels and parts, then whole models through the step function (whole prompts, decoding token by token, portions down
to two tokens, mixed batches over a small pool whose pages and state slots come back and go out again), and greedy
generation through the engine's entry point and scheduler.  Sizes differ from test to test; where random numbers would
hide a fault (one far key among hundreds, a window's edge, a slope, a state that must last, a filter's inputs at a
portion's start) the inputs are made so that it shows.  In bfloat16 two experts of nearly equal scores may be ranked the
other way round: the engine reports its choices through the layer debug hook and the plain model follows them where they
are as good as its own."""
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import helpers
import plain_mogevik as P
from helpers import quick
from mogevik_models import CONFIG_D, CONFIG_E, CONFIG_F, att, config, layer, make_model, moe, rec, replay_routed

pytestmark = pytest.mark.gpu
DEV = helpers.DEVICE
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
TOL = {"float32": 2e-5, "bfloat16": 3e-2}
SLACK = {"float32": 1e-5, "bfloat16": 0.06}      # how far below the plain model's last choice an engine's choice may score
MIX = lambda d: d["mixer"]


def bf16(a):
    """What bfloat16 keeps of an array (as float64)."""
    return torch.tensor(np.asarray(a), dtype=torch.float32).to(torch.bfloat16).double().numpy()


def dev(a, dtype=torch.int32):
    return torch.tensor(np.asarray(a), dtype=dtype, device=DEV)


def host(t):
    return t.double().cpu().numpy()


def tb(a):
    return torch.tensor(np.asarray(a), dtype=torch.float32).to(torch.bfloat16)


# ------------------------------------------------------------------------------------------ mixers alone
def attention_weights(rng, m, width):
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    nrm = lambda *shape, s=0.2: rng.normal(size=shape) * s
    return {"mix.q": nrm(H * D, width), "mix.k": nrm(G * D, width), "mix.v": nrm(G * Dv, width), "mix.q.b": nrm(H * D, s=0.5),
            "mix.k.b": nrm(G * D, s=0.5), "mix.v.b": nrm(G * Dv, s=0.5), "mix.g": nrm(H * Dv, width, s=0.5), "mix.o": nrm(width, H * Dv)}


def recurrence_weights(rng, m, width):
    C, B, K = m["width"], m["blocks"], m["conv"]
    n = C // B
    nrm = lambda *shape, s=0.2: rng.normal(size=shape) * s
    return {"mix.y": nrm(C, width), "mix.y.b": nrm(C), "mix.x": nrm(C, width), "mix.x.b": nrm(C, s=0.5), "mix.conv": nrm(C, K, s=0.6),
            "mix.conv.b": nrm(C, s=0.3), "mix.ra": nrm(B, n, n, s=n ** -0.5), "mix.ra.b": nrm(B, n, s=1.0), "mix.ri": nrm(B, n, n, s=n ** -0.5),
            "mix.ri.b": nrm(B, n, s=1.0), "mix.lam": rng.uniform(-7.0, 2.0, size=C), "mix.o": nrm(width, C)}


def build_part(kind, m, width, W, dtype):
    from deliverance_amd.config.mogevik import head_slopes
    from deliverance_amd.config.specs import AttentionSpec, RealGatedRecurrenceSpec
    from deliverance_amd.parts import build_mixer
    t = lambda k: tb(W["mix." + k])
    if kind == "attention":
        spec = AttentionSpec("attention", width, m["heads"], m["kv_heads"], m["dim"], m["scale"], qkv_bias=True, out_bias=False,
                             window=(m["mask"] or {}).get("size"), v_head_dim=m["vdim"], out_gate="sigmoid", distance_slopes=head_slopes(m["heads"]))
        params = {"qkv_weight": torch.cat([t(k) for k in "qkvg"]), "out_weight": t("o"),
                  "qkv_bias": torch.cat([t("q.b"), t("k.b"), t("v.b"), torch.zeros(m["heads"] * m["vdim"], dtype=torch.bfloat16)])}
    else:
        spec = RealGatedRecurrenceSpec("real_gated_recurrence", width, m["width"], m["blocks"], m["conv"], 8.0)
        params = {"in_weight": torch.cat([t("y"), t("x")]), "in_bias": torch.cat([t("y.b"), t("x.b")]), "conv_weight": t("conv"),
                  "conv_bias": t("conv.b"), "gate_weight": torch.cat([t("ra"), t("ri")], 1), "gate_bias": torch.cat([t("ra.b"), t("ri.b")], 1),
                  "lam": t("lam"), "out_weight": t("o")}
    return build_mixer(spec, params, DTYPES[dtype], DEV)


class MixerBench:
    """One mixer part with weights of its own, fed with rows h of whole sequences in steps of any cut; its additions to
    the stream are compared with the plain mixer over the whole sequences.  Pages are handed out in a shuffled order and
    start as NaN; state slots are given in any order, and a slot may be used again after its sequence."""

    def __init__(self, dtype, kind, m, width, seqs, page=16, seed=0, make=None, slots=None):
        from deliverance_amd.parts import KVNeed
        rng = np.random.default_rng(seed)
        W = attention_weights(rng, m, width) if kind == "attention" else recurrence_weights(rng, m, width)
        if make is not None:
            make(W)
        self.W = {k: bf16(v) for k, v in W.items()}
        self.plain = (lambda h, W=self.W: P.attention(W, "", m, h)) if kind == "attention" else (lambda h, W=self.W: P.recurrent_block(W, "", h))
        self.width, self.dtype, self.page = width, dtype, page
        self.part = build_part(kind, m, width, self.W, dtype)
        self.seqs = [bf16(s) for s in seqs]                       # h of every sequence, [T, width]
        self.want = [self.plain(s) for s in self.seqs]
        need = self.part.cache_need()
        self.kv = self.state = None
        n_pages = sum(-(-len(s) // page) for s in seqs) + 3
        perm = torch.randperm(n_pages, generator=torch.Generator().manual_seed(7)).tolist()
        self.tables = [[perm.pop() for _ in range(-(-len(s) // page))] for s in seqs]
        if isinstance(need, KVNeed):
            shape = (2, need.n_kv_heads, page, need.head_dim) if need.v_head_dim is None else (need.n_kv_heads * page * (need.head_dim + need.v_head_dim),)
            self.kv = torch.full((n_pages, *shape), float("nan"), dtype=DTYPES[dtype], device=DEV)
        else:
            self.slots = list(slots) if slots is not None else list(range(len(seqs)))[::-1]
            self.state = torch.zeros(max(self.slots) + 2, need.elems, dtype=torch.float32, device=DEV)
        self.done = [0] * len(seqs)

    def step(self, takes):
        """takes: {sequence: number of next tokens}; returns the largest error of the step relative to the largest
        value of the plain result."""
        from deliverance_amd.parts import Arena, StepContext
        order = sorted(takes, key=lambda s: (takes[s] != 1, s))
        ctx = StepContext()
        ctx.device, ctx.dtype = torch.device(DEV), DTYPES[self.dtype]
        lens = [takes[s] for s in order]
        total = [self.done[s] + takes[s] for s in order]
        ctx.n_seqs, ctx.n_tokens, ctx.n_decode = len(order), sum(lens), sum(1 for n in lens if n == 1)
        mb = max(len(self.tables[s]) for s in order)
        bt = torch.full((len(order), mb), -1, dtype=torch.int32)
        pos, seq_of, rows, q_start = [], [], [], [0]
        for i, s in enumerate(order):
            bt[i, :len(self.tables[s])] = torch.tensor(self.tables[s], dtype=torch.int32)
            for p in range(self.done[s], total[i]):
                pos.append(p); seq_of.append(i); rows.append(self.tables[s][p // self.page] * self.page + p % self.page)
            q_start.append(len(pos))
        ctx.positions, ctx.seq_of_token, ctx.q_start, ctx.seq_lens = dev(pos), dev(seq_of), dev(q_start), dev(total)
        ctx.tokens = dev([0] * len(pos))
        ctx.q_start_host, ctx.seq_lens_host = q_start, total
        ctx.max_query_len, ctx.max_seq_len = max(lens), max(total)
        ctx.block_tables, ctx.slot_maps = [bt.to(DEV)], [dev(rows)]
        slots = [self.slots[s] for s in order] if self.state is not None else list(range(len(order)))
        ctx.state_slots, ctx.state_slots_host = dev(slots), slots
        ctx._arena = Arena(DEV)
        ctx.cache = SimpleNamespace(page_size=self.page, group_of_slot={0: 0}, kv={0: self.kv}, state={0: self.state})
        h = np.concatenate([self.seqs[s][self.done[s]:self.done[s] + takes[s]] for s in order])
        x = torch.zeros(len(h), self.width, dtype=torch.float32, device=DEV)
        self.part.forward(ctx, dev(h, DTYPES[self.dtype]), x, SimpleNamespace(layer=0, cache=0, write=True))
        want = np.concatenate([self.want[s][self.done[s]:self.done[s] + takes[s]] for s in order])
        for s in order:
            self.done[s] += takes[s]
        scale = max(np.abs(w).max() for w in self.want)
        return np.abs(host(x) - want).max() / scale


def walk(b, tol):
    """Three sequences of 70, 33 and 1 tokens in portions, decoded tokens and both at once."""
    assert b.step({0: 33, 1: 2}) <= tol                  # portions; the second ends inside a page
    assert b.step({0: 1, 1: 1, 2: 1}) <= tol             # decoding beside a first token
    assert b.step({0: 30, 1: 14}) <= tol                 # across a tile of 32 keys and page borders
    assert b.step({0: 1, 1: 1}) <= tol
    assert b.step({0: 5, 1: 15}) <= tol
    assert b.done == [70, 33, 1]


ATTENTIONS = [quick(MIX(att(4, 2, 16, 8, 0.25, 24))),      # matrix cores; the window ends inside pages
              MIX(att(3, 1, 12, 20, 0.3, 500)),            # a head size left to the plain kernel
              quick(MIX(att(2, 2, 64, 64, 0.125, 17))),    # values of the keys' size: decode rows on the decode kernel
              MIX(att(2, 1, 32, 128, 0.2, 33)),            # values four times the keys
              quick(MIX(att(6, 3, 32, 16, 0.2, 1))),       # a token sees itself only
              MIX(att(5, 1, 128, 64, 0.1, 32)),            # a window of two pages; five heads: odd slopes
              MIX(att(1, 1, 40, 72, 0.2, None)),           # every earlier key
              MIX(att(2, 1, 200, 24, 0.08, 33))]           # more entries than the matrix cores take
RECURRENCES = [quick(MIX(rec(48, 3, 4))),
               MIX(rec(60, 5, 3)),                         # blocks of 12 channels: the walking form
               quick(MIX(rec(40, 5, 1))),                  # blocks of 8; no earlier input in the filter
               quick(MIX(rec(192, 2, 2))),                 # blocks of 96: two workgroups a block in a portion
               MIX(rec(64, 1, 6)),                         # more taps than four
               MIX(rec(400, 2, 4)),                        # blocks of 200 channels
               MIX(rec(256, 1, 5)),                        # the widest block the matrix cores take
               MIX(rec(264, 1, 4))]                        # one that they do not take


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("m", ATTENTIONS)
def test_attention_part_prompt_portions_and_decoding(m, dtype):
    rng = np.random.default_rng(5)
    helpers.skip_in_simulation_if(m["dim"] > 100 and dtype == "float32")
    walk(MixerBench(dtype, "attention", m, 64, [rng.normal(size=(n, 64)) for n in (70, 33, 1)]), TOL[dtype])


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("m", RECURRENCES)
def test_recurrent_part_prompt_portions_and_decoding(m, dtype):
    """The state rows are handed out in any order."""
    rng = np.random.default_rng(7)
    helpers.skip_in_simulation_if(m["width"] > 200 and dtype == "float32")
    walk(MixerBench(dtype, "rglru", m, 48, [rng.normal(size=(n, 48)) for n in (70, 33, 1)], slots=[3, 0, 2]), TOL[dtype])


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("cut", [(300,), quick((64, 65, 2, 63, 1, 105)), (128, 3, 1, 1, 167), (2, 298), (255, 45)])
def test_recurrent_part_across_chunks(cut, dtype):
    """Portions of one, two and five chunks of tokens and of lengths at a chunk's edge, beside a portion that ends within
    the first chunk and one of three tokens (shorter than the filter)."""
    rng = np.random.default_rng(8)
    helpers.skip_in_simulation_if(dtype == "float32")
    b = MixerBench(dtype, "rglru", MIX(rec(48, 2, 5)), 32, [rng.normal(size=(300, 32)), rng.normal(size=(70, 32)), rng.normal(size=(11, 32))], slots=[1, 3, 0])
    for i, n in enumerate(cut):
        takes = {0: n}
        if i == 0:
            takes.update({1: 20, 2: 3})
        if i == 1:
            takes.update({1: 50, 2: 2})
        assert b.step(takes) <= TOL[dtype], f"portion {i}"
    assert b.done[0] == 300


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
def test_a_state_slot_that_is_used_again(dtype):
    """A second sequence in the slot of a first one that has ended: the engine clears a slot when it hands it out, so the
    second starts from zeros; without that its first outputs would be the first one's."""
    rng = np.random.default_rng(9)
    b = MixerBench(dtype, "rglru", MIX(rec(32, 2, 4)), 32, [rng.normal(size=(40, 32)), rng.normal(size=(40, 32))], slots=[1, 1])
    assert b.step({0: 39}) <= TOL[dtype] and b.step({0: 1}) <= TOL[dtype]
    left = b.state.clone()
    assert float(left[1].abs().max()) > 0.0 and float(left[0].abs().max()) == 0.0 and float(left[2].abs().max()) == 0.0
    assert b.step({1: 5}) > TOL[dtype]                   # what is left in the slot shows
    b.done[1] = 0
    b.state[1].zero_()
    assert b.step({1: 5}) <= TOL[dtype] and b.step({1: 1}) <= TOL[dtype] and b.step({1: 34}) <= TOL[dtype]


# ------------------------------------------------------------------------------------------ keys at a window's edge
def marked(W):
    """Input channel 0 makes a key, channel 1 a query of the same direction: of all pairs the one marked pair of tokens
    has by far the largest score, whatever it loses by its distance."""
    for k in ("mix.q", "mix.k"):
        W[k] *= 0.05
        W[k + ".b"] *= 0.05
    W["mix.k"][:, 0] = np.tile([1.0, -1.0], W["mix.k"].shape[0] // 2)
    W["mix.q"][:, 1] = np.tile([1.0, -1.0], W["mix.q"].shape[0] // 2)


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("vdim", [16, quick(24)])
@pytest.mark.parametrize("window,last", [quick(56, 167), (56, 63), (24, 240), quick(16, 48), (33, 65), (1, 20), (300, 260), (90, 178), (7, 200),
                                         (128, 255), (100, 201), (64, 300)])
def test_a_key_at_a_windows_edge(window, last, vdim, dtype):
    """The last query, at position ``last``, matches one key far better than any other: the oldest key that its window
    holds, then the one before that, which it must not see.  An edge that is one token off, or a key read from a page that
    was given back, shows as an error of the order of the output; in a prompt, in a portion and in decoding."""
    width, T = 32, last + 1
    oldest = max(0, last - window + 1)
    m = MIX(att(2, 1, 16, vdim, 8.0, window))
    for mark in [oldest] + ([oldest - 1] if oldest else []):
        if mark == last:
            continue
        rng = np.random.default_rng(window + last)
        h = rng.normal(size=(T, width)) * 0.1
        h[mark, 0] = 6.0
        h[last, 1] = 6.0
        cuts = [[T], [T - 1, 1], [max(oldest + 1, 1), T - max(oldest + 1, 1)], [max(oldest - 2, 1), T - max(oldest - 2, 1)]]
        for cut in cuts if not helpers.SIMT else cuts[:2]:
            b = MixerBench(dtype, "attention", m, width, [h], seed=1, make=marked)
            for n in [n for n in cut if n]:
                err = b.step({0: n})
                assert err <= TOL[dtype], f"mark {mark}, cut {cut}: {err}"
        # the test sees what it is meant to see: with an edge one token off the result at the last position is another
        keep = P.seen

        def off(T_, size):
            mask = keep(T_, size)
            mask[last, mark] = not mask[last, mark]
            return mask
        P.seen = off
        try:
            wrong = P.attention(b.W, "", m, b.seqs[0])[-1]
        finally:
            P.seen = keep
        right = b.want[0][-1]
        assert np.abs(wrong - right).max() > 0.2 * max(np.abs(wrong).max(), np.abs(right).max())


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim", [quick(4, 2, 16, 24), (4, 2, 16, 16), (3, 1, 12, 12), (8, 8, 32, 32)])
def test_every_head_has_a_slope_of_its_own_and_every_key_a_distance(heads, kv_heads, dim, vdim, dtype):
    """All keys are alike (their weights are zero, the bias is all there is), so the weights are the slopes alone; values
    differ from token to token.  Another head's slope, a distance that is one off for some keys, or slopes that the scale
    multiplies would show; so does a result at the 400th position that depends on how it came there."""
    T, width = 400, 32
    rng = np.random.default_rng(3)
    m = MIX(att(heads, kv_heads, dim, vdim, 0.25, 350))

    def make(W):
        W["mix.k"][:] = 0.0
        W["mix.g"] *= 0.1
    b = MixerBench(dtype, "attention", m, width, [rng.normal(size=(T, width))], seed=2, make=make)
    for change in (lambda s: np.roll(s, 1), lambda s: s * 0.25, lambda s: -s * 0.0):
        keep = P.head_slopes
        P.head_slopes = lambda H: change(keep(H))
        try:
            wrong = P.attention(b.W, "", m, b.seqs[0])
        finally:
            P.head_slopes = keep
        assert np.abs(wrong - b.want[0]).max() > 0.1 * np.abs(b.want[0]).max()
    cuts = [(T - 3, 1, 1, 1), (100, 2, 197, 1, 100)] if not helpers.SIMT else [(30, 1, 1)]
    for cut in cuts:
        b.done = [0]
        b.kv.fill_(float("nan"))
        for n in cut:
            assert b.step({0: n}) <= TOL[dtype]


# ------------------------------------------------------------------------------------------ the recurrence
def test_the_recurrence_remembers_the_first_token():
    """Channels whose decays are nearly 1 keep the first token's input; after 300 tokens, cut into portions and decoded
    tokens, it is still there; the channels beside them have forgotten it."""
    T, width = 300, 32
    rng = np.random.default_rng(8)
    h = rng.normal(size=(T, width)) * 0.02
    h[0, 0] = 30.0
    m = MIX(rec(32, 2, 4))

    def make(W):
        W["mix.x"][:, 0] = 1.0
        W["mix.x"][:, 1:] *= 0.1
        W["mix.x.b"][:] = 0.0
        W["mix.conv.b"][:] = 0.0
        W["mix.y.b"][:] = 1.0
        W["mix.y"][:, 0] = 0.0
        W["mix.o"][:, 16:] *= 0.02                             # (their share of the result: small)
        W["mix.ra"] *= 0.02
        W["mix.lam"][:16] = -10.0
        W["mix.lam"][16:] = 1.0
    for dtype in ("float32", "bfloat16"):
        b = MixerBench(dtype, "rglru", m, width, [h], seed=3, make=make, slots=[1])
        lost = dict(b.W)
        lost["mix.lam"] = np.where(b.W["mix.lam"] < 0, -6.0, b.W["mix.lam"])        # a little forgetting already shows
        assert np.abs(P.recurrent_block(lost, "", b.seqs[0])[-1] - b.want[0][-1]).max() > 0.2 * np.abs(b.want[0][-1]).max()
        assert np.abs(b.want[0][-1]).max() > 0.1 * np.abs(b.want[0]).max()
        for n in (150, 2, 100, 1, 1, 44, 1, 1):
            assert b.step({0: n}) <= TOL[dtype]
        assert b.done == [T]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_filters_inputs_at_a_portions_start(dtype):
    """One token's input is far larger than any other: the three tokens behind it see it through the filter, whether they
    come in the same portion, in the next one, or one by one; with it lost, or one place off, they would not."""
    width = 32
    rng = np.random.default_rng(11)
    h = rng.normal(size=(40, width)) * 0.05
    h[20, 0] = 20.0
    m = MIX(rec(32, 2, 4))

    def make(W):
        W["mix.x"][:, 0] = 1.0
        W["mix.lam"][:] = 3.0                                  # the state forgets at once: only the filter carries it on
        W["mix.y.b"][:] = 1.0
    for cut in ((40,), (21, 19), (20, 2, 18), (20, 1, 1, 1, 1, 16), (22, 18), (18, 2, 2, 2, 2, 14), (21, 1, 18)):
        b = MixerBench(dtype, "rglru", m, width, [h], seed=4, make=make)
        far = np.abs(b.want[0][21:24]).max(1) / np.abs(b.want[0][25:]).max()
        assert (far > 3.0).all(), far
        for n in cut:
            assert b.step({0: n}) <= TOL[dtype], cut


@pytest.mark.parametrize("bs,blocks,K,lam", [quick(64, 2, 4, (-7.0, 2.0)), quick(16, 3, 1, (-30.0, 30.0)), (8, 1, 2, (-3.0, 3.0)), (40, 2, 16, (-7.0, 2.0)),
                                             (128, 1, 3, (-12.0, -8.0)), (72, 2, 4, (4.0, 20.0)), (256, 1, 7, (-7.0, 2.0))])
def test_the_forms_for_serving_against_the_recurrence(bs, blocks, K, lam):
    """Portions of many lengths (inside a tile of 16 tokens, at its edge, at a chunk's edge and past it) and one-token
    sequences, from given states and filter inputs, with rates from ones whose decay is 1 to ones that leave nothing.
    The outputs and the states that are kept against the recurrence written out; states that nobody has, and states that
    are not to be written, stay as they are."""
    from deliverance_amd.kernels import ops
    from deliverance_amd.parts import Arena
    rng = np.random.default_rng(bs + K)
    lens = [1] * 18 + [2, 15, 16, 17, 63, 64, 65, 200] if not helpers.SIMT else [1, 1, 1, 2, 17, 66]
    nd, S, N, C = sum(n == 1 for n in lens), len(lens), sum(lens), bs * blocks
    for longest in (200, 64):                            # with and without portions of several chunks
        ls = [n for n in lens if n <= longest]
        S, N = len(ls), sum(ls)
        yx = bf16(rng.normal(size=(N, 2 * C)))
        conv, conv_b = bf16(rng.normal(size=(C, K)) * 0.6), bf16(rng.normal(size=C) * 0.3)
        gates, gates_b = bf16(rng.normal(size=(blocks, 2 * bs, bs)) * bs ** -0.5), bf16(rng.normal(size=(blocks, 2 * bs)))
        lam_v = rng.uniform(*lam, size=C)
        rate = (-8.0 * P.softplus(lam_v)).astype(np.float32)
        state0 = np.concatenate([rng.normal(size=(S + 1, C)), bf16(rng.normal(size=(S + 1, (K - 1) * C)))], 1).astype(np.float32)
        slots = rng.permutation(S + 1)[:S]
        slots[1] = -1
        if S > 19:
            slots[19] = -1
        q_start = np.concatenate([[0], np.cumsum(ls)])
        want, kept = np.zeros((N, C)), state0.astype(np.float64)
        for i in range(S):
            rows = slice(q_start[i], q_start[i + 1])
            st = kept[slots[i]] if slots[i] >= 0 else np.zeros(K * C)
            x = np.concatenate([st[C:].reshape(K - 1, C), yx[rows, C:]])
            u = bf16(P.causal_filter(x, conv, conv_b)[K - 1:])
            r = P.per_block(u, gates[:, :bs], gates_b[:, :bs])
            g = P.per_block(u, gates[:, bs:], gates_b[:, bs:])
            a = np.exp(rate.astype(np.float64) * P.logistic(r))
            add = np.sqrt(-np.expm1(2 * rate.astype(np.float64) * P.logistic(r))) * P.logistic(g) * u
            s = st[:C].copy()
            for t in range(ls[i]):
                s = a[t] * s + add[t]
                want[q_start[i] + t] = s * P.gelu_tanh(yx[q_start[i] + t, :C])
            if slots[i] >= 0:
                kept[slots[i]] = np.concatenate([s, x[len(x) - (K - 1):].reshape(-1)])
        ctx = SimpleNamespace(q_start=dev(q_start), state_slots=dev(slots), n_seqs=S, n_decode=nd, max_query_len=max(ls), buf=Arena(DEV).get)
        for write in (True, False):
            st = dev(state0, torch.float32)
            out = torch.full((N, C + 8), 7.0, dtype=torch.bfloat16, device=DEV)
            dyx = dev(yx, torch.bfloat16)
            assert ops.rglru_serve_takes(dyx, bs)
            ops.rglru_serve(ctx, dyx, dev(conv.T.copy(), torch.float32), dev(conv_b, torch.float32), dev(gates, torch.bfloat16),
                            dev(gates_b, torch.float32), dev(rate, torch.float32), "gelu_pytorch_tanh", st, out[:, :C], write=write)
            err = np.abs(host(out)[:, :C] - want)
            # (u is rounded to bfloat16 where the filter's sum lies: a sum in another order may round to the neighbour)
            assert err.max() <= 2.0 ** -6 * np.abs(want).max(), f"outputs: {err.max()} at row {int(err.max(1).argmax())}"
            assert float((out[:, C:] - 7.0).abs().max()) == 0.0
            ref = kept if write else state0.astype(np.float64)
            got = host(st)
            assert np.abs(got[:, C:] - ref[:, C:]).max(initial=0.0) == 0.0, f"filter inputs, write={write}"
            assert np.abs(got[:, :C] - ref[:, :C]).max() <= 1e-2 * np.abs(ref[:, :C]).max(), f"states, write={write}"
            assert np.sqrt(((got[:, :C] - ref[:, :C]) ** 2).mean()) <= 5e-4 * np.abs(ref[:, :C]).max(), f"states, write={write}"


def test_a_token_in_a_batch_is_the_token_alone():
    """Decode rows of many sequences at once give the bits of each alone, and a portion gives the bits of that portion
    beside others."""
    from deliverance_amd.kernels import ops
    from deliverance_amd.parts import Arena
    helpers.skip_in_simulation_if(True)
    rng = np.random.default_rng(2)
    C, bs, K, S = 64, 32, 4, 37
    W = (dev(rng.normal(size=(K, C)), torch.float32), dev(rng.normal(size=C), torch.float32), dev(rng.normal(size=(2, 64, 32)) * 0.2, torch.bfloat16),
         dev(rng.normal(size=(2, 64)), torch.float32), dev(-np.exp(rng.normal(size=C)), torch.float32))

    def go(yx, lens, st):
        q = np.concatenate([[0], np.cumsum(lens)])
        ctx = SimpleNamespace(q_start=dev(q), state_slots=dev(np.arange(len(lens))), n_seqs=len(lens), n_decode=sum(n == 1 for n in lens),
                              max_query_len=max(lens), buf=Arena(DEV).get)
        out = torch.zeros(len(yx), C, dtype=torch.bfloat16, device=DEV)
        ops.rglru_serve(ctx, yx, *W, "gelu_pytorch_tanh", st, out)
        return out
    lens = [1] * S + [5, 30, 200]
    yx = dev(rng.normal(size=(sum(lens), 2 * C)), torch.bfloat16)
    state = dev(rng.normal(size=(len(lens), K * C)), torch.float32)
    both = state.clone()
    out = go(yx, lens, both)
    at = 0
    for i, n in enumerate(lens):
        one = state[i:i + 1].clone()
        alone = go(yx[at:at + n].contiguous(), [n], one)
        if n != 5 and n != 30:          # (a portion within a chunk is not cut when nothing beside it is longer)
            assert torch.equal(alone, out[at:at + n]) and torch.equal(one[0], both[i]), f"sequence {i}"
        else:
            assert float((alone.float() - out[at:at + n].float()).abs().max()) <= 2.0 ** -7 * float(alone.float().abs().max())
        at += n


# ------------------------------------------------------------------------------------------ experts
@pytest.mark.parametrize("experts,top,groups", [(10, 4, None), quick(12, 3, (4, 2)), (3, 3, None), (1, 1, (1, 1)), quick(14, 2, (2, 1)), (70, 7, (7, 3)),
                                                (300, 5, (100, 40)), (1024, 8, (8, 2)), (64, 64, None), (8, 2, (8, 2))])
def test_the_choice_of_experts(experts, top, groups):
    """Corrections of both signs, large enough to decide; scores that tie (the lower index comes first); choice scores
    below zero, so that an entry outside the kept groups must count as less than any number."""
    from deliverance_amd.kernels import ops
    helpers.skip_in_simulation_if(experts > 200)
    rng = np.random.default_rng(experts)
    N = 37
    z = (rng.normal(size=(N, experts)) * 2).astype(np.float32)
    for corr in (rng.normal(size=experts) * 0.2, np.full(experts, -2.0), np.linspace(-1.0, 1.0, experts), np.zeros(experts)):
        corr = corr.astype(np.float32)
        z[3, :] = 0.25                                          # every logit the same
        ids = torch.zeros(N, top, dtype=torch.int32, device=DEV)
        w = torch.zeros(N, top, dtype=torch.float32, device=DEV)
        wide = torch.cat([dev(z, torch.float32), torch.full((N, 2), 99.0, device=DEV)], 1)
        ops.moe_choose(wide, experts, dev(corr, torch.float32), top, groups[0] if groups else 0, groups[1] if groups else 0, ids, w)
        g = None if groups is None else {"count": groups[0], "keep": groups[1]}
        want_ids, want_w = P.choose(z.astype(np.float64), corr.astype(np.float64), top, g)
        got = ids.cpu().numpy()
        c = P.softmax(z.astype(np.float64)) + corr
        for t in range(N):                                      # (32-bit scores may tie where these do not)
            assert got[t].tolist() == want_ids[t].tolist() or P.nearly_as_good(c[t], got[t].tolist(), g, 3e-7), t
        assert got[3].tolist() == want_ids[3].tolist() or corr.any()
        want_w = P.weights_of(P.softmax(z.astype(np.float64)), got)
        assert np.abs(host(w) - want_w).max() <= 2e-6


@pytest.mark.parametrize("rows,experts,ident,top,groups,extra", [quick(5, 6, 2, 3, (4, 2), 2), (1, 1, 0, 1, None, 1), (13, 9, 3, 4, (3, 2), 0), (16, 8, 2, 2, (2, 1), 2),
                                                                 (11, 50, 14, 6, (16, 5), 4), (2, 3, 5, 2, None, 3)])
def test_the_choice_and_the_layout_in_one_launch(rows, experts, ident, top, groups, extra):
    """The same ids and weights as the choice alone, ids of experts that hand their input on moved up, the further experts'
    pairs behind them with a logistic weight; every pair of an expert with matrices in a slot of its expert's tiles."""
    from deliverance_amd.kernels import ops
    rng = np.random.default_rng(rows)
    E, each, tile = experts + ident, top + extra, 32
    z = dev(rng.normal(size=(rows, E + 1)) * 2, torch.float32)
    corr = dev(rng.normal(size=E) * 0.3, torch.float32)
    g = groups or (0, 0)
    i1, w1 = torch.zeros(rows, top, dtype=torch.int32, device=DEV), torch.zeros(rows, top, dtype=torch.float32, device=DEV)
    ops.moe_choose(z, E, corr, top, *g, i1, w1)
    tiles, space = ops.moe_slot_space(rows, each, experts + extra, tile)
    i2, w2 = torch.full((rows, each), -7, dtype=torch.int32, device=DEV), torch.zeros(rows, each, dtype=torch.float32, device=DEV)
    slot, row_of, tile_of = (torch.full((n,), -9, dtype=torch.int32, device=DEV) for n in (rows * each, space, tiles))
    ops.moe_choose_route(ops.ExpertChoice(z, E, corr, *g), top, extra, experts, tile, i2, w2, slot, row_of, tile_of, rows)
    i1, i2, slot, row_of, tile_of = (t.cpu().numpy() for t in (i1, i2, slot, row_of, tile_of))
    assert np.array_equal(i2[:, :top], np.where(i1 < experts, i1, i1 + extra)) and torch.equal(w2[:, :top].contiguous(), w1)
    assert np.array_equal(i2[:, top:], np.tile(np.arange(experts, experts + extra), (rows, 1)))
    if extra:
        assert np.abs(host(w2)[:, top:] - P.logistic(host(z)[:, E:])).max() <= 1e-6
    slot, used = slot.reshape(rows, each), set()
    for n in range(rows):
        for k in range(each):
            if i2[n, k] >= experts + extra:
                assert slot[n, k] == -1
            else:
                assert row_of[slot[n, k]] == n and tile_of[slot[n, k] // tile] == i2[n, k] and slot[n, k] not in used
                used.add(slot[n, k])
    assert all(row_of[i] == -1 for i in range(space) if i not in used)
    # the choice alone, with the further experts behind it
    i5, w5 = torch.zeros(rows, each, dtype=torch.int32, device=DEV), torch.zeros_like(w2)
    ops.moe_choose(z, E, corr, top, *g, i5, w5, extra, experts)
    assert np.array_equal(i5.cpu().numpy(), i2) and float((w5 - w2).abs().max()) <= 1e-6
    # ... and with the router's product inside (a step of few tokens)
    h, router = bf16(rng.normal(size=(rows, 1104))), bf16(rng.normal(size=(E + 1, 1104)) * 0.1)
    zz = dev((h @ router.T).astype(np.float32), torch.float32)
    i3, w3, i4, w4 = torch.zeros(rows, each, dtype=torch.int32, device=DEV), torch.zeros_like(w2), torch.zeros(rows, each, dtype=torch.int32, device=DEV), torch.zeros_like(w2)
    lay = [torch.full((n,), -9, dtype=torch.int32, device=DEV) for n in (rows * each, space, tiles)]
    ops.moe_choose_route(ops.ExpertChoice(zz, E, corr, *g), top, extra, experts, tile, i3, w3, *lay, rows)
    ops.moe_choose_route(ops.ExpertChoice(torch.full_like(zz, float("nan")), E, corr, *g, dev(router, torch.bfloat16)), top, extra, experts, tile,
                         i4, w4, *lay, rows, dev(h, torch.bfloat16))
    same = (i3 == i4).all(1)                            # (two scores may lie within rounding of one another)
    assert int((~same).sum()) <= 1 and (not bool(same.any()) or float((w3 - w4)[same].abs().max()) <= 1e-5)


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("rows,width,centre", [quick(5, 52, True), (3, 320, True), (700, 768, True), (2, 1600, True), (9, 4096, False), quick(4, 64, False)])
def test_the_pairs_sum_the_streams_additions_and_the_next_norm_in_one_pass(rows, width, centre, dtype):
    from deliverance_amd.kernels import ops
    helpers.skip_in_simulation_if(rows > 100)
    rng = np.random.default_rng(width)
    top, slots = 3, 40
    out, y0 = rng.normal(size=(slots, width)).astype(np.float32), rng.normal(size=(rows, width)).astype(np.float32)
    slot = rng.integers(-1, slots, size=(rows, top))
    w = rng.random(size=(rows, top)).astype(np.float32)
    h, shared, gate = bf16(rng.normal(size=(rows, width))), rng.normal(size=(rows, width)).astype(np.float32), rng.normal(size=(rows, 5)).astype(np.float32)
    add, vec = rng.normal(size=(rows, width)).astype(np.float32), rng.normal(size=width).astype(np.float32)
    gain, bias = bf16(1 + 0.2 * rng.normal(size=width)), bf16(rng.normal(size=width))
    f = lambda a: dev(a, torch.float32)
    for full in (True, False):
        y = f(y0)
        nxt = torch.zeros(rows, width, dtype=DTYPES[dtype], device=DEV)
        ops.moe_combine_norm(f(out), dev(slot), f(w) if full else None, 0.5, top, y, full, dev(h, DTYPES[dtype]) if full else None,
                             f(shared) if full else None, f(gate)[:, 3:] if full else None, f(add) if full else None, f(vec) if full else None,
                             (centre, dev(gain, torch.bfloat16), dev(bias, torch.bfloat16) if full else None, 0.25, 1e-3), nxt)
        want = y0.astype(np.float64) if full else np.zeros((rows, width))
        for n in range(rows):
            for k in range(top):
                wk = w[n, k] if full else 0.5
                if slot[n, k] >= 0:
                    want[n] += wk * out[slot[n, k]]
                elif full:
                    want[n] += wk * h[n]
        if full:
            want += P.logistic(gate[:, 3:4].astype(np.float64)) * shared + add + vec
        assert np.abs(host(y) - want).max() <= 1e-5
        d = want - (want.mean(1, keepdims=True) if centre else 0.0)
        normed = d / np.sqrt((d * d).mean(1, keepdims=True) + 1e-3) * (0.25 + gain) + (bias if full else 0.0)
        assert np.abs(host(nxt) - normed).max() <= (2e-5 if dtype == "float32" else 2.0 ** -8) * np.abs(normed).max()


EXPERTS = [quick(9, moe(7, 3, 24, identity=2, groups=(3, 2), shared=48)), (150, moe(7, 3, 24, identity=2, groups=(3, 2), shared=48)),
           quick(20, moe(4, 2, 32, shared=40)), (600, moe(4, 2, 32, shared=40)), (6, moe(1, 1, 40)), (33, moe(2, 2, 16, identity=4, groups=(1, 1), shared=16)),
           (70, moe(3, 4, 20, identity=1, groups=(2, 2), shared=12)), (1, moe(12, 5, 8, identity=3, groups=(5, 3), shared=24)),
           quick(40, moe(2, 1, 24, identity=14)), (300, moe(6, 2, 64, shared=64))]


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("rows,mlp", EXPERTS)
@pytest.mark.parametrize("store", [False, True])
def test_experts_part(dtype, rows, mlp, store):
    """Few rows (the grouped kernels that stream an expert's weights) and many (rows gathered by expert); experts that
    hand their input on, also ones that most tokens choose; a shared expert whose gate is one number a token, of the
    others' size, a multiple of it and neither; added into a stream and stored."""
    helpers.skip_in_simulation_if(rows > 100)
    width = 64 if mlp["expert"]["ff"] % 8 == 0 else 52
    ro = mlp["router"]
    n, top, ff, ident, shared = ro["experts"], ro["top"], mlp["expert"]["ff"], ro.get("identity", 0), (mlp["shared"] or {}).get("ff", 0)
    rng = np.random.default_rng(rows + n)
    W = {"router": bf16(rng.normal(size=(n + ident, width)) * 0.4), "correction": bf16(rng.normal(size=n + ident) * 0.2)}
    for e in [f"e{j}" for j in range(n)] + (["shared"] if shared else []):
        f = shared if e == "shared" else ff
        W.update({f"{e}.gate": bf16(rng.normal(size=(f, width)) * 0.3), f"{e}.up": bf16(rng.normal(size=(f, width)) * 0.3),
                  f"{e}.down": bf16(rng.normal(size=(width, f)) * 0.2)})
    if shared:
        W["shared.sg"] = bf16(rng.normal(size=(1, width)) * 0.5)
    h, x0 = bf16(rng.normal(size=(rows, width))), rng.normal(size=(rows, width)).astype(np.float32)
    from deliverance_amd.config.specs import ExpertsFeedForwardSpec
    from deliverance_amd.parts import Arena, StepContext, build_feed_forward
    gr = ro.get("groups") or {"count": 0, "keep": 0}
    spec = ExpertsFeedForwardSpec("experts", width, ff, n, top, "silu", router="softmax_all", groups=gr["count"], groups_kept=gr["keep"],
                                  identity=ident, shared_inner=shared, shared_activation="silu", shared_gated=True, shared_token_gate=True)
    both = lambda e: torch.cat([tb(W[e + ".gate"]), tb(W[e + ".up"])])
    params = {"gate_up_weight": torch.stack([both(f"e{j}") for j in range(n)]), "down_weight": torch.stack([tb(W[f"e{j}.down"]) for j in range(n)]),
              "router_weight": tb(W["router"]), "router_correction": tb(W["correction"])}
    if shared:
        params.update(shared_gate_up_weight=both("shared"), shared_down_weight=tb(W["shared.down"]), shared_token_gate=tb(W["shared.sg"]))
    part = build_feed_forward(spec, params, DTYPES[dtype], DEV)
    ctx = StepContext()
    ctx.device, ctx.dtype, ctx.n_tokens, ctx._arena = torch.device(DEV), DTYPES[dtype], rows, Arena(DEV)
    ctx.tokens, ctx.part_accumulate = dev([0] * rows), not store
    ctx.debug_hook = lambda *a: None                        # so that the part keeps its choice
    x = dev(x0, torch.float32)
    part.forward(ctx, dev(h, DTYPES[dtype]), x)
    ctx.debug_hook = None
    x2 = dev(x0, torch.float32)
    part.last_choice, chosen = None, {t: [int(e) for e in row] for t, row in enumerate(part.last_choice.cpu().numpy())}
    part.forward(ctx, dev(h, DTYPES[dtype]), x2)
    assert part.last_choice is None and torch.equal(x, x2)
    want = P.experts(W, "", mlp, h, routes=chosen, slack=SLACK[dtype])
    err = np.abs(host(x) - (0 if store else x0) - want)
    assert err.max() <= (3e-6 if dtype == "float32" else 2e-2) * np.abs(want).max()


def test_kernels_refuse_what_they_cannot_take():
    from deliverance_amd.kernels import ops
    z, w = torch.zeros(2, 6, device=DEV), torch.zeros(2, 4, device=DEV)
    ids = torch.zeros(2, 4, dtype=torch.int32, device=DEV)
    with pytest.raises(ops.KernelError, match="groups"):
        ops.moe_choose(z, 6, torch.zeros(6, device=DEV), 4, 2, 1, ids, w)
    with pytest.raises(ops.KernelError, match="groups"):
        ops.moe_choose(z, 6, torch.zeros(6, device=DEV), 2, 4, 1, ids, w)
    with pytest.raises(ops.KernelError, match="correction"):
        ops.moe_choose(z, 6, torch.zeros(5, device=DEV), 2, 0, 0, ids, w)
    ctx = SimpleNamespace(q_start=dev([0, 2]), state_slots=dev([0]), n_seqs=1, n_decode=0, max_query_len=2, buf=lambda *a: None)
    yx = torch.zeros(2, 32, dtype=torch.bfloat16, device=DEV)
    f = lambda *s: torch.zeros(*s, device=DEV)
    gates = torch.zeros(1, 32, 16, dtype=torch.bfloat16, device=DEV)
    with pytest.raises(ops.KernelError, match="state row"):
        ops.rglru_serve(ctx, yx, f(4, 16), f(16), gates, f(1, 32), f(16), "silu", f(1, 48), torch.zeros(2, 16, dtype=torch.bfloat16, device=DEV))
    with pytest.raises(ops.KernelError, match="gate_w"):
        ops.rglru_serve(ctx, yx, f(4, 16), f(16), gates[:, :16].contiguous(), f(1, 32), f(16), "silu", f(1, 64),
                        torch.zeros(2, 16, dtype=torch.bfloat16, device=DEV))
    assert not ops.rglru_serve_takes(yx, 12) and not ops.rglru_serve_takes(yx, 264) and ops.rglru_serve_takes(yx, 256)
    with pytest.raises(ops.KernelError, match="slopes"):
        ops.attention_rel_ref(yx, torch.zeros(1, 512, dtype=torch.bfloat16, device=DEV), dev([[0]]), dev([0, 0]), dev([0, 1]), 2, 1, 16, 16, 16, 1.0,
                              None, None, 0.0, 0, torch.zeros_like(yx), slopes=f(3))
    with pytest.raises(ops.KernelError, match="add_rows"):
        ops.add_rows(f(2, 8), f(1, 8), None)


@pytest.mark.parametrize("rows,width", [quick(3, 50), (70, 64), (1, 7)])
def test_adding_the_embedding_output_and_a_vector(rows, width):
    from deliverance_amd.kernels import ops
    rng = np.random.default_rng(width)
    x, e, v = (rng.normal(size=s).astype(np.float32) for s in ((rows, width), (rows, width), (width,)))
    for src, vec in ((e, v), (e, None), (None, v)):
        got = ops.add_rows(dev(x, torch.float32), None if src is None else dev(src, torch.float32), None if vec is None else dev(vec, torch.float32))
        want = x.astype(np.float64) + (0 if src is None else src) + (0 if vec is None else vec)
        assert np.abs(host(got) - want).max() <= 1e-6


# ------------------------------------------------------------------------------------------ whole models
@pytest.fixture(scope="module")
def mmodels(tmp_path_factory):
    return {"D": make_model(tmp_path_factory.mktemp("md"), CONFIG_D, 61), "E": make_model(tmp_path_factory.mktemp("me"), CONFIG_E, 62),
            "F": make_model(tmp_path_factory.mktemp("mf"), CONFIG_F, 63)}


def check(model, got, routes, requests, dtype, what=""):
    """32-bit: every logit within 3e-5 of the largest plain logit.  bfloat16: the largest error within 6 % of the logits'
    root mean square and the rms error within 2^-6 of it.  The plain model follows the engine's choice of experts where
    two scores are nearly equal, and fails where the engine's choice is not nearly as good as its own."""
    for rid, ids in requests:
        ref = model.plain_logits(ids, routes.get(rid, {}), SLACK[dtype])
        out = got[rid].astype(np.float64)
        assert out.shape == ref.shape, f"{what} {rid}: shape {out.shape} vs {ref.shape}"
        err = np.abs(out - ref)
        rms = float(np.sqrt((ref ** 2).mean()))
        bound = 3e-5 * np.abs(ref).max() if dtype == "float32" else 6e-2 * rms
        over = err.max(axis=1) > bound
        first = int(np.argmax(over))
        assert not over.any(), f"{what} {rid} ({dtype}): max error {err[first].max():.3e} > {bound:.3e}, first at position {first}"
        if dtype == "bfloat16":
            assert float(np.sqrt((err ** 2).mean())) <= 2.0 ** -6 * rms, f"{what} {rid}: rms error"


def run(model, session, steps, requests, dtype, what):
    got, routes = replay_routed(session, steps, model.cfg)
    check(model, got, routes, requests, dtype, what)
    return got


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("name", [quick("D"), "E", "F"])
def test_whole_prompts_and_first_tokens(mmodels, name, dtype):
    m = mmodels[name]
    reqs = [("one", m.prompt(1)), ("two", m.prompt(2)), ("three", m.prompt(3)), ("long", m.prompt(90))]
    s = helpers.trace_session(m.folder, dtype, 256, state_slots=2)
    for rid, ids in reqs:
        run(m, s, helpers.trace_whole(rid, ids), [(rid, ids)], dtype, "whole")
    s.cache.manager.check()


def test_the_model_tests_see_the_loop_the_norm_and_the_pieces(mmodels):
    """What the whole-model comparisons stand for: with one of the design's steps left out or done elsewhere the plain
    model's logits move by far more than the bounds."""
    m = mmodels["D"]
    ids = m.prompt(30)
    ref = m.plain_logits(ids)
    rms = float(np.sqrt((ref ** 2).mean()))

    def moved(cfg=None, **changes):
        W = dict(m.W)
        W.update(changes)
        return float(np.abs(P.forward(cfg or m.plain_cfg, W, ids) - ref).max()) / rms
    loops = m.W["loop.step"]
    assert moved(**{"loop.step": np.zeros_like(loops)}) > 0.2 and moved(**{"loop.step": loops[[1, 2, 0]]}) > 0.2
    assert moved(cfg=dict(m.plain_cfg, loop={"start": 1, "stop": 3, "times": 2})) > 0.2
    assert moved(**{"l0.mlp.correction": np.zeros(9)}) > 0.1 and moved(**{"l0.mlp.shared.sg": np.zeros((1, 64))}) > 0.1
    assert moved(**{"l0.mix.conv.b": np.zeros(48)}) > 0.06 and moved(**{"l1.mix.v.b": np.zeros(48)}) > 0.06


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("name", ["D", quick("E"), "F"])
def test_prefill_against_token_by_token_decoding(mmodels, name, dtype):
    """All but the last 45 tokens at once, the rest one by one, across page borders, tiles of keys and the windows'
    edges; then a request that is decoded from its very first token on."""
    m = mmodels[name]
    ids = m.prompt(75, salt=1)
    s = helpers.trace_session(m.folder, dtype, 128, state_slots=1)
    run(m, s, helpers.trace_bulk_then_single("r", ids, tail=45), [("r", ids)], dtype, "decode")
    ids2 = m.prompt(20, salt=2)
    run(m, s, helpers.trace_bulk_then_single("q", ids2, tail=19), [("q", ids2)], dtype, "decode from 1")


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("name", [quick("D"), "E", "F"])
@pytest.mark.parametrize("sizes", [(7, 2, 13, 3, 5, 2), quick((2, 2, 31, 1, 16, 33, 2))])
def test_portions_of_any_size(mmodels, name, dtype, sizes):
    m = mmodels[name]
    ids = m.prompt(97, salt=3)
    s = helpers.trace_session(m.folder, dtype, 128, poison_freed=True, state_slots=1)
    run(m, s, helpers.trace_portions("r", ids, sizes), [("r", ids)], dtype, f"portions {sizes}")


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("name", ["D", quick("E"), "F"])
def test_mixed_batches_over_a_small_pool(mmodels, name, dtype):
    """Seven unequal requests, four live at a time, over a pool that holds just what is live and four state slots:
    pages and slots come back and go out again (freed pages are filled with NaN, windows give pages back while a
    request runs).  Then some of them alone: what a request gets must not depend on its neighbours beyond rounding."""
    m = mmodels[name]
    reqs = [(f"r{i}", m.prompt(n, salt=10 + i)) for i, n in enumerate((40, 3, 71, 18, 64, 1, 33))]
    steps = helpers.trace_mixed(reqs, seed=5, max_live=4)
    s = helpers.trace_session(m.folder, dtype, helpers.max_live_tokens(steps), poison_freed=True, state_slots=4)
    got = run(m, s, steps, reqs, dtype, "mixed")
    s.cache.manager.check()
    if dtype == "float32":
        alone = helpers.trace_session(m.folder, dtype, 128, state_slots=1)
        for rid, ids in reqs[:3]:
            one = helpers.replay(alone, helpers.trace_whole(rid, ids))[rid]
            scale = float(np.sqrt((one.astype(np.float64) ** 2).mean()))
            assert np.abs(one.astype(np.float64) - got[rid]).max() <= 3e-5 * scale


@pytest.mark.parametrize("name", ["D", quick("E"), "F"])
def test_a_blocks_last_kernel_does_what_is_next(mmodels, name):
    """With the layer debug hook every step of a block is a launch of its own; without it a block's last kernel also adds
    what joins the stream before the next block and makes its norm.  The logits are the same but for rounding."""
    m = mmodels[name]
    ids = m.prompt(50, salt=70)
    steps = helpers.trace_portions("r", ids, (30, 1, 1, 5, 1))
    one = helpers.replay(helpers.trace_session(m.folder, "float32", 128, state_slots=1), steps)["r"]
    two, _ = replay_routed(helpers.trace_session(m.folder, "float32", 128, state_slots=1), steps, m.cfg)
    assert np.abs(one - two["r"]).max() <= 2e-5 * np.abs(one).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts(mmodels, dtype):
    """Prompts of several hundred tokens at once and in long portions (the forms that kernels keep for long portions),
    beside a short one; then decoding goes on from what they left."""
    helpers.skip_in_simulation_if(True)
    m = mmodels["D"]
    ids, other = m.prompt(700, salt=40), m.prompt(9, salt=41)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ids[:300], "want": list(range(300))}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": other[:8], "want": list(range(8))},
                                     {"id": "a", "tokens": ids[300:690], "want": list(range(390))}], "end": []}]
    for i in range(690, 700):
        entries = [{"id": "a", "tokens": [ids[i]], "want": [0]}]
        if i == 690:
            entries.append({"id": "b", "tokens": [other[8]], "want": [0]})
        steps.append({"step": len(steps), "entries": entries, "end": ["b"] if i == 690 else []})
    steps[-1]["end"].append("a")
    s = helpers.trace_session(m.folder, dtype, 832, poison_freed=True, state_slots=2)
    run(m, s, steps, [("a", ids), ("b", other)], dtype, "long prompts")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(tmp_path, dtype):
    """Three hundred tokens one by one beside a neighbour that comes and goes, in a model whose layers use all of their
    experts (nothing hangs on a choice) and whose windows pass over decoded tokens."""
    helpers.skip_in_simulation_if(True)
    cfg = config(90, 40, 1e-5, 2.0,
                 [layer(rec(32, 2, 4), moe(2, 3, 24, identity=1, shared=8)), layer(att(2, 1, 16, 24, 0.25, 50), moe(3, 3, 16)),
                  layer(rec(24, 3, 3)), layer(att(4, 1, 16, 16, 0.3, 100), moe(1, 1, 24, shared=16))], loop=(0, 2, 2))
    m = make_model(tmp_path / "m", cfg, 31)
    ids, other = m.prompt(310, salt=20), m.prompt(60, salt=21)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ids[:10], "want": list(range(10))}], "end": []}]
    for i in range(10, len(ids)):
        entries = [{"id": "a", "tokens": [ids[i]], "want": [0]}]
        j = i - 50
        if 0 <= j < len(other):
            entries.append({"id": "b", "tokens": [other[j]], "want": [0]})
        steps.append({"step": len(steps), "entries": entries, "end": ["b"] if j == len(other) - 1 else []})
    steps[-1]["end"].append("a")
    s = helpers.trace_session(m.folder, dtype, 448, poison_freed=True, state_slots=2)
    got = helpers.replay(s, steps)
    check(m, got, {}, [("a", ids), ("b", other)], dtype, "long decode")


@pytest.mark.needs_device
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["D", "E"])
def test_greedy_generation_through_the_engine(mmodels, name, dtype):
    """The engine's own entry point and scheduler: several prompts at once over a pool that forces portions, with
    recorded decode steps and steps launched ahead.  Every generated token must be (nearly) the best under the plain
    model given the tokens before it; in bfloat16 an expert chosen the other way round may cost a few."""
    from deliverance_amd import AutoModelForCausalLM, GeneratorParameters
    m = mmodels[name]
    prompts = [m.prompt(n, salt=30 + n) for n in (5, 33, 70, 2)]
    model = AutoModelForCausalLM.from_pretrained(m.folder, dtype=dtype, max_cached_tokens=512, max_num_seqs=3,
                                                 max_batch_tokens=48, max_chunk=32)
    outs = model.generate(prompts, GeneratorParameters(max_tokens=24, ignore_eos=True))
    worse = 0
    for prompt, out in zip(prompts, outs):
        assert out.finish_reason == "length" and len(out.generated_tokens) == 24
        ids = list(prompt) + list(out.generated_tokens)
        ref = m.plain_logits(ids)
        for k, t in enumerate(out.generated_tokens):
            row = ref[len(prompt) + k - 1]
            slack = 1e-3 if dtype == "float32" else 2 * 6e-2 * float(np.sqrt((row ** 2).mean()))
            worse += row[t] < row.max() - slack
    assert worse <= (0 if dtype == "float32" else 8)


@pytest.mark.needs_device
def test_recorded_decode_steps_give_the_eager_ones_logits(mmodels):
    """Decode steps replayed from recorded graphs, several in a row with a prompt's portion between them, against the
    same steps kernel by kernel: the same logits, every time."""
    m = mmodels["D"]
    ids, other = m.prompt(80, salt=60), m.prompt(20, salt=61)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": ids[:30], "want": [29]}], "end": []}]
    for i in range(30, 80):
        if i == 55:
            steps.append({"step": len(steps), "entries": [{"id": "b", "tokens": other, "want": [19]}], "end": ["b"]})
        steps.append({"step": len(steps), "entries": [{"id": "a", "tokens": [ids[i]], "want": [0]}], "end": []})
    steps[-1]["end"] = ["a"]
    eager = helpers.replay(helpers.trace_session(m.folder, "bfloat16", 192, state_slots=2), steps)
    replayed = helpers.replay(helpers.trace_session(m.folder, "bfloat16", 192, state_slots=2, use_graphs=True), steps)
    for rid in eager:
        rms = float(np.sqrt((eager[rid].astype(np.float64) ** 2).mean()))
        assert np.abs(eager[rid] - replayed[rid]).max() <= 2e-2 * rms


# ------------------------------------------------------------------------------------------ random configurations
def random_config(seed):
    """Sizes drawn at random, among them what the kernels take only on their plain paths, one expert, as many experts a
    token as can be chosen, windows of one key and longer than the prompt, loops anywhere."""
    rng = np.random.default_rng(seed)
    pick = lambda *a: a[int(rng.integers(0, len(a)))]
    width = pick(40, 50, 64, 100, 72, 36)
    layers = []
    for _ in range(int(rng.integers(1, 5))):
        n, ident, groups = pick(1, 2, 5, 9), pick(0, 0, 1, 3), None
        can = n + ident
        divisors = [d for d in range(1, can + 1) if can % d == 0]
        if rng.random() < 0.6:
            count = pick(*divisors)
            groups = (count, int(rng.integers(1, count + 1)))
            can = can // count * groups[1]
        mlp = moe(n, pick(1, can, max(1, can // 2)), pick(8, 20, 32), ident, groups, pick(None, 8, 32, 40)) if rng.random() < 0.75 else None
        if rng.random() < 0.5:
            blocks = pick(1, 2, 3, 5)
            layers.append(layer(rec(blocks * pick(4, 8, 16, 20, 24, 40, 72), blocks, pick(1, 2, 3, 4, 5, 9)), mlp))
        else:
            g = pick(1, 2, 3)
            layers.append(layer(att(g * pick(1, 2, 3), g, pick(8, 16, 20, 32, 64), pick(8, 12, 16, 32, 40, 64), float(pick(0.1, 0.25, 0.4)),
                                    pick(1, 7, 16, 40, 1000, None)), mlp))
    loop = None
    if rng.random() < 0.6:
        a = int(rng.integers(0, len(layers)))
        loop = (a, int(rng.integers(a + 1, len(layers) + 1)), pick(1, 2, 3))
    return config(pick(50, 130, 257), width, float(pick(1e-6, 1e-5, 1e-3)), float(pick(0.5, 1.0, 4.0, 12.0)), layers, loop)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(16))
def test_random_configurations(tmp_path, seed, dtype):
    m = make_model(tmp_path / "m", random_config(seed), 100 + seed)
    ids = m.prompt(45, salt=seed)
    s = helpers.trace_session(m.folder, dtype, 128, poison_freed=True, state_slots=2)
    run(m, s, helpers.trace_whole("w", ids), [("w", ids)], dtype, f"seed {seed} whole")
    run(m, s, helpers.trace_portions("p", ids, (5, 2, 17, 1, 1, 9)), [("p", ids)], dtype, f"seed {seed} portions")
