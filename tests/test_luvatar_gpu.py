"""Luvatar on the engine against the plain implementation (tests/plain_luvatar.py): each mechanism alone through its
kernels and parts, then whole models through the step function (whole prompts, decoding token by token, portions down
to two tokens, mixed batches over a small pool whose pages and state slots come back and go out again), and greedy
generation through the engine's entry point and scheduler.  Sizes differ from test to test; where random numbers would
hide a fault (one far key among hundreds, a chunk's edge, the term without a key in a softmax, a state that must last)
the inputs are made so that it shows."""
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import helpers
import plain_luvatar as P
from helpers import quick
from luvatar_models import CONFIG_A, CONFIG_B, CONFIG_C, att, config, gla, layer, make_model, rot

pytestmark = pytest.mark.gpu
DEV = helpers.DEVICE
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
TOL = {"float32": 2e-5, "bfloat16": 3e-2}


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
def turn_spec(m):
    from deliverance_amd.config.specs import LinearSpeedsSpec, RotarySpec
    r = m["rot"]
    if r is None:
        return None
    return RotarySpec("rotary", r["dims"], r["base"], True, LinearSpeedsSpec(r["scaling"]["factor"]) if r.get("scaling") else None)


def attention_part(m, width, eps, W, dtype, shared):
    from deliverance_amd.config.specs import AttentionSpec, QKNormSpec
    from deliverance_amd.parts import build_mixer
    spec = AttentionSpec("attention", width, m["heads"], m["kv_heads"], m["dim"], m["scale"], qkv_bias=False, out_bias=False,
                         position=turn_spec(m), v_head_dim=m["vdim"], chunk=(m["mask"] or {}).get("size"),
                         qk_norm=QKNormSpec(eps, whole=False), sink="learned", out_gate="sigmoid", shared_kv=shared)
    t = lambda k: tb(W["mix." + k])
    params = {"qkv_weight": torch.cat([t(k) for k in (("q", "g") if shared else ("q", "k", "v", "g"))]), "out_weight": t("o"),
              "sink": t("sink"), "q_norm": t("q.norm")}
    if not shared:
        params["k_norm"] = t("k.norm")
    return build_mixer(spec, params, DTYPES[dtype], DEV)


def attention_weights(rng, m, width):
    H, G, D, Dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    nrm = lambda *shape, s=0.2: rng.normal(size=shape) * s
    return {"mix.q": nrm(H * D, width), "mix.k": nrm(G * D, width), "mix.v": nrm(G * Dv, width), "mix.g": nrm(H * Dv, width, s=0.5),
            "mix.o": nrm(width, H * Dv), "mix.sink": nrm(H, s=1.0), "mix.q.norm": 1 + nrm(D), "mix.k.norm": 1 + nrm(D)}


class MixerBench:
    """One mixer part with weights of its own, fed with rows h of whole sequences in steps of any cut; its additions
    to the stream are compared with the plain mixer over the whole sequences.  Pages are handed out in a shuffled
    order and start as NaN; state slots are given in any order.  ``reader``: a second attention part on the first one's
    keys and values, with queries and chunks of its own, which runs behind it and is compared instead."""

    def __init__(self, dtype, kind, m, width, seqs, page=16, seed=0, make=None, slots=None, reader=None, eps=1e-5):
        from deliverance_amd.config.specs import GatedLinearSpec
        from deliverance_amd.parts import KVNeed, build_mixer
        rng = np.random.default_rng(seed)
        nrm = lambda *shape, s=0.2: rng.normal(size=shape) * s
        if kind == "attention":
            W = attention_weights(rng, m, width)
            plain = lambda h: P.attention(self.W, "", m, h, eps, P.keys_and_values(self.W, "", m, h, eps))
        else:
            H, D, Dv, R = m["heads"], m["dim"], m["vdim"], m["a_rank"]
            W = {"mix.q": nrm(H * D, width), "mix.k": nrm(H * D, width), "mix.v": nrm(H * Dv, width), "mix.g": nrm(H * Dv, width, s=0.5),
                 "mix.o": nrm(width, H * Dv), "mix.norm": 1 + nrm(Dv), "mix.a1": nrm(R, width), "mix.a2": nrm(H * D, R, s=0.5),
                 "mix.a2.b": nrm(H * D, s=1.0)}
            plain = lambda h: P.gated_linear(self.W, "", m, h, eps)
        if make is not None:
            make(W)
        self.W = {k: bf16(v) for k, v in W.items()}
        self.width, self.dtype, self.page = width, dtype, page
        self.seqs = [bf16(s) for s in seqs]                       # h of every sequence, [T, width]
        self.reader = None
        if kind == "attention":
            self.part = attention_part(m, width, eps, self.W, dtype, False)
            if reader is not None:
                W2 = attention_weights(rng, reader, width)
                self.W2 = {k: bf16(v) for k, v in W2.items() if k not in ("mix.k", "mix.v", "mix.k.norm")}
                self.reader = attention_part(reader, width, eps, self.W2, dtype, True)
                plain = lambda h: P.attention(self.W2, "", reader, h, eps, P.keys_and_values(self.W, "", m, h, eps))
        else:
            t = lambda k: tb(self.W["mix." + k])
            self.part = build_mixer(GatedLinearSpec("gated_linear", width, m["heads"], m["dim"], m["vdim"], m["tau"], eps),
                                    {"q_weight": t("q"), "k_weight": t("k"), "v_weight": t("v"), "gate_weight": t("g"), "decay_down": t("a1"),
                                     "decay_up": t("a2"), "decay_bias": t("a2.b"), "out_norm": t("norm"), "out_weight": t("o")}, DTYPES[dtype], DEV)
        self.want = [plain(s) for s in self.seqs]
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
        hd = dev(h, DTYPES[self.dtype])
        self.part.forward(ctx, hd, x, SimpleNamespace(layer=0, cache=0, write=True))
        if self.reader is not None:
            x.zero_()
            self.reader.forward(ctx, hd, x, SimpleNamespace(layer=1, cache=0, write=False))
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


MIX = lambda d: d["mixer"]
ATTENTIONS = [quick(MIX(att(4, 2, 16, 8, 0.25, 24, rot(10000.0, 8, 3.0)))),      # matrix cores; chunks end inside pages
              MIX(att(3, 1, 12, 20, 0.3, 500, rot(500.0, 6))),                   # a head size left to the plain kernel
              MIX(att(2, 2, 64, 128, 0.125, 17, rot(1e6, 64, 8.0))),             # every entry turns; values twice the keys
              quick(MIX(att(6, 3, 32, 32, 0.2, 1, rot(10000.0, 0)))),            # a token sees itself only; nothing turns
              MIX(att(5, 1, 128, 64, 0.1, 32, rot(10000.0, 96, 0.5))),           # chunks of two pages; a factor below one
              MIX(att(1, 1, 40, 72, 0.2, None, None)),                           # every earlier key, no position encoding
              MIX(att(2, 1, 200, 24, 0.08, 33, rot(100.0, 200, 2.0)))]           # more entries than the matrix cores take
GLAS = [quick(MIX(gla(2, 16, 24, 4.0, 8))),
        MIX(gla(3, 18, 12, 0.5, 5)),                 # key rows and ranks that only the walking form takes; fast decays
        quick(MIX(gla(1, 64, 40, 16.0, 40))),        # a rank that goes through a product of its own
        MIX(gla(2, 100, 128, 1.0, 16)),              # two pieces a lane, the widest values
        MIX(gla(2, 136, 8, 2.0, 4)),                 # nine rows a lane
        quick(MIX(gla(5, 4, 4, 8.0, 12))),           # one lane's worth
        MIX(gla(1, 32, 72, 0.02, 32))]               # decays that leave nothing of the state


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("m", ATTENTIONS)
def test_attention_part_prompt_portions_and_decoding(m, dtype):
    rng = np.random.default_rng(5)
    helpers.skip_in_simulation_if(m["dim"] > 100 and dtype == "float32")
    walk(MixerBench(dtype, "attention", m, 64, [rng.normal(size=(n, 64)) for n in (70, 33, 1)]), TOL[dtype])


READERS = [quick(MIX(att(4, 2, 16, 8, 0.25, 24, rot(10000.0, 8, 3.0))), MIX(att(2, 2, 16, 8, 0.4, 50, rot(10000.0, 8, 3.0)))),
           (MIX(att(2, 1, 12, 20, 0.3, 64, rot(500.0, 12))), MIX(att(3, 1, 12, 20, 0.5, 7, rot(500.0, 12)))),
           (MIX(att(2, 2, 64, 64, 0.125, 17, rot(1e6, 32))), MIX(att(6, 2, 64, 64, 0.1, None, rot(1e6, 32)))),
           (MIX(att(1, 1, 32, 16, 0.2, None, None)), MIX(att(5, 1, 32, 16, 0.2, 32, None)))]


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("m,reader", READERS)
def test_attention_on_another_layers_keys_and_values(m, reader, dtype):
    """The second part has queries, a sink, a gate, a scale and chunks of its own, longer or shorter than the first's."""
    rng = np.random.default_rng(6)
    walk(MixerBench(dtype, "attention", m, 64, [rng.normal(size=(n, 64)) for n in (70, 33, 1)], reader=reader), TOL[dtype])


def test_a_part_without_keys_of_its_own_does_not_write():
    rng = np.random.default_rng(6)
    m = MIX(att(2, 1, 16, 16, 0.25, 24, rot(10000.0, 8)))
    b = MixerBench("float32", "attention", m, 32, [rng.normal(size=(5, 32))], reader=m)
    read = b.reader.forward
    b.reader.forward = lambda ctx, h, x, call: read(ctx, h, x, SimpleNamespace(layer=1, cache=0, write=True))
    with pytest.raises(ValueError, match="cannot write"):
        b.step({0: 5})


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("m", GLAS)
def test_gated_linear_part_prompt_portions_and_decoding(m, dtype):
    """The state rows are handed out in any order.  (A tolerance of the result's largest value: where a head's state
    holds little more than one token, its read-out norm divides by |q . k|.)"""
    rng = np.random.default_rng(7)
    helpers.skip_in_simulation_if(m["dim"] > 90 and dtype == "float32")
    sure = make_sure_of_the_readout(m)
    b = MixerBench(dtype, "gated_linear", m, 48, [rng.normal(size=(n, 48)) for n in (70, 33, 1)], slots=[3, 0, 2], make=sure)
    walk(b, TOL[dtype])


def make_sure_of_the_readout(m):
    """Keys near the queries, so that a token's own q . k never lies near zero: the read-out of a head that forgets at
    once, or of a first token, is q . k times one value, whose sign rounding would decide."""
    def make(W):
        W["mix.k"] = W["mix.q"] + 0.2 * W["mix.k"]
    return make


def marked(W):
    """Input channel 0 makes a key, channel 1 a query of the same direction: of all pairs the one marked pair of tokens
    has by far the largest score (norms make all keys and queries of one length, so it is the direction that counts)."""
    for k in ("mix.q", "mix.k"):
        W[k] *= 0.3
        W[k + ".norm"][:] = 1.0
    W["mix.k"][:, 0] = np.tile([1.0, -1.0], W["mix.k"].shape[0] // 2)
    W["mix.q"][:, 1] = np.tile([1.0, -1.0], W["mix.q"].shape[0] // 2)
    W["mix.sink"][:] = -2.0


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("chunk,last", [quick(56, 167), (56, 168), (24, 239), quick(24, 240), (16, 47), (16, 48), (33, 65), (33, 66),
                                        (300, 260), (90, 179), (90, 178), (7, 200), (128, 255), (100, 201)])
@pytest.mark.parametrize("shared", [False, True])
def test_a_key_at_a_chunks_edge(chunk, last, shared, dtype):
    """The last query, at position ``last``, matches one key far better than any other: the first key of its own chunk,
    then the last key of the chunk before, which it must not see.  A chunk counted from elsewhere, an edge that is one
    token off, or a key read from a page that was given back, shows as an error of the order of the output; in a prompt,
    in a portion that starts inside the chunk, and in decoding."""
    width, T = 32, last + 1
    first = last // chunk * chunk
    m = MIX(att(2, 1, 16, 16, 1.0, chunk, rot(10000.0, 0)))
    other = MIX(att(2, 1, 16, 16, 1.0, 1000 if chunk < 100 else 13, rot(10000.0, 0)))
    marks = [first] + ([first - 1] if first else [])
    for mark in marks:
        if mark == last:
            continue
        rng = np.random.default_rng(chunk + last)
        h = rng.normal(size=(T, width)) * 0.1
        h[mark, 0] = 6.0
        h[last, 1] = 6.0
        cuts = [[T], [T - 1, 1]] + ([[first + 3, T - first - 3]] if T - first - 3 > 1 else []) + [[max(first - 2, 1), T - max(first - 2, 1)]]
        for cut in cuts if not helpers.SIMT else cuts[:2]:
            b = MixerBench(dtype, "attention", other if shared else m, width, [h], seed=1, make=marked, reader=m if shared else None)
            if shared:
                b.W2.update({k: b.W[k] for k in ("mix.q", "mix.q.norm", "mix.sink")})
                b.reader = attention_part(m, width, 1e-5, b.W2, dtype, True)
                b.want = [P.attention(b.W2, "", m, s, 1e-5, P.keys_and_values(b.W, "", m, s, 1e-5)) for s in b.seqs]
            for n in cut:
                err = b.step({0: n})
                assert err <= TOL[dtype], f"mark {mark}, cut {cut}: {err}"
        # the test sees what it is meant to see: with an edge one token off the result at the last position is another
        W = b.W2 if shared else b.W
        kv = P.keys_and_values(b.W, "", m, b.seqs[0], 1e-5)
        keep = P.chunk_mask

        def off(T_, size):
            mask = keep(T_, size)
            mask[last, mark] = not mask[last, mark]
            return mask
        P.chunk_mask = off
        try:
            wrong = P.attention(W, "", m, b.seqs[0], 1e-5, kv)[-1]
        finally:
            P.chunk_mask = keep
        right = b.want[0][-1]
        assert np.abs(wrong - right).max() > 0.2 * max(np.abs(wrong).max(), np.abs(right).max())


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
def test_the_term_without_a_key_takes_its_share(dtype):
    """A sink above all scores in one head and below in the other; left out, scaled, or counted once a share of the
    keys, the result would be another."""
    T, width = 70, 32
    rng = np.random.default_rng(3)
    h = rng.normal(size=(T, width))
    m = MIX(att(2, 1, 16, 16, 0.5, 64, rot(10000.0, 16)))

    def make(W):
        W["mix.sink"][:] = [3.0, 4.0]
    b = MixerBench(dtype, "attention", m, width, [h], seed=2, make=make)
    kv = P.keys_and_values(b.W, "", m, b.seqs[0], 1e-5)
    for change in (lambda s: np.full_like(s, -1e9), lambda s: s * m["scale"], lambda s: s + np.log(2.0)):
        other = dict(b.W)
        other["mix.sink"] = change(b.W["mix.sink"])
        assert np.abs(P.attention(other, "", m, b.seqs[0], 1e-5, kv) - b.want[0]).max() > 0.1 * np.abs(b.want[0]).max()
    assert b.step({0: T - 4}) <= TOL[dtype]
    assert b.step({0: 2}) <= TOL[dtype]
    for _ in range(2):
        assert b.step({0: 1}) <= TOL[dtype]


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
def test_the_norm_of_queries_and_keys_comes_before_the_turn_with_gains_by_entry(dtype):
    """Gains that differ from entry to entry, inputs of very different lengths: a norm behind the turn, one over all
    heads, or a gain off by an entry would show; so would a rotation of the wrong pairs or a factor left out."""
    rng = np.random.default_rng(4)
    h = rng.normal(size=(40, 32)) * np.exp(rng.normal(size=(40, 1)))
    m = MIX(att(4, 2, 24, 8, 1.5, 40, rot(3.0, 12, 5.0)))

    def make(W):
        W["mix.q.norm"][:] = np.linspace(0.2, 2.0, 24)
        W["mix.k.norm"][:] = np.linspace(1.5, -1.0, 24)
    b = MixerBench(dtype, "attention", m, 32, [h], seed=5, make=make)
    for other in (rot(3.0, 12), rot(3.0, 10, 5.0)):
        mm = dict(m, rot=other)
        wrong = P.attention(b.W, "", mm, b.seqs[0], 1e-5, P.keys_and_values(b.W, "", mm, b.seqs[0], 1e-5))
        assert np.abs(wrong - b.want[0]).max() > 0.1 * np.abs(b.want[0]).max()
    assert b.step({0: 30}) <= TOL[dtype]
    for _ in range(3):
        assert b.step({0: 1}) <= TOL[dtype]


# ------------------------------------------------------------------------------------------ the recurrence
@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
def test_gated_linear_attention_remembers_the_first_token(dtype):
    """A head whose decays are nearly 1 keeps the first token's key and value: after 300 tokens, cut into portions and
    decoded tokens, a query that matches that key alone reads that value; the head beside it has forgotten it."""
    T, width = 300, 32
    rng = np.random.default_rng(8)
    h = rng.normal(size=(T, width)) * 0.02
    h[0, 0] = 8.0
    h[T - 1, 1] = 8.0
    m = MIX(gla(2, 16, 16, 2.0, 4))

    def make(W):
        W["mix.q"] *= 0.1
        W["mix.k"] *= 0.1
        W["mix.k"][:, 0] = 1.0
        W["mix.q"][:, 1] = 1.0
        W["mix.a2"] *= 0.1
        W["mix.a2.b"][:16] = 12.0
        W["mix.a2.b"][16:] = -1.0
    b = MixerBench(dtype, "gated_linear", m, width, [h], seed=3, make=make, slots=[1])
    lost = dict(b.W)
    lost["mix.a2.b"] = np.where(b.W["mix.a2.b"] > 0, 4.0, b.W["mix.a2.b"])        # a little forgetting already shows
    assert np.abs(P.gated_linear(lost, "", m, b.seqs[0], 1e-5)[-1] - b.want[0][-1]).max() > 0.05 * np.abs(b.want[0][-1]).max()
    for n in (150, 2, 100, 1, 1, 44, 1):
        b.step({0: n})           # (rows between the two are noise over noise behind the read-out's norm: not compared)
    assert b.step({0: 1}) <= TOL[dtype]
    assert b.done == [T]


def recurrence(q, k, v, a, S0):
    """Token by token, float64: o [T, Dv], S [D, Dv]."""
    S, o = S0.copy(), []
    for t in range(len(q)):
        S = a[t][:, None] * S + np.outer(k[t], v[t])
        o.append(S.T @ q[t])
    return np.array(o), S


@pytest.mark.parametrize("H,D,Dv,tau,lift", [quick(2, 44, 28, 12.0, 0.0), (3, 16, 20, 1.0, 0.0), (1, 64, 64, 0.5, -4.0), quick(2, 20, 40, 0.05, -2.0),
                                             (2, 128, 128, 8.0, 1.0), (1, 68, 72, 0.3, -6.0), (2, 32, 128, 1.0, -30.0), (1, 4, 4, 2.0, 6.0)])
@pytest.mark.parametrize("low", [True, False])
def test_the_forms_for_serving_against_the_recurrence(H, D, Dv, tau, lift, low):
    """Portions of many lengths (inside a block of 16, at its edge, at a chunk's edge and past it) and one-token
    sequences, from given states, with decays from gentle to ones that leave nothing within a block (where the blocks'
    scores are summed pair by pair), the decays' arguments as rows or through a low rank.  The states that are kept and
    the gated, normalised read-outs against the recurrence written out; states that nobody has, and states that are not
    to be written, stay as they are."""
    from deliverance_amd.kernels import ops
    rng = np.random.default_rng(D + Dv)
    lens = [1, 1, 1, 2, 15, 16, 17, 64, 65, 150] if not helpers.SIMT else [1, 1, 2, 17, 70]
    S, N, R, nd = len(lens), sum(lens), 8, sum(1 for n in lens if n == 1)
    cols = 2 * H * D + 2 * H * Dv + R
    x = bf16(rng.normal(size=(N, cols + 3)) * 0.7)
    q, k = x[:, 1:1 + H * D], x[:, 1 + H * D:1 + 2 * H * D]
    v, gate, low_x = x[:, 1 + 2 * H * D:][:, :H * Dv], x[:, 1 + 2 * H * D + H * Dv:][:, :H * Dv], x[:, 1 + 2 * H * D + 2 * H * Dv:][:, :R]
    up = bf16(rng.normal(size=(H * D, R)))
    bias = (rng.normal(size=H * D) + lift).astype(np.float32).astype(np.float64)
    z = low_x @ up.T
    z_in = z.astype(np.float32).astype(np.float64)
    a = np.exp(P.log_logistic((z if low else z_in) + bias) / tau)
    gain = bf16(1 + 0.3 * rng.normal(size=Dv))
    slots = list(rng.permutation(S + 1)[:S])
    slots[1] = -1
    if S > 5:
        slots[5] = -1
    state0 = rng.normal(size=(S + 1, H * Dv * D)).astype(np.float32)
    q_start = np.concatenate([[0], np.cumsum(lens)])
    from deliverance_amd.parts import Arena
    arena = Arena(DEV)
    ctx = SimpleNamespace(q_start=dev(q_start), state_slots=dev(slots), n_seqs=S, n_decode=nd, max_query_len=max(lens), buf=arena.get)
    want, kept = np.zeros((N, H * Dv)), state0.astype(np.float64)
    for i in range(S):
        r = slice(q_start[i], q_start[i + 1])
        for h in range(H):
            S0 = np.zeros((D, Dv)) if slots[i] < 0 else state0[slots[i], h * Dv * D:(h + 1) * Dv * D].reshape(Dv, D).T.astype(np.float64)
            o, S1 = recurrence(q[r, h * D:(h + 1) * D] * D ** -0.5, k[r, h * D:(h + 1) * D], v[r, h * Dv:(h + 1) * Dv], a[r, h * D:(h + 1) * D], S0)
            g = gate[r, h * Dv:(h + 1) * Dv]
            want[r, h * Dv:(h + 1) * Dv] = P.rms_scaled(o, gain, 1e-2) * P.swish(g)
            if slots[i] >= 0:
                kept[slots[i], h * Dv * D:(h + 1) * Dv * D] = S1.T.reshape(-1)
    proj = dev(np.concatenate([x, np.full((N, 1), np.nan)], 1), torch.bfloat16)
    raw = None if low else dev(z_in, torch.float32)
    for write in (True, False):
        st = dev(state0, torch.float32)
        assert ops.gla_serve_takes(proj, st, D, Dv) and ops.gla_low_takes(R, dev(up, torch.bfloat16))
        y = torch.full((N, H * Dv + 1), 7.0, dtype=torch.bfloat16, device=DEV)
        ops.gla_serve(ctx, proj, 1, 1 + H * D, 1 + 2 * H * D, 1 + 2 * H * D + H * Dv, 1 + 2 * H * D + 2 * H * Dv,
                      dev(up, torch.bfloat16) if low else None, raw, dev(bias, torch.float32), tau, D ** -0.5, dev(gain, torch.bfloat16),
                      1e-2, st, y[:, :H * Dv], H, D, Dv, write=write)
        err = np.abs(host(y)[:, :H * Dv] - want)
        assert err.max() <= 2.0 ** -7 * np.abs(want).max(), f"read-outs: {err.max()} at row {int(err.max(1).argmax())}"
        assert float((y[:, H * Dv:] - 7.0).abs().max()) == 0.0
        ref = kept if write else state0.astype(np.float64)
        assert np.abs(host(st) - ref).max() <= 1e-5 * np.abs(ref).max(), f"states, write={write}"
        # the walking form from the same inputs
        o = torch.zeros(N, H * Dv, dtype=torch.float32, device=DEV)
        st2 = dev(state0, torch.float32)
        ops.gla_walk(ctx, proj, 1, 1 + H * D, 1 + 2 * H * D, dev(z_in, torch.float32), dev(bias, torch.float32), tau, D ** -0.5, st2, o, H, D, Dv, write=write)
        assert np.abs(host(st2) - ref).max() <= 1e-5 * np.abs(ref).max()
        y2 = P.rms_scaled(host(o).reshape(N, H, Dv), gain, 1e-2).reshape(N, H * Dv) * P.swish(gate)
        assert np.abs(y2 - want).max() <= 1e-4 * np.abs(want).max()


def test_a_block_with_gentle_and_thin_rows_side_by_side():
    """One row of the state forgets within a token while the others last: the block's scores are summed pair by pair,
    and a pair of neighbours deep inside a block still meets in the fast row."""
    from deliverance_amd.kernels import ops
    from deliverance_amd.parts import Arena
    H, D, Dv, N = 1, 16, 16, 40
    rng = np.random.default_rng(1)
    x = bf16(rng.normal(size=(N, 2 * D + 2 * Dv)))
    z = rng.normal(size=(N, D)).astype(np.float32)
    z[:, 3] = np.where(np.arange(N) % 5 == 0, -40.0, 3.0)             # nothing gets past every fifth token
    z[:, 7] = -12.0
    z[20:, 9] = -300.0
    bias = np.zeros(D, dtype=np.float32)
    a = np.exp(P.log_logistic(z.astype(np.float64)))
    q, k, v, g = x[:, :D], x[:, D:2 * D], x[:, 2 * D:2 * D + Dv], x[:, 2 * D + Dv:]
    o, S1 = recurrence(q * D ** -0.5, k, v, a, np.zeros((D, Dv)))
    want = P.rms_scaled(o, np.ones(Dv), 1e-2) * P.swish(g)
    ctx = SimpleNamespace(q_start=dev([0, N]), state_slots=dev([0]), n_seqs=1, n_decode=0, max_query_len=N, buf=Arena(DEV).get)
    st = torch.zeros(1, D * Dv, dtype=torch.float32, device=DEV)
    y = torch.zeros(N, Dv, dtype=torch.bfloat16, device=DEV)
    ops.gla_serve(ctx, dev(x, torch.bfloat16), 0, D, 2 * D, 2 * D + Dv, 0, None, dev(z, torch.float32), dev(bias, torch.float32), 1.0,
                  D ** -0.5, dev(np.ones(Dv), torch.float32), 1e-2, st, y, H, D, Dv)
    assert np.abs(host(y) - want).max() <= 2.0 ** -7 * np.abs(want).max()
    assert np.abs(host(st).reshape(Dv, D).T - S1).max() <= 1e-5 * np.abs(S1).max()


def test_kernels_refuse_what_they_cannot_take():
    from deliverance_amd.kernels import ops
    ctx = SimpleNamespace(q_start=dev([0, 2]), state_slots=dev([0]), n_seqs=1, n_decode=0, max_query_len=2, buf=lambda *a: None)
    p = torch.zeros(2, 64, dtype=torch.bfloat16, device=DEV)
    st = torch.zeros(1, 64, dtype=torch.float32, device=DEV)
    y = torch.zeros(2, 8, dtype=torch.bfloat16, device=DEV)
    bias, gain = torch.zeros(8, dtype=torch.float32, device=DEV), torch.ones(8, dtype=torch.float32, device=DEV)
    with pytest.raises(ops.KernelError, match="as rows or from a low rank"):
        ops.gla_serve(ctx, p, 0, 8, 16, 24, 32, None, None, bias, 1.0, 1.0, gain, 1e-5, st, y, 1, 8, 8)
    with pytest.raises(ops.KernelError, match="leave the row"):
        ops.gla_serve(ctx, p, 60, 8, 16, 24, 32, None, torch.zeros(2, 8, device=DEV), bias, 1.0, 1.0, gain, 1e-5, st, y, 1, 8, 8)
    with pytest.raises(ops.KernelError, match="state row"):
        ops.gla_walk(ctx, p, 0, 8, 16, torch.zeros(2, 16, device=DEV), torch.zeros(16, device=DEV), 1.0, 1.0, st,
                     torch.zeros(2, 16, device=DEV), 2, 8, 8)
    assert not ops.gla_serve_takes(p, st, 18, 8) and not ops.gla_serve_takes(p, st, 8, 132) and not ops.gla_low_takes(36, p)


# ------------------------------------------------------------------------------------------ whole models
@pytest.fixture(scope="module")
def lmodels(tmp_path_factory):
    return {"A": make_model(tmp_path_factory.mktemp("la"), CONFIG_A, 51), "B": make_model(tmp_path_factory.mktemp("lb"), CONFIG_B, 52),
            "C": make_model(tmp_path_factory.mktemp("lc"), CONFIG_C, 53)}


def check(model, got, requests, dtype, what=""):
    """32-bit: every logit within 1e-4 of the largest plain logit (a typical error is a tenth of that).  bfloat16: against
    what rounding alone does to a position's logits in the plain model.  The design's norms behind its parts and read-outs
    make that very uneven (a head whose state holds little more than one token reads out (q . k) times one value and
    divides by its length, so rounding decides the sign where the product is near zero): the error over all positions may
    be 2.5 times rounding's, and one position in ten may be off by more than 4 times the larger of rounding's error there
    and its median."""
    for rid, ids in requests:
        ref = model.plain_logits(ids)
        out = got[rid].astype(np.float64)
        assert out.shape == ref.shape, f"{what} {rid}: shape {out.shape} vs {ref.shape}"
        err = np.abs(out - ref)
        if dtype == "float32":
            worst = int(err.max(axis=1).argmax())
            assert err.max() <= 1e-4 * np.abs(ref).max(), f"{what} {rid}: {err.max():.3e} at position {worst}"
            continue
        base = np.maximum(model.rounding_error(ids), 2.0 ** -8 * float(np.sqrt((ref ** 2).mean())))
        here = np.sqrt((err ** 2).mean(axis=1))
        over = here > 4.0 * np.maximum(base, np.median(base))
        assert over.sum() <= max(1, len(ids) // 10), f"{what} {rid}: over at {np.nonzero(over)[0].tolist()}"
        if len(ids) > 10:
            assert np.sqrt((here ** 2).mean()) <= 2.5 * np.sqrt((base ** 2).mean()), f"{what} {rid}: rms error"


def run(model, session, steps, requests, dtype, what):
    got = helpers.replay(session, steps)
    check(model, got, requests, dtype, what)
    return got


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("name", [quick("A"), "B", "C"])
def test_whole_prompts_and_first_tokens(lmodels, name, dtype):
    m = lmodels[name]
    reqs = [("one", m.prompt(1)), ("two", m.prompt(2)), ("three", m.prompt(3)), ("long", m.prompt(90))]
    s = helpers.trace_session(m.folder, dtype, 256, state_slots=2)
    for rid, ids in reqs:
        run(m, s, helpers.trace_whole(rid, ids), [(rid, ids)], dtype, "whole")
    s.cache.manager.check()


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("name", ["A", quick("B"), "C"])
def test_prefill_against_token_by_token_decoding(lmodels, name, dtype):
    """All but the last 45 tokens at once, the rest one by one, across page borders, tiles of keys and the chunks'
    edges; then a request that is decoded from its very first token on."""
    m = lmodels[name]
    ids = m.prompt(75, salt=1)
    s = helpers.trace_session(m.folder, dtype, 128, state_slots=1)
    run(m, s, helpers.trace_bulk_then_single("r", ids, tail=45), [("r", ids)], dtype, "decode")
    ids2 = m.prompt(20, salt=2)
    run(m, s, helpers.trace_bulk_then_single("q", ids2, tail=19), [("q", ids2)], dtype, "decode from 1")


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("name", [quick("A"), "B", "C"])
@pytest.mark.parametrize("sizes", [(7, 2, 13, 3, 5, 2), quick((2, 2, 31, 1, 16, 33, 2))])
def test_portions_of_any_size(lmodels, name, dtype, sizes):
    m = lmodels[name]
    ids = m.prompt(97, salt=3)
    s = helpers.trace_session(m.folder, dtype, 128, poison_freed=True, state_slots=1)
    run(m, s, helpers.trace_portions("r", ids, sizes), [("r", ids)], dtype, f"portions {sizes}")


@pytest.mark.parametrize("dtype", ["float32", quick("bfloat16")])
@pytest.mark.parametrize("name", ["A", "B", quick("C")])
def test_mixed_batches_over_a_small_pool(lmodels, name, dtype):
    """Seven unequal requests, four live at a time, over a pool that holds just what is live and four state slots:
    pages and slots come back and go out again (freed pages are filled with NaN, chunks give pages back while a request
    runs).  Then some of them alone: what a request gets must not depend on its neighbours beyond rounding."""
    m = lmodels[name]
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
            assert np.abs(one.astype(np.float64) - got[rid]).max() <= 5e-5 * scale


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts(lmodels, dtype):
    """Prompts of several hundred tokens at once and in long portions, beside a short one; then decoding goes on from
    what they left."""
    helpers.skip_in_simulation_if(True)
    m = lmodels["A"]
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
    """Three hundred tokens one by one beside a neighbour that comes and goes, across the edges of chunks of two sizes
    that read the same keys, with decays from slow to fast."""
    helpers.skip_in_simulation_if(True)
    cfg = config(90, 40, 1e-5, 2.0,
                 [layer(gla(2, 8, 16, 16.0, 4), 24), layer(att(2, 1, 16, 24, 0.25, 50, rot(10000.0, 16, 2.0)), 32),
                  layer(gla(1, 24, 8, 1.0, 6)), layer(att(4, 1, 16, 24, 0.3, 130, rot(10000.0, 16, 2.0), kv_from=1))])
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
    run(m, s, steps, [("a", ids), ("b", other)], dtype, "long decode")


@pytest.mark.needs_device
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_through_the_engine(lmodels, name, dtype):
    """The engine's own entry point and scheduler: several prompts at once over a pool that forces portions, with
    recorded decode steps and steps launched ahead.  Every generated token must be (nearly) the best under the plain
    model given the tokens before it."""
    from deliverance_amd import AutoModelForCausalLM, GeneratorParameters
    m = lmodels[name]
    prompts = [m.prompt(n, salt=30 + n) for n in (5, 33, 70, 2)]
    model = AutoModelForCausalLM.from_pretrained(m.folder, dtype=dtype, max_cached_tokens=512, max_num_seqs=3,
                                                 max_batch_tokens=48, max_chunk=32)
    outs = model.generate(prompts, GeneratorParameters(max_tokens=24, ignore_eos=True))
    for prompt, out in zip(prompts, outs):
        assert out.finish_reason == "length" and len(out.generated_tokens) == 24
        ids = list(prompt) + list(out.generated_tokens)
        ref = m.plain_logits(ids)
        worse = 0
        for k, t in enumerate(out.generated_tokens):
            row = ref[len(prompt) + k - 1]
            slack = 1e-3 if dtype == "float32" else 2 * 0.12 * float(np.sqrt((row ** 2).mean()))
            worse += row[t] < row.max() - slack
        assert worse <= (0 if dtype == "float32" else 2)


@pytest.mark.needs_device
def test_recorded_decode_steps_give_the_eager_ones_logits(lmodels):
    """Decode steps replayed from recorded graphs, several in a row with a prompt's portion between them, against the
    same steps kernel by kernel: the same logits, every time."""
    m = lmodels["A"]
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
    """Sizes drawn at random, among them what the kernels take only on their plain paths (widths and ranks that are no
    multiple of 8, head sizes that the matrix-core attention does not take), chunks of one key and longer than the
    prompt, layers on other layers' keys."""
    rng = np.random.default_rng(seed)
    pick = lambda *a: a[int(rng.integers(0, len(a)))]
    width = pick(40, 50, 64, 100, 72, 36)
    layers, own = [], []
    for i in range(int(rng.integers(2, 6))):
        ff = pick(None, 16, 40, 100)
        if rng.random() < 0.45:
            layers.append(layer(gla(pick(1, 2, 5), pick(4, 16, 18, 24, 40, 64), pick(4, 16, 24, 40), float(pick(0.5, 1.0, 4.0, 16.0)), pick(2, 4, 8, 16, 33)), ff))
            continue
        scale, chunk = float(pick(0.1, 0.25, 0.4)), pick(1, 7, 16, 24, 40, 1000)
        if own and rng.random() < 0.5:
            j = pick(*own)
            s = layers[j]["mixer"]
            mixer = att(s["kv_heads"] * pick(1, 2, 3), s["kv_heads"], s["dim"], s["vdim"], scale, chunk, s["rot"], kv_from=j)
        else:
            g, d = pick(1, 2, 3), pick(8, 16, 20, 32, 64)
            mixer = att(g * pick(1, 2, 3), g, d, pick(8, 12, 16, 40, 64), scale, chunk,
                        rot(float(pick(100.0, 1e4, 1e6)), pick(0, 2, d // 2, d), pick(None, 1.0, 2.0, 8.0)))
            own.append(i)
        layers.append(layer(mixer, ff))
    return config(pick(50, 130, 257), width, float(pick(1e-6, 1e-5, 1e-3)), float(pick(0.5, 1.0, 4.0, 12.0)), layers)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", range(14))
def test_random_configurations(tmp_path, seed, dtype):
    m = make_model(tmp_path / "m", random_config(seed), 100 + seed)
    ids = m.prompt(45, salt=seed)
    s = helpers.trace_session(m.folder, dtype, 128, poison_freed=True, state_slots=2)
    run(m, s, helpers.trace_whole("w", ids), [("w", ids)], dtype, f"seed {seed} whole")
    run(m, s, helpers.trace_portions("p", ids, (5, 2, 17, 1, 1, 9)), [("p", ids)], dtype, f"seed {seed} portions")
