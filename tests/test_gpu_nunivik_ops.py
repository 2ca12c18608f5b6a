"""Each mechanism of the Nunivik decoder alone, on the GPU, against the oracle: gated SiLU, gated norm, softmax attention
over pages (window, soft cap, rotation, head norms, mixed values), the gated delta rule and the state-space form."""
import pytest
import torch

from electrock_infer_amd.layers import decoder_ops as ops
from electrock_infer_amd.layers.attention import CarriedValues, SoftmaxAttention
from electrock_infer_amd.layers.dense_mlp import DenseMLP
from electrock_infer_amd.layers.recurrent import GatedDeltaRule, StateSpaceMixer
from oracle import nunivik_oracle as N
from tests.gpu_util import DEV, announce
from tests.nunivik_util import attn, config, delta, mamba, random_weights
from tests.test_gpu_decoder_ops import BF16, BLOCK, F32, Feed, close, rand, to

pytestmark = pytest.mark.gpu
EPS = 1e-5
NAN = float("nan")


def load(mix, w):
    for name, (param, section) in mix.TENSORS.items():
        p = mix.get_parameter(param)
        p.weight_loader(p, w["mix." + name].to(DEV), section) if section else p.data.copy_(w["mix." + name])
    if hasattr(mix, "finish_loading"):
        mix.finish_loading()
    return mix


def weights(entry, W, seed=0):
    """Float32 weights of a one-layer model's mixer, as bf16 numbers."""
    return {k[3:]: t.float() for k, t in random_weights(config(W, 4, [(entry, None)]), seed).items() if k.startswith("l0.mix.")}


def attention(entry, W, dtype, w):
    m, rot = entry["mixer"], entry["mixer"].get("rot", {})
    return load(SoftmaxAttention(W, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], EPS, dtype, rot.get("dims", 0), rot.get("base", 1.0),
                                 rot.get("scaling", {}).get("factor", 1.0), m.get("softcap", 0.0), m.get("mask", {}).get("size", 0), m["v_mix"]).to(DEV), w)


def recurrent(entry, W, dtype, w):
    m = entry["mixer"]
    if entry["type"] == "delta":
        mix = GatedDeltaRule(W, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], EPS, dtype)
    else:
        mix = StateSpaceMixer(W, m["heads"], m["groups"], m["state"], m["vdim"], m["conv"], m["norm_groups"], EPS, dtype)
    return load(mix.to(DEV), w)


def oracle(entry, h, w, carried=None):
    w = {k: t.double() for k, t in w.items()}
    return N.MIXERS[entry["type"]](h.double(), w, "mix.", entry["mixer"], EPS, {} if carried is None else carried).float()


def pages(mix, feed, dtype):
    return torch.full((feed.num_blocks, BLOCK, mix.row_elems()), NAN, dtype=dtype, device=DEV)


def slots(mix, n):
    c = mix.new_cache(0, BLOCK, n, DEV)
    c.states.fill_(NAN)
    c.ring.fill_(NAN)
    return c


class Alone:
    """A mixer as Feed calls it; the values that are mixed in are a layer's of their own or none."""

    def __init__(self, mix):
        self.mix = mix

    def __call__(self, h, batch, cache):
        return self.mix(h, batch, cache, CarriedValues())


# ---- rows ----
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,W,ff", [(1, 64, 40), (5, 90, 77), (16, 128, 136), (33, 192, 24), (64, 256, 512), (90, 64, 100), (3, 2048, 2048)])
def test_gated_feed_forward(T, W, ff, dtype):
    """The fused decode-batch product (bf16, widths of 64) and the library's with the activation behind it."""
    announce(f"silu gate {T} {W} {ff} {dtype}")
    x = rand(T, W, seed=1).to(dtype)
    w = {"gate": rand(ff, W, seed=2, scale=2 * W ** -0.5), "up": rand(ff, W, seed=3, scale=W ** -0.5), "down": rand(W, ff, seed=4, scale=ff ** -0.5)}
    w = {k: t.to(dtype).float() for k, t in w.items()}
    mlp = DenseMLP(W, ff, dtype, "silu_gate").to(DEV)
    for n, (param, section) in mlp.TENSORS.items():
        p = mlp.get_parameter(param)
        p.weight_loader(p, w[n].to(DEV), section) if section else p.data.copy_(w[n])
    inner = N.silu(x.double() @ w["gate"].double().t()) * (x.double() @ w["up"].double().t())
    close(ops.linear_silu_gate(to(x, dtype), mlp.up), inner, dtype, bf16=1e-2)
    y = mlp(to(x, dtype))
    close(y.sum(0) if y.dim() == 3 else y, N.feed_forward(x.float(), w, "", {"kind": "dense"}), dtype)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,parts,size", [(1, 1, 5), (3, 3, 30), (17, 1, 384), (4, 8, 512), (5, 2, 4096), (2, 1, 9000)])
def test_gated_norm(T, parts, size, dtype):
    announce(f"gated norm {T} {parts} {size} {dtype}")
    y, z, w = rand(T, parts * size, seed=1).to(dtype), rand(T, parts * size + 24, seed=2).to(dtype), rand(parts * size, seed=3)
    y[:, :size] *= 30                                    # parts of unequal size: each by its own root mean square
    zg = to(z, dtype)
    got = ops.gated_norm_(to(y, dtype), zg.data_ptr() + 8 * zg.element_size(), zg.stride(0), to(w), parts, 1e-3)
    close(got, N.gated_group_norm(y.double(), z[:, 8:8 + parts * size].double(), w.double(), parts, 1e-3), dtype, bf16=1e-2)


# ---- softmax attention ----
ATTN = [attn(6, 2, 22, 19, size=7, cap=5.0, rot=10, base=500.0, factor=1.5), attn(4, 1, 128, 96, size=40, cap=60.0, rot=64, factor=4.0),
        attn(3, 3, 11, 13), attn(8, 2, 64, 64, size=64, cap=20.0, rot=64), attn(2, 1, 256, 128, size=100, rot=2), attn(5, 1, 72, 200, size=33, cap=1.0),
        attn(16, 1, 40, 24, size=1, cap=50.0, rot=40), attn(2, 2, 1, 1, size=9, scale=2.0), attn(17, 1, 96, 128, size=130, rot=96)]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("entry", ATTN, ids=lambda e: "-".join(str(e["mixer"][k]) for k in ("heads", "kv_heads", "dim", "vdim")))
def test_attention_prompts_steps_and_portions(entry, dtype):
    announce(f"attention {entry['mixer']} {dtype}")
    W = 56
    w = weights(entry, W)
    mix = attention(entry, W, dtype, w)
    hs = [rand(n, W, seed=50 + n).to(dtype).float() for n in (1, 2, BLOCK, BLOCK + 1, 31, 147)]
    want = [oracle(entry, h, w) for h in hs]
    for sizes in ([1000], [1], [2], [3, 1, 16], [64, 83], [70, 1], [BLOCK]):
        feed = Feed(hs)
        for got, ref in zip(feed.run(Alone(mix), pages(mix, feed, dtype), sizes, dtype), want):
            close(got, ref, dtype, bf16=3e-2)
    feed = Feed(hs)
    cache = pages(mix, feed, dtype)
    parts = [feed.step(Alone(mix), cache, [1, 1, 2, 8, 13, 72], dtype), feed.step(Alone(mix), cache, [0, 1, 6, 1, 18, 75], dtype)]
    for i, ref in enumerate(want):
        close(torch.cat([parts[0][i]] + ([parts[1][i - 1]] if i >= 1 else [])), ref, dtype, bf16=3e-2)


def planted(entry, n, key, seed=1, strength=1.0):
    """Hidden rows and weights for which the last query's score with one key stands out from all others: of a row, the first
    part makes queries, the second keys and the third values (no rotation)."""
    m = entry["mixer"]
    H, G, d, v = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    W = 2 * d + v
    w = {"mix.q": torch.cat([torch.eye(d, W)] * H), "mix.k": torch.cat([torch.eye(d, W).roll(d, 1)] * G),
         "mix.v": torch.cat([torch.eye(v, W).roll(2 * d, 1)] * G), "mix.q.norm": torch.full((d,), strength), "mix.k.norm": torch.ones(d),
         "mix.o": rand(W, H * v, seed=seed + 1, scale=(H * v) ** -0.5)}
    h = rand(n, W, seed=seed)
    h[n - 1, :d] = h[key, d:2 * d]
    return h, w, W


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("size", [1, 2, 31, 32, 33, 64, 65, 100, 127, 128, 129, 199])
@pytest.mark.parametrize("cap", [None, 30.0])
def test_attention_window_edges(size, cap, dtype):
    """The key just inside the window takes all the weight; the one just outside has none."""
    announce(f"attention window {size} cap {cap} {dtype}")
    n, entry = 200, attn(4, 2, 32, 24, size=size, cap=cap, scale=1.0)
    for key, inside in ((n - size, True), (n - size - 1, False)):
        if key < 0:
            continue
        h, w, W = planted(entry, n, key)
        h = h.to(dtype).float()
        mix = attention(entry, W, dtype, w)
        ref = oracle(entry, h, w)
        value = h[key, 64:] @ sum(w["mix.o"][:, i * 24:(i + 1) * 24] for i in range(4)).t()
        assert (float((ref[-1] - value).abs().max()) < 0.2) == inside                # it does stand out
        for sizes in ([1000], [n - 1, 1], [150, 1000], [3, 40, 2], [n - 2, 2]):
            feed = Feed([h])
            got = feed.run(Alone(mix), pages(mix, feed, dtype), sizes, dtype)[0]
            close(got, ref, dtype, bf16=6e-2)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("key", [0, 1, BLOCK - 1, BLOCK, 31, 32, 63, 64, 127, 128, 255, 256, 298])
def test_attention_finds_one_key_among_many(key, dtype):
    """Far keys and keys at the borders of pages and tiles, without a window: the result is that key's value alone."""
    announce(f"attention far key {key} {dtype}")
    n, entry = 300, attn(2, 1, 40, 16, scale=1.0)
    h, w, W = planted(entry, n, key)
    h = h.to(dtype).float()
    mix = attention(entry, W, dtype, w)
    ref = oracle(entry, h, w)
    for sizes in ([1000], [n - 1, 1], [90, 1000], [64, 64, 2, 70, 2]):
        feed = Feed([h])
        close(feed.run(Alone(mix), pages(mix, feed, dtype), sizes, dtype)[0][-1], ref[-1], dtype, bf16=6e-2)


@pytest.mark.parametrize("splits", [1, 2, 5, 64])
def test_attention_is_the_same_for_every_number_of_splits(splits, monkeypatch):
    announce(f"attention splits {splits}")
    for entry in (attn(6, 2, 24, 20, size=50, cap=7.0, rot=8), attn(2, 2, 40, 72)):
        w = weights(entry, 56)
        mix = attention(entry, 56, F32, w)
        monkeypatch.setattr(mix, "splits", lambda batch: splits)
        h = rand(150, 56, seed=9)
        feed = Feed([h])
        close(feed.run(Alone(mix), pages(mix, feed, F32), [100, 1, 2, 30], F32)[0], oracle(entry, h, w), F32)


@pytest.mark.parametrize("entry", ATTN, ids=lambda e: "-".join(str(e["mixer"][k]) for k in ("heads", "kv_heads", "dim", "vdim")))
def test_prompt_kernel_matches_the_paged_kernel(entry):
    """Both kernels of long portions on the same bf16 inputs, with a cached context in front and unequal sequences."""
    announce(f"attention, prompt against paged {entry['mixer']}")
    W, w = 64, weights(entry, 64)
    mix = attention(entry, W, BF16, w)
    hs = [rand(n, W, seed=n).to(BF16).float() for n in (300, 129, 65, 200)]
    for limit in (1, 10 ** 9):
        mix.PROMPT_TOKENS = limit
        feed = Feed(hs)
        cache = pages(mix, feed, BF16)
        first = feed.step(Alone(mix), cache, [100, 129, 1, 37], BF16)
        second = feed.step(Alone(mix), cache, [200, 0, 64, 163], BF16)
        outs = [torch.cat((first[0], second[0])), first[1], torch.cat((first[2], second[1])), torch.cat((first[3], second[2]))]
        for got, h in zip(outs, hs):
            close(got, oracle(entry, h, w), BF16, bf16=3e-2)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("lam", [0.0, 0.3, 1.0, -0.5])
def test_mixed_values(lam, dtype):
    """A first layer's values go into a second one's, also where the second has heads of other sizes; the first layer's own
    share is not used."""
    announce(f"value mixing {lam} {dtype}")
    W, first, second = 48, attn(4, 2, 16, 20, size=9, mix=True, rot=16), attn(2, 2, 24, 20, size=12, mix=True)
    w1, w2 = weights(first, W, 1), weights(second, W, 2)
    w1["mix.vmix"], w2["mix.vmix"] = torch.tensor(0.7), torch.tensor(lam)
    a, b = attention(first, W, dtype, w1), attention(second, W, dtype, w2)

    class Both:
        def __call__(self, h, batch, cache):
            carried = CarriedValues()
            y = a(h, batch, cache[0], carried).float()
            z = b(h * 2, batch, cache[1], carried).float()
            return torch.cat((y, z), -1)
    h, carried = rand(60, W, seed=3).to(dtype).float(), {}
    want = torch.cat((oracle(first, h, w1, carried), oracle(second, h * 2, w2, carried)), -1)
    for sizes in ([1000], [1], [2, 7], [50, 1]):
        feed = Feed([h])
        got = feed.run(Both(), (pages(a, feed, dtype), pages(b, feed, dtype)), sizes, dtype)[0]
        close(got, want, dtype, bf16=3e-2)


def test_rotation_at_far_positions():
    """Angles of positions in the tens of thousands, in 32 bits: the same two tokens far from the start."""
    announce("rotation at far positions")
    entry = attn(2, 1, 32, 16, size=6, rot=32, base=1e6, factor=2.0)
    W, w = 48, weights(entry, 48)
    mix, h = attention(entry, 48, F32, w), rand(20, 48, seed=3)
    w = {k: t.double() for k, t in w.items()}
    for at in (0, 4096, 50000):
        ref = N.attention(h.double(), w, "mix.", entry["mixer"], EPS, {}, first_position=at).float()[6:]   # windows that are full
        feed = Feed([torch.cat((rand(at, 48, seed=4) if at else h[:0], h))])
        feed.seqs[0].num_computed_tokens = at
        cache = torch.zeros(feed.num_blocks, BLOCK, mix.row_elems(), device=DEV)
        close(feed.step(Alone(mix), cache, [20], F32)[0][6:], ref, F32, f32=5e-3 if at > 5000 else 1e-3)


# ---- recurrences ----
RECURRENT = [delta(6, 3, 19, 27, 5), delta(2, 1, 64, 48, 3), delta(1, 1, 130, 144, 4), delta(3, 3, 16, 256, 1), delta(2, 2, 256, 5, 2), delta(2, 1, 1, 1, 16),
             delta(4, 2, 128, 128, 4), mamba(6, 2, 21, 10, 2, 3), mamba(4, 4, 48, 32, 4, 4), mamba(1, 1, 256, 256, 4), mamba(5, 1, 9, 7, 1), mamba(2, 1, 1, 4, 9),
             mamba(8, 1, 128, 64, 4, 2), mamba(3, 3, 33, 150, 3)]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("entry", RECURRENT, ids=lambda e: e["type"] + "-" + "-".join(str(v) for v in e["mixer"].values()))
def test_recurrence_prompts_steps_and_portions(entry, dtype):
    announce(f"{entry} {dtype}")
    W, w = 48, weights(entry, 48)
    mix = recurrent(entry, W, dtype, w)
    hs = [rand(n, W, seed=50 + n).to(dtype).float() for n in (1, 2, 15, 33, 97)]
    want = [oracle(entry, h, w) for h in hs]
    tol = dict(f32=1e-4, bf16=4e-2)
    for sizes in ([1000], [1], [2], [3, 1, 16], [17, 31], [32]):
        # every slot is full of NaN: a sequence starts from zero, not from what is there
        cache, feed = slots(mix, 7), Feed(hs, order=[4, 0, 6, 2, 1])
        for got, ref in zip(feed.run(mix, cache, sizes, dtype), want):
            close(got, ref, dtype, **tol)
        for t in cache:
            assert bool(t[5].isnan().all()) and bool(t[3].isnan().all())             # nobody else's slot was touched
    # one batch of all, in unequal portions
    cache, feed = slots(mix, 7), Feed(hs, order=[4, 0, 6, 2, 1])
    parts = [feed.step(mix, cache, [1, 2, 9, 20, 64], dtype), feed.step(mix, cache, [0, 0, 6, 13, 33], dtype)]
    for i, ref in enumerate(want):
        close(torch.cat([parts[0][i]] + ([parts[1][i - 2]] if i >= 2 else [])), ref, dtype, **tol)


@pytest.mark.parametrize("entry", [delta(2, 1, 64, 48, 3), delta(2, 2, 40, 32, 4), mamba(4, 2, 48, 32, 4), mamba(2, 1, 128, 64, 4)], ids=lambda e: e["type"])
@pytest.mark.parametrize("kept", ["everything", "nothing", "some"])
def test_recurrence_with_extreme_decays(entry, kept):
    """Heads that forget everything within a token beside heads that keep everything over several chunks."""
    announce(f"{entry['type']} decays: {kept}")
    W, w, H = 48, weights(entry, 48), entry["mixer"]["heads"]
    w["mix.A_log"] = {"everything": torch.full((H,), -12.0), "nothing": torch.full((H,), 5.0), "some": torch.linspace(-10.0, 6.0, H)}[kept]
    w["mix.dt_bias"] = torch.zeros(H)
    mix = recurrent(entry, W, F32, w)
    hs = [rand(n, W, seed=n) for n in (40, 300)]
    want = [oracle(entry, h, w) for h in hs]
    for sizes in ([1000], [1], [7]):
        for got, ref in zip(Feed(hs, chunk=64).run(mix, slots(mix, 2), sizes, F32), want):
            close(got, ref, F32, f32=2e-4)


@pytest.mark.parametrize("back", [1, 3, 4, 5, 15, 16, 17, 31, 32, 255, 256, 300])
@pytest.mark.parametrize("kind", ["delta", "mamba2"])
def test_recurrence_recalls_one_far_token(kind, back):
    """One token is written at full strength, all others hardly, and read `back` tokens later, across block and chunk
    borders."""
    announce(f"{kind} recall {back}")
    W, n = 40, 320
    entry = delta(2, 1, 24, 16, 3) if kind == "delta" else mamba(2, 1, 24, 16, 3)
    w = weights(entry, W)
    w["mix.A_log"], w["mix.dt_bias"] = torch.full((2,), -14.0), torch.zeros(2)
    h = rand(n, W, seed=3)
    # column 0 alone opens the write: beta of the delta rule, dt of the state-space form
    opening = torch.zeros(2, W)
    opening[:, 0] = 1.0
    if kind == "delta":
        w["mix.b"] = opening
    else:
        w["mix.in"] = torch.cat((w["mix.in"][:-2], opening))
    h[:, 0] = -12.0
    h[n - 1 - back, 0] = 6.0
    mix, ref = recurrent(entry, W, F32, w), oracle(entry, h, w)
    without = h.clone()
    without[n - 1 - back, 0] = -12.0
    # the read-outs behind it hang on that token
    assert float((oracle(entry, without, w)[-1] - ref[-1]).abs().max()) > 0.1 * float(ref.abs().max())
    for sizes in ([1000], [n - back, 1000], [n - 1, 1], [n - 1 - back, 1, 2]):
        got = Feed([h], chunk=256).run(mix, slots(mix, 1), sizes, F32)[0]
        close(got[-1], ref[-1], F32, f32=1e-3)


def test_recurrence_over_many_chunks_in_a_batch():
    """Sequences of one and of several chunks in one step, some of them with a state in front, against themselves alone."""
    announce("recurrences, chunks of unequal sequences")
    for entry in (delta(2, 1, 48, 40, 4), mamba(4, 2, 32, 24, 4, 2)):
        W, w = 48, weights(entry, 48)
        mix = recurrent(entry, W, F32, w)
        hs = [rand(n, W, seed=n) for n in (210, 20, 128, 65, 1)]
        want = [oracle(entry, h, w) for h in hs]
        cache, feed = slots(mix, 5), Feed(hs, chunk=32)
        parts = [feed.step(mix, cache, [10, 0, 64, 1, 0], F32), feed.step(mix, cache, [200, 20, 64, 64, 1], F32)]
        first = {0: parts[0][0], 2: parts[0][1], 3: parts[0][2]}
        for i, ref in enumerate(want):
            close(torch.cat([first[i], parts[1][i]] if i in first else [parts[1][i]]), ref, F32, f32=1e-4)


def test_convolution_windows_at_the_borders_of_portions():
    """Portions shorter than the taps, one after the other: every token still sees its predecessors' projections."""
    announce("short convolutions over tiny portions")
    for entry in (delta(2, 2, 16, 12, 9), mamba(2, 1, 16, 12, 9), delta(1, 1, 8, 8, 16)):
        W, w = 32, weights(entry, 32)
        mix, h = recurrent(entry, W, F32, w), rand(50, 32, seed=2)
        ref = oracle(entry, h, w)
        for sizes in ([2, 3], [1, 1, 2], [5, 1], [9], [8, 16], [20, 2, 1]):
            close(Feed([h]).run(mix, slots(mix, 1), sizes, F32)[0], ref, F32, f32=1e-4)
