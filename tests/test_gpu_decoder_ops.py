"""Each mechanism of the decoder library alone, on the GPU, against the oracle: row kernels, gated linear attention
(prompt chunks, single steps, portions), latent attention (pages, portions, written-out prompts)."""
import math

import pytest
import torch

from electrock_infer_amd.harness.batch import make_ragged
from electrock_infer_amd.harness.config import SamplingParams
from electrock_infer_amd.harness.sequence import Sequence
from electrock_infer_amd.layers import decoder_ops as ops
from electrock_infer_amd.layers.dense_mlp import DenseMLP
from electrock_infer_amd.layers.gla import GatedLinearAttention
from electrock_infer_amd.layers.latent_attention import LatentAttention
from electrock_infer_amd.layers.token_side import TokenSideInput
from oracle import feguvik_oracle as F
from tests.gpu_util import DEV, announce

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
BLOCK = 8


def rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed)) * scale


def close(got, want, dtype, f32=2e-5, bf16=2e-2):
    """Largest difference relative to the largest expected value."""
    err = float((got.double().cpu() - want.double()).abs().max() / want.double().abs().max())
    assert math.isfinite(err) and err < (f32 if dtype == F32 else bf16), err


def to(t, dtype=F32):
    return t.to(DEV, dtype).contiguous()


# ---- row kernels ----
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,W", [(1, 5), (3, 90), (17, 256), (5, 2052), (2, 9001), (2, 12288)])
def test_embedding_and_residual_norm(T, W, dtype):
    announce(f"rows T={T} W={W} {dtype}")
    table, toks = rand(11, W, seed=1).to(dtype), torch.arange(T) * 7 % 11
    both = torch.full((T, 2 * W), 7.0, dtype=dtype, device=DEV)
    x = ops.embed_rows(toks.int().to(DEV), to(table, dtype), 0.3, both[:, W:])
    want = table.float()[toks] * 0.3
    assert torch.equal(x.cpu(), want) and torch.equal(both[:, W:].cpu(), want.to(dtype)) and bool((both[:, :W] == 7).all())
    y, post, nxt, eps = rand(T, W, seed=2).to(dtype), rand(W, seed=3), rand(W, seed=4), 1e-3
    for update in (ops.KEEP, ops.ADD_NORMED, ops.REPLACE):
        ref = {ops.KEEP: want, ops.ADD_NORMED: want + F.rms_norm(y.float(), post, eps), ops.REPLACE: y.float() + post}[update]
        for next_w, out in ((nxt, torch.empty(T, W, dtype=dtype, device=DEV)), (None, both[:, :W])):
            xg = to(want)
            ops.residual_norm(update, xg, None if update == ops.KEEP else to(y, dtype), to(post), eps, out,
                              None if next_w is None else to(next_w))
            close(xg, ref, F32)
            close(out, ref if next_w is None else F.rms_norm(ref, next_w, eps), dtype, bf16=5e-3)
    if dtype == BF16:                                    # a float32 result into the stream of a bf16 model
        xg = to(want)
        ops.residual_norm(ops.REPLACE, xg, to(y.float() * 1.001), None, eps, torch.empty(T, W, dtype=dtype, device=DEV), to(nxt))
        close(xg, y.float() * 1.001, F32)


@pytest.mark.parametrize("dtype", [F32, BF16])
def test_feed_forward_and_token_side_input(dtype):
    announce(f"dense mlp, token side {dtype}")
    T, W, ff, dim, layer = 13, 90, 77, 5, 2
    x = rand(T, W, seed=1).to(dtype)
    w = {"up": rand(ff, W, seed=2, scale=0.1), "down": rand(W, ff, seed=3, scale=0.1), "l2.side.gate": rand(dim, W, seed=4, scale=0.2),
         "l2.side.proj": rand(W, dim, seed=5), "l2.side.norm": rand(W, seed=6), "side.embed": rand(30, 4 * dim, seed=7)}
    w = {k: v.to(dtype).float() for k, v in w.items()}
    mlp, side = DenseMLP(W, ff, dtype).to(DEV), TokenSideInput(W, dim, layer * dim, dtype).to(DEV)
    mlp.up.data.copy_(w["up"]), mlp.down.data.copy_(w["down"])
    y = mlp(to(x, dtype))
    close(y.sum(0) if y.dim() == 3 else y, F.feed_forward(x.float(), w, "", {"kind": "dense"}), dtype)
    side.gate.data.copy_(w["l2.side.gate"]), side.proj.data.copy_(w["l2.side.proj"]), side.norm.data.copy_(w["l2.side.norm"])
    toks = torch.arange(T) * 5 % 30
    y = side(to(x, dtype), toks.int().to(DEV), to(w["side.embed"], dtype))
    stream = torch.zeros(T, W, device=DEV)
    ops.residual_norm(ops.ADD_NORMED, stream, y, side.norm, 1e-5, None)
    close(stream, F.token_side_input(x.float(), toks, w, layer, dim, 1e-5), dtype)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,W,dim", [(1, 92, 5), (9, 260, 64), (33, 256, 24), (530, 128, 100), (17, 2048, 64), (40, 1024, 160), (530, 384, 32), (20, 4092, 16), (19, 4096, 96), (3, 4100, 7)])
def test_end_of_a_layer_with_token_side_input(T, W, dim, dtype):
    """The one-launch form and the form in steps (float32, or a width that the first does not take)."""
    announce(f"token side, end of layer T={T} W={W} dim={dim} {dtype}")
    eps, vocab, layer = 1e-4, 13, 1
    w = {"l1.side.gate": rand(dim, W, seed=4, scale=W ** -0.5), "l1.side.proj": rand(W, dim, seed=5), "side.embed": rand(vocab, 3 * dim, seed=7)}
    w = {k: v.to(dtype).float() for k, v in w.items()}
    w["l1.side.norm"] = rand(W, seed=6)
    x, y, post, nxt = rand(T, W, seed=1), rand(T, W, seed=2).to(dtype).float(), rand(W, seed=3), rand(W, seed=8)
    toks = torch.arange(T) * 5 % vocab
    ref = x + F.rms_norm(y, post, eps)
    ref = ref + F.token_side_input(ref, toks, w, layer, dim, eps)
    side = TokenSideInput(W, dim, layer * dim, dtype).to(DEV)
    side.gate.data.copy_(w["l1.side.gate"]), side.proj.data.copy_(w["l1.side.proj"]), side.norm.data.copy_(w["l1.side.norm"])
    both = torch.full((T, 2 * W), 5.0, dtype=dtype, device=DEV)
    for next_w, out, one_launch in ((nxt, torch.empty(T, W, dtype=dtype, device=DEV), 0), (None, both[:, :W], 0),
                                    (nxt, torch.empty(T, W, dtype=dtype, device=DEV), 10 ** 9)):
        xg, side.ONE_LAUNCH_ROWS = to(x), one_launch
        side.close_layer(xg, to(y, dtype), to(post), toks.int().to(DEV), to(w["side.embed"], dtype), eps, out,
                         None if next_w is None else to(next_w))
        close(xg, ref, dtype)
        close(out, ref if next_w is None else F.rms_norm(ref, next_w, eps), dtype)
        # no row is worse than the others: the rows of a tile do not mix
        rows = (xg.cpu() - ref).pow(2).mean(-1).sqrt()
        assert float(rows.max()) < (1e-4 if dtype == F32 else 5e-2)
    assert bool((both[:, W:] == 5).all())


@pytest.mark.parametrize("T,N,K", [(1, 5, 64), (16, 300, 192), (17, 48, 640), (33, 33, 1024), (64, 2048, 2048), (32, 2048, 6144), (3, 9000, 128), (16, 9000, 128), (65, 40, 64), (7, 40, 72)])
def test_decode_batch_products(T, N, K):
    """The weight-streaming product in its three forms (and the library's, for shapes that it does not take)."""
    announce(f"skinny gemm {T} {N} {K}")
    x, w = rand(T, K, seed=1).to(BF16), rand(N, K, seed=2, scale=K ** -0.5).to(BF16)
    ref = x.double() @ w.double().t()
    xg, wg = to(x, BF16), to(w, BF16)
    close(ops.linear(xg, wg), ref, BF16, bf16=4e-3)
    close(ops.linear(xg, wg, "relu_squared"), F.relu_squared(ref), BF16, bf16=8e-3 if ops._skinny_splits(xg, wg) else 2e-2)
    close(ops.linear_f32(xg, wg), ref, F32)
    parts = ops.linear_parts(xg, wg, exact=True)
    assert parts.dim() == (3 if ops._skinny_splits(xg, wg) > 1 else 2)
    close(parts.sum(0) if parts.dim() == 3 else parts, ref, F32)
    stream, out = torch.zeros(T, N, device=DEV), torch.empty(T, N, dtype=BF16, device=DEV)
    ops.residual_norm(ops.ADD_NORMED, stream, parts, torch.ones(N, device=DEV), 1e-6, out)
    close(stream, F.rms_norm(ref, torch.ones(N, dtype=torch.float64), 1e-6), F32)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T,H,N,K", [(1, 3, 5, 7), (16, 2, 64, 32), (17, 5, 70, 33), (90, 1, 300, 130), (1, 2, 100, 512), (20, 3, 72, 300)])
def test_head_gemm(T, H, N, K, dtype):
    announce(f"head gemm {T} {H} {N} {K} {dtype}")
    a, b = rand(T, H, K, seed=1).to(dtype), rand(H, N, K, seed=2).to(dtype)
    out = torch.full((T, H, N + 3), 9.0, dtype=dtype, device=DEV)
    ops.head_gemm(to(a, dtype), H * K, K, ops.pad_k(to(b, dtype)), K, out, H * (N + 3), N + 3, T)
    close(out[:, :, :N], torch.einsum("thk,hnk->thn", a.float(), b.float()), dtype)
    assert bool((out[:, :, N:] == 9).all())


# ---- sequences of portions over a pool of pages and slots ----
def portions(total, sizes):
    """Sizes repeated until they cover `total`."""
    out, i = [], 0
    while sum(out) < total:
        out.append(min(sizes[i % len(sizes)], total - sum(out)))
        i += 1
    return out


class Feed:
    """Sequences whose hidden rows are fed portion by portion to one mixer."""

    def __init__(self, hs, chunk=32, order=None):
        Sequence.block_size = BLOCK
        blocks = sum(-(-h.shape[0] // BLOCK) for h in hs)
        free = torch.randperm(blocks + 3, generator=torch.Generator().manual_seed(5)).tolist()
        self.num_blocks, self.chunk, self.hs, self.seqs = blocks + 3, chunk, hs, []
        for i, h in enumerate(hs):
            s = Sequence([0] * h.shape[0], SamplingParams())
            s.block_table, s.state_slot = [free.pop() for _ in range(s.num_blocks)], (order or list(range(len(hs))))[i]
            self.seqs.append(s)

    def step(self, mixer, cache, counts, dtype):
        """Feed counts[i] rows of sequence i (0: not in this step); returns the rows' results by sequence."""
        live = [(s, h, n) for s, h, n in zip(self.seqs, self.hs, counts) if n]
        for s, _, n in live:
            s.num_scheduled_tokens = n
        batch = make_ragged([s for s, _, _ in live], BLOCK, self.chunk, DEV)
        h = torch.cat([h[s.num_computed_tokens:s.num_computed_tokens + n] for s, h, n in live])
        out = mixer(to(h, dtype), batch, cache).float().cpu()
        out = out.sum(0) if out.dim() == 3 else out
        for s, _, n in live:
            s.num_computed_tokens += n
        return list(out.split([n for _, _, n in live]))

    def run(self, mixer, cache, sizes, dtype):
        """Every sequence alone, in portions."""
        outs = []
        for i, h in enumerate(self.hs):
            parts = []
            for n in portions(h.shape[0], sizes):
                parts += self.step(mixer, cache, [n if j == i else 0 for j in range(len(self.hs))], dtype)
            outs.append(torch.cat(parts))
        return outs


def gla_module(W, m, rank, eps, dtype, seed=0, bias=3.0, spread=1.5):
    h, d, v = m["heads"], m["dim"], m["vdim"]
    w = {"q": rand(h * d, W, seed=seed, scale=W ** -0.5), "k": rand(h * d, W, seed=seed + 1, scale=W ** -0.5),
         "v": rand(h * v, W, seed=seed + 2, scale=W ** -0.5), "g": rand(h * v, W, seed=seed + 3, scale=W ** -0.5),
         "o": rand(W, h * v, seed=seed + 4, scale=(h * v) ** -0.5), "norm": 1 + rand(v, seed=seed + 5, scale=0.2),
         "a1": rand(rank, W, seed=seed + 6, scale=W ** -0.5), "a2": rand(h * d, rank, seed=seed + 7, scale=rank ** -0.5),
         "a2.b": bias + rand(h * d, seed=seed + 8, scale=spread)}
    w = {k: (t.to(dtype).float() if t.dim() == 2 else t) for k, t in w.items()}
    mix = GatedLinearAttention(W, h, d, v, m["tau"], rank, eps, dtype).to(DEV)
    for name, (param, section) in mix.TENSORS.items():
        p = mix.get_parameter(param)
        p.weight_loader(p, w[name].to(DEV), section) if section else p.data.copy_(w[name])
    return mix, w


GLA_SIZES = [({"heads": 2, "dim": 19, "vdim": 27, "tau": 5.0}, 7), ({"heads": 3, "dim": 64, "vdim": 48, "tau": 16.0}, 12),
             ({"heads": 1, "dim": 130, "vdim": 144, "tau": 1.0}, 33), ({"heads": 2, "dim": 16, "vdim": 256, "tau": 8.0}, 1),
             ({"heads": 1, "dim": 256, "vdim": 5, "tau": 1.0}, 8)]


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("m,rank", GLA_SIZES)
def test_gla_prompts_steps_and_portions(m, rank, dtype):
    announce(f"gla {m} rank {rank} {dtype}")
    W, eps = 48, 1e-5
    mix, w = gla_module(W, m, rank, eps, dtype)
    w = {"m." + k: t for k, t in w.items()}
    hs = [rand(n, W, seed=50 + n).to(dtype).float() for n in (1, 2, 15, 33, 97)]
    want = [F.gated_linear_attention(h.double(), {k: t.double() for k, t in w.items()}, "m.", m, eps).float() for h in hs]
    for sizes in ([1000], [1], [2], [3, 1, 16], [17, 31], [32]):
        # every slot is full of NaN: a sequence starts from zero, not from what is there
        states = torch.full((7, *mix.state_shape()), float("nan"), device=DEV)
        feed = Feed(hs, order=[4, 0, 6, 2, 1])
        for got, ref in zip(feed.run(mix, states, sizes, dtype), want):
            close(got, ref, dtype, f32=5e-5)
        assert bool(states[5].isnan().all()) and bool(states[3].isnan().all())       # nobody else's slot was touched
    # one batch of all, in unequal portions
    states = torch.full((7, *mix.state_shape()), float("nan"), device=DEV)
    feed = Feed(hs, order=[4, 0, 6, 2, 1])
    parts = [feed.step(mix, states, [1, 2, 9, 20, 64], dtype), feed.step(mix, states, [0, 0, 6, 13, 33], dtype)]
    for i, ref in enumerate(want):
        got = torch.cat([parts[0][i]] + ([parts[1][i - 2]] if i >= 2 else []))
        close(got, ref, dtype, f32=5e-5)


def test_gla_with_decays_that_no_factor_can_hold():
    """Channels that forget everything within a token beside channels that keep everything: e^(-sum of log alpha) of a
    block is far outside float32, and what the lasting channels carry must come through exactly."""
    announce("gla, extreme decays")
    m, W, eps = {"heads": 2, "dim": 40, "vdim": 32, "tau": 1.0}, 48, 1e-6
    mix, w = gla_module(W, m, 4, eps, F32)
    b = torch.full((80,), 60.0)
    b[::3] = -90.0
    b[1::6] = -6.0
    mix.a2_bias.data.copy_(b)
    w["a2.b"] = b
    hs = [rand(n, W, seed=n) for n in (40, 300)]
    want = [F.gated_linear_attention(h.double(), {"m." + k: t.double() for k, t in w.items()}, "m.", m, eps).float() for h in hs]
    for sizes in ([1000], [1], [7]):
        states = torch.full((2, *mix.state_shape()), float("nan"), device=DEV)
        for got, ref in zip(Feed(hs, chunk=64).run(mix, states, sizes, F32), want):
            close(got, ref, F32, f32=5e-5)


@pytest.mark.parametrize("back", [1, 15, 16, 17, 31, 32, 255, 256, 300])
def test_gla_recalls_one_far_token(back):
    """One key stands out and the query asks for it `back` tokens later, across block and chunk borders: read-outs are
    dominated by that token's value."""
    announce(f"gla recall {back}")
    m, W, eps, n = {"heads": 1, "dim": 24, "vdim": 16, "tau": 16.0}, 64, 1e-6, 320
    mix, w = gla_module(W, m, 4, eps, F32, bias=14.0, spread=0.1)          # alpha about 1
    h = rand(n, W, seed=3, scale=0.05)
    h[n - 1 - back] *= 400.0
    key = h[n - 1 - back] @ w["k"].t()
    h[n - 1] += torch.linalg.lstsq(w["q"], key[:, None]).solution[:, 0] * 3
    ref = F.gated_linear_attention(h.double(), {"m." + k: t.double() for k, t in w.items()}, "m.", m, eps).float()
    assert float((ref[n - 1] - F.gated_linear_attention(torch.cat((h[:n - 1 - back], h[n - back:])).double(),
                  {"m." + k: t.double() for k, t in w.items()}, "m.", m, eps).float()[-1]).abs().max()) > 0.1
    for sizes in ([1000], [n - back, 1000], [n - 1, 1], [n - 1 - back, 1, 2]):
        got = Feed([h], chunk=256).run(mix, torch.zeros(1, *mix.state_shape(), device=DEV), sizes, F32)[0]
        close(got[n - 1], ref[n - 1], F32, f32=1e-4)


def mla_module(W, m, eps, dtype, seed=0, q_scale=2.0, sink=None):
    h, d, r, v, c = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    w = {"q": rand(h * (d + r), W, seed=seed, scale=q_scale * W ** -0.5), "dkv": rand(c + r, W, seed=seed + 1, scale=W ** -0.5),
         "dkv.norm": 1 + rand(c, seed=seed + 2, scale=0.2), "uk": rand(h * d, c, seed=seed + 3, scale=c ** -0.5),
         "uv": rand(h * v, c, seed=seed + 4, scale=c ** -0.5), "sink": rand(h, seed=seed + 5) if sink is None else torch.full((h,), sink),
         "o": rand(W, h * v, seed=seed + 6, scale=(h * v) ** -0.5)}
    w = {k: (t.to(dtype).float() if t.dim() == 2 else t) for k, t in w.items()}
    mix = LatentAttention(W, h, d, r, v, c, m["scale"], m["rot"]["base"], eps, dtype).to(DEV)
    for name, (param, section) in mix.TENSORS.items():
        p = mix.get_parameter(param)
        p.weight_loader(p, w[name].to(DEV), section) if section else p.data.copy_(w[name])
    mix.finish_loading()
    return mix, w


def mla(heads, dim, rot, vdim, rank, scale=None, base=10000.0):
    return {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "scale": scale or (dim + rot) ** -0.5,
            "rot": {"base": base, "dims": rot}}


MLA_SIZES = [mla(3, 22, 6, 20, 37, base=300.0), mla(5, 48, 16, 40, 72), mla(1, 64, 32, 128, 200, scale=0.2),
             mla(17, 8, 2, 8, 9), mla(2, 40, 128, 24, 512), mla(2, 128, 64, 100, 256)]


def latent_oracle(h, w, m, eps):
    return F.latent_attention(h.double(), {"m." + k: t.double() for k, t in w.items()}, "m.", m, eps).float()


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("m", MLA_SIZES)
def test_latent_attention_prompts_steps_and_portions(m, dtype):
    announce(f"latent {m} {dtype}")
    W, eps = 56, 1e-5
    mix, w = mla_module(W, m, eps, dtype)
    hs = [rand(n, W, seed=50 + n).to(dtype).float() for n in (1, 2, BLOCK, BLOCK + 1, 31, 131)]
    want = [latent_oracle(h, w, m, eps) for h in hs]
    for sizes in ([1000], [1], [2], [3, 1, 16], [64, 67], [70, 1], [BLOCK]):
        feed = Feed(hs)
        cache = torch.full((feed.num_blocks, BLOCK, mix.row_elems()), float("nan"), dtype=dtype, device=DEV)
        for got, ref in zip(feed.run(mix, cache, sizes, dtype), want):
            close(got, ref, dtype, bf16=3e-2)
    feed = Feed(hs)
    cache = torch.full((feed.num_blocks, BLOCK, mix.row_elems()), float("nan"), dtype=dtype, device=DEV)
    parts = [feed.step(mix, cache, [1, 1, 2, 8, 13, 66], dtype), feed.step(mix, cache, [0, 1, 6, 1, 18, 65], dtype)]
    for i, ref in enumerate(want):
        got = torch.cat([parts[0][i]] + ([parts[1][i - 1]] if i >= 1 else []))
        close(got, ref, dtype, bf16=3e-2)
    assert mix.pitch == m["kv_rank"] or not bool(cache[..., m["kv_rank"]:mix.pitch].nan_to_num().any())


@pytest.mark.parametrize("splits", [1, 2, 5, 64])
def test_latent_attention_is_the_same_for_every_number_of_splits(splits, monkeypatch):
    announce(f"latent splits {splits}")
    m, W = mla(3, 24, 8, 16, 40), 56
    mix, w = mla_module(W, m, 1e-5, F32)
    monkeypatch.setattr(mix, "splits", lambda batch: splits)
    h = rand(150, W, seed=9)
    feed = Feed([h])
    cache = torch.full((feed.num_blocks, BLOCK, mix.row_elems()), float("nan"), device=DEV)
    close(feed.run(mix, cache, [100, 1, 2, 30], F32)[0], latent_oracle(h, w, m, 1e-5), F32)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("sink", [-30.0, 0.0, 12.0, 200.0])
def test_latent_attention_sink(sink, dtype):
    announce(f"latent sink {sink} {dtype}")
    m, W = mla(4, 32, 16, 32, 48), 64
    mix, w = mla_module(W, m, 1e-5, dtype, sink=sink)
    h = rand(80, W, seed=9).to(dtype).float()
    ref = latent_oracle(h, w, m, 1e-5)
    for sizes in ([1000], [79, 1], [9]):
        feed = Feed([h])
        cache = torch.zeros(feed.num_blocks, BLOCK, mix.row_elems(), dtype=dtype, device=DEV)
        got = feed.run(mix, cache, sizes, dtype)[0]
        if sink > 100:
            assert float(got.abs().max()) < 1e-6                  # the sink takes all the weight
        else:
            close(got, ref, dtype, bf16=3e-2)


@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("key", [0, 1, BLOCK - 1, BLOCK, 31, 32, 63, 64, 127, 128, 190, 198, 199])
def test_latent_attention_finds_one_key_among_many(key, dtype):
    """The last query and one key are scaled up against each other: the result is that key's value alone, so a key that
    is dropped, doubled or read from another page shows at full size."""
    announce(f"latent far key {key} {dtype}")
    n, W = 200, 96
    m = mla(2, 32, 8, 32, 64, scale=0.2)
    mix, w = mla_module(W, m, 1e-6, dtype, q_scale=1.0, sink=-5.0)
    h = rand(n, W, seed=1)
    # the query of head 0 points at the key that token `key` has there
    c = F.rms_norm(h[key] @ w["dkv"][:64].t(), w["dkv.norm"], 1e-6)
    k = c @ w["uk"][:32].t()
    if key != n - 1:
        h[n - 1] = torch.linalg.lstsq(w["q"][:32], (k * 12)[:, None]).solution[:, 0]
    h = h.to(dtype).float()
    ref = latent_oracle(h, w, m, 1e-6)
    for sizes in ([1000], [n - 1, 1], [90, 1000], [64, 64, 70, 2]):
        feed = Feed([h])
        cache = torch.full((feed.num_blocks, BLOCK, mix.row_elems()), float("nan"), dtype=dtype, device=DEV)
        got = feed.run(mix, cache, sizes, dtype)[0]
        close(got[n - 1], ref[n - 1], dtype, bf16=6e-2)


def test_written_out_prompts_match_the_paged_kernel():
    """The two kernels of long portions on the same bf16 inputs, with a cached context in front and unequal sequences."""
    announce("latent, written out against paged")
    for m in (mla(4, 64, 32, 64, 128), mla(2, 48, 16, 40, 72), mla(3, 128, 64, 128, 512), mla(2, 24, 8, 12, 16), mla(1, 184, 72, 128, 64)):
        W = 64
        mix, w = mla_module(W, m, 1e-6, BF16)
        hs = [rand(n, W, seed=n).to(BF16).float() for n in (300, 129, 65, 200)]
        outs = []
        for limit in (64, 10 ** 9):
            mix.PROMPT_TOKENS = limit
            feed = Feed(hs)
            cache = torch.full((feed.num_blocks, BLOCK, mix.row_elems()), float("nan"), dtype=BF16, device=DEV)
            first = feed.step(mix, cache, [100, 129, 1, 37], BF16)
            second = feed.step(mix, cache, [200, 0, 64, 163], BF16)
            outs.append([torch.cat((first[0], second[0])), first[1], torch.cat((first[2], second[1])), torch.cat((first[3], second[2]))])
        assert mix.writes_out(type("B", (), {"max_q": 10 ** 9})(), BF16)
        for a, b, h in zip(*outs, hs):
            ref = latent_oracle(h, w, m, 1e-6)
            close(a, ref, BF16, bf16=3e-2)
            close(b, ref, BF16, bf16=3e-2)
