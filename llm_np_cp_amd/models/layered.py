"""GPU engine of the layer-list designs: paged mixed-batch steps.

One batch holds any mix of prompt portions and single decoded tokens, each
row with its own sequence and position.  ``step()`` runs such a batch from
the pages and state slots that earlier steps left; prompts, the row
primitives of the batching server and the captured decode step all run
the same layer stack over the same cache.

The residual stream, projections, norms, scores, routing and recurrent
state are fp32; dtype "bf16" keeps weights, the normed layer input and the
cached latents, keys and values in bf16 (fp32 accumulation), "fp32"
everything in true fp32.
"""

from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Sequence as Seq

import numpy as np
import torch

from ..core.layered import LayeredConfig
from ..ops import hip_ops as ho
from ..ops import hybrid_ops as hy
from ..parallel import tp as tpu
from ..runtime.cache_manager import CacheFull, CacheManager, Sequence
from ..utils.tracing import trace_range
from .blocks import BLOCKS
from .decode_loop import DecodeLoop, DeviceCacheHandle
from .mixers import FEW, Packer, pad_to


@dataclass
class StepEntry:
    """The next tokens of one sequence; ``want`` are the places among them
    whose logits are returned."""
    seq: Sequence
    tokens: np.ndarray
    want: Seq[int] = ()


@dataclass
class Rows:
    """One batch on the device.  Rows [0, nd) are single tokens; the rest
    belong to nseg runs of at least two tokens."""
    T: int
    nd: int
    ids: torch.Tensor
    slot: torch.Tensor
    pos: torch.Tensor
    seg_row0: torch.Tensor
    seg_len: torch.Tensor
    seg_slot: torch.Tensor
    seg_pos0: torch.Tensor
    nseg: int = 0
    nchunk: int = 0
    seg_chunk0: object = 0
    chunk_row0: object = 0
    chunk_len: object = 0
    chunk_seg: object = 0
    tiles: Dict[int, tuple] = field(default_factory=dict)


class LayeredModel(DecodeLoop):
    def __init__(self, config: LayeredConfig, weights, dtype: str = "bf16",
                 max_seq: Optional[int] = 4096, prefill_chunk: int = 2048,
                 device: Optional[str] = None, seed: int = 0,
                 kv_dtype: str = "bf16", max_batch: int = 1,
                 pool_tokens: Optional[int] = None):
        """``pool_tokens`` sizes the page pool (default: max_seq tokens for
        each of max_batch sequences); ``max_batch`` is the number of
        sequence slots."""
        if dtype not in ("bf16", "fp32"):
            raise ValueError(f"{config.model_type} runs in bf16 or fp32, "
                             f"not {dtype!r}")
        if kv_dtype != "bf16":
            raise ValueError(f"{config.model_type} caches in the compute "
                             f"dtype; kv_dtype {kv_dtype!r} is not "
                             f"available")
        if not torch.cuda.is_available():
            raise RuntimeError("LayeredModel requires a GPU (MI355X)")
        from ..io.loader import validate_weights
        validate_weights(config, weights)
        assert 1 <= max_batch <= 256
        self.rank, self.world = tpu.init_distributed()
        if self.world > 1:
            raise ValueError(f"{config.model_type} runs on one GPU "
                             f"(no tensor parallelism)")
        self.config = self.cfg = config
        self.seed, self.dtype, self.kv_dtype = seed, dtype, kv_dtype
        self.f32 = 1 if dtype == "fp32" else 0
        self.T = torch.float32 if self.f32 else torch.bfloat16
        self.device = torch.device(device or "cuda:0")
        torch.cuda.set_device(self.device)
        self.W = config.hidden_size
        self.Wp = pad_to(self.W, 64)
        self.max_batch = max_batch
        self.max_seq = max_seq or min(config.max_position_embeddings, 131072)
        self.no_rewind = config.recurrent
        pages = -(-(pool_tokens or max_batch * pad_to(self.max_seq, hy.PAGE))
                  // hy.PAGE)
        self.cache = CacheManager(pages, max_batch, hy.PAGE, self.max_seq)
        self._tables: Dict[tuple, tuple] = {}
        self._upload(weights)
        self._alloc(min(prefill_chunk, pad_to(self.max_seq * max_batch, 64)))
        self._graph = None
        self._graph_mode = None
        self.reset()

    # ------------------------------------------------------------------
    # weights, cache, scratch
    # ------------------------------------------------------------------
    def rope_tables(self, base: float, dims: int):
        """cos/sin of position * base**(-2i/dims), fp32 from fp64."""
        f = base ** (-2.0 * np.arange(dims // 2) / dims)
        return self._position_table(("rope", base, dims), lambda p: [
            fn(np.outer(p, f)) for fn in (np.cos, np.sin)])

    def query_temperature(self, coef: float, every: float):
        """1 + coef ln(floor((p + 1) / every) + 1) per position p."""
        return self._position_table(("temp", coef, every), lambda p: [
            1.0 + coef * np.log(np.floor((p + 1) / every) + 1.0)])[0]

    def _position_table(self, key, make):
        if key not in self._tables:
            n = self.cache.table.shape[1] * hy.PAGE
            self._tables[key] = tuple(
                torch.from_numpy(t.astype(np.float32)).to(self.device)
                for t in make(np.arange(n, dtype=np.float64)))
        return self._tables[key]

    def _upload(self, weights):
        cfg = self.cfg
        pk = Packer(weights, self.device, self.T)
        self.embed = pk.raw("embed").to(self.T).contiguous()
        self.head = pk.rows(["head"], self.W)
        self.g_final = pk.f32("final.norm") * cfg.logit_scale
        self.streams, self.pairs = cfg.streams, None
        if cfg.streams > hy.MAX_STREAMS:
            raise ValueError(f"{cfg.model_type}: {cfg.streams} streams "
                             f"exceed the built kernels ({hy.MAX_STREAMS})")
        if cfg.streams:
            self.read_all = torch.ones(cfg.streams, device=self.device)
        if cfg.bigram:
            self.pairs = pk.raw("bigram").to(self.T).contiguous()
            # the token before the next one of every slot's sequence
            self.last = torch.zeros(self.max_batch, dtype=torch.int32,
                                    device=self.device)
        self.win_loop = (pk.rows(["loop.in"], 2 * self.W)
                         if cfg.loop and cfg.design.loop == "project"
                         else None)
        block = BLOCKS[cfg.design.block]
        # layers that use another one's tensors have none of their own
        self.layers = {i: block(self, cfg.layers[i], pk, i)
                       for i in sorted({i for i, _ in cfg.runs})}
        # every run of a looped or shared layer has its own cache or state
        self.caches = [self.layers[i].new_cache(self) for i, _ in cfg.runs]

    def decode_splits(self, rows: int) -> int:
        """Key-range splits of single-token attention: fixed by the cache
        size and the number of rows, so a captured step keeps its grid.
        (Measured: 64 up to 4 rows, 32 at 16, from 100 to 7000 keys.)"""
        tiles = -(-self.cache.table.shape[1] * hy.PAGE // 32)
        return int(max(2, min(64, tiles // 2, 512 // rows)))

    def run_splits(self, tiles: int, longest: int) -> int:
        """Splits for `tiles` query tiles against up to `longest` keys."""
        if tiles >= 256:
            return 1
        return int(max(1, min(32, 512 // tiles, longest // 256)))

    def max_chunks(self, rows: int) -> int:
        """Recurrence chunks that a batch of `rows` rows can have."""
        return rows // hy.CHUNK + self.max_batch + 1

    def _alloc(self, PC: int):
        cfg, dev, B = self.cfg, self.device, self.max_batch
        PC = self.PC = max(PC, B, FEW)
        f32 = dict(dtype=torch.float32, device=dev)
        i32 = dict(dtype=torch.int32, device=dev)
        tt = dict(dtype=self.T, device=dev)
        S = max(self.streams, 1)
        self.x = torch.zeros(PC, S * self.W, **f32)
        self.xb = torch.zeros(PC, S * self.W, **f32)
        self.x0 = torch.zeros(PC, self.W, **f32) if cfg.loop else None
        self.h = torch.zeros(PC, self.Wp, **tt)
        self.cat = (torch.zeros(PC, self.win_loop.shape[1], **tt)
                    if self.win_loop is not None else None)
        self.y = (torch.zeros(PC, self.W, **f32)
                  if cfg.design.block != "parallel" else None)
        if self.streams:             # two halves of a pair's output
            self.y = torch.zeros(2, PC, self.W, **f32)
        self.pend, self.add0, self.turn = None, False, None
        layers = self.layers.values()
        self.P = torch.zeros(PC * max(l.p_floats for l in layers), **f32)
        need: Dict[str, int] = {}
        for l in layers:
            for k, n in l.mixer.sizes(self, PC).items():
                need[k] = max(need.get(k, 0), n)
        for k in ("q", "qn", "qa", "olat", "o", "part", "ml", "raw", "gF",
                  "gi", "gm", "cm0", "U", "un", "decay", "local", "cq", "qf",
                  "u"):
            kw = tt if k in ("q", "qn", "qa", "olat", "o", "cq") else f32
            setattr(self, k, torch.zeros(max(need.get(k, 0), 1), **kw))
        ex = [l.experts or l.ff.experts for l in layers
              if l.experts or getattr(l, "ff", None) and l.ff.experts]
        K1 = max((e.K1 for e in ex), default=1)
        self.ridx = torch.zeros(PC * K1, **i32)
        self.rwt = torch.zeros(PC * K1, **f32)
        self.act = torch.zeros(
            max(1, PC * max(l.act_floats for l in layers)), **tt)
        self.ypair = torch.zeros(PC * K1 * self.W if ex else 1, **tt)
        self.perm = torch.zeros(PC * K1, **i32)
        nt = PC * K1 // 32 + max((e.spec.experts + 1 for e in ex), default=1)
        self.tile_e, self.tile_row0, self.tile_n = (
            torch.zeros(nt, **i32) for _ in range(3))
        # block table and per-row decode state
        self.table = torch.zeros(self.cache.table.shape, **i32)
        self._table_version = -1
        S, V = self.max_seq, cfg.vocab_size
        i64 = dict(dtype=torch.int64, device=dev)
        self.bt_slot = torch.zeros(B, **i32)
        self.bt_lens = torch.zeros(B, **i32)
        self.bt_next = torch.zeros(B, **i32)
        self.bt_nout = torch.zeros(B, **i32)
        self.bt_cnt = torch.zeros(B, **i32)
        self.bt_gmax = torch.zeros(B, **i64)
        self.bt_pick = torch.zeros(B, **i64)
        self.bt_ring = torch.zeros(B, S + 16, **i32)
        self.bt_logits32 = torch.zeros(B, V, **f32)
        self.rng_ctr = torch.zeros(1, **i64)
        self._iota = torch.arange(B, **i32)
        self._ones = torch.ones(B, **i32)
        # a single sequence is row 0 of the batch
        self.b_logits = self.bt_logits32[0]
        self.len_buf, self.next_token = self.bt_lens[:1], self.bt_next[:1]
        self.nout, self.out_ring = self.bt_nout[:1], self.bt_ring[0]
        self.s_gmax, self.s_pick = self.bt_gmax[:1], self.bt_pick[:1]
        self.s_cnt = self.bt_cnt[:1]
        heads = {l.mixer.tile_pairs for l in layers} - {None}
        self._tile_pairs = sorted(heads)
        self._meta = torch.zeros(
            3 * PC + 8 * (B + 2) + 3 * (PC // hy.CHUNK + B + 2) + PC +
            sum(2 * (PC * h // hy.TILE + B + 2) for h in heads), **i32)

    # ------------------------------------------------------------------
    # layer stack
    # ------------------------------------------------------------------
    def _sync_table(self):
        if self._table_version != self.cache.version:
            self.table.copy_(torch.from_numpy(self.cache.table))
            self._table_version = self.cache.version

    def _layer_stack(self, b: Rows, layer_hook=None):
        """Embedding and every layer run over the batch; leaves the
        residual stream of its rows in self.x."""
        cfg, T = self.cfg, b.T
        self.pend, self.add0, self.turn = None, False, None
        if self.pairs is not None:
            hy.embed_pairs(self.embed, self.pairs, self.last, b, self.x,
                           self.W, self.streams, cfg.bigram)
        else:
            hy.embed_rows(self.embed, b.ids, self.x, self.x0, T,
                          cfg.embed_scale)
        if layer_hook is not None:
            layer_hook(-1, self._residual(T, 1.0 / max(self.streams, 1)))
        for j, (i, comes_in) in enumerate(cfg.runs):
            if comes_in:
                if self.win_loop is None:      # x + x0, with what comes next
                    self.add0 = True
                else:                          # x <- W_in [x; x0]
                    self.project(self.win_loop, self.cat, self.xb, T)
                    self.x, self.xb = self.xb, self.x
            self.layers[i].run(self, b, self.caches[j])
            if layer_hook is not None:
                self._settle(T)
                layer_hook(j, self._residual(T))

    def _residual(self, T: int, scale: float = 1.0):
        """The residual of the first T rows; of several streams the sum."""
        x = self.x[:T]
        return (x.view(T, self.streams, self.W).sum(1) * scale
                if self.streams else x)

    def _pending(self):
        """What the residual still lacks: staging arguments, then cleared."""
        kw = {}
        if self.pend is not None:
            kw.update(y=self.y, gb=self.pend)
        if self.add0:
            kw.update(xadd=self.x0)
        self.pend, self.add0 = None, False
        return kw

    def _turning(self):
        """What the streams still lack: staging arguments, then cleared."""
        kw = {"S": self.streams}
        if self.turn is not None:
            c, halves = self.turn
            kw.update(y=self.y[0], mix=c.mix, feed=c.feed, **halves)
        self.turn = None
        return kw

    def _settle(self, T: int):
        if self.turn is not None:
            hy.hyper_rows(self.x, None, T, self.W, self.W, self.cfg.norm_eps,
                          xout=self.x, **self._turning())
        kw = self._pending()
        if kw:
            hy.norm_rows(self.x, None, None, T, self.W, self.W,
                         self.cfg.norm_eps, xout=self.x, **kw)

    def one_row(self, w, T: int) -> bool:
        return T == 1 and w.shape[1] * w.element_size() <= 1 << 17

    def project(self, w, staged, out, T: int, g=None, rows=None, cap=None,
                bias=None, epi=hy.EPI_F32):
        """out[T, N] = w . norm(x) with weights g, or w . [x | x0] without;
        the staged input stays in `staged`.  Whatever is pending on the
        residual is done on the way.  One row runs as a fused GEMV."""
        (N, K), W, eps = w.shape, self.W, self.cfg.norm_eps
        kw = self._pending()
        keep = bool(kw) and rows is None
        if self.one_row(w, T):
            if keep:           # other blocks still read x: write beside it
                kw["xout"] = self.xb
            res = {"res": kw.pop("y")} if "y" in kw else {}
            hy.lin_row(w, self.x, out, W, eps, g=g,
                       x0=self.x0 if g is None else None, rows=rows,
                       hout=staged, cap=cap or 0.0, bias=bias, epi=epi,
                       **res, **kw)
            if keep:
                self.x, self.xb = self.xb, self.x
            return
        if g is None:
            hy.norm_rows(self.x, None, staged, T, W, K, eps, x0=self.x0)
        else:
            if keep:
                kw["xout"] = self.x
            hy.norm_rows(self.x, g, staged, T, W, K, eps, rows=rows, **kw)
        hy.gemm_rows(staged, w, out, T, K, N,
                     epi if cap is None else hy.EPI_SOFTCAP, mult=cap or 0.0,
                     bias=bias)

    def read_streams(self, w, out, T: int, read, g, rows=None, bias=None,
                     epi=hy.EPI_F32):
        """out[T, N] = w . norm(sum of the streams weighted by read), a norm
        with the single gain g.  What is due on the streams is done on the
        way.  One row runs as a fused GEMV."""
        (N, K), W, eps = w.shape, self.W, self.cfg.norm_eps
        kw = self._turning()
        keep = "y" in kw and rows is None
        one = self.one_row(w, T)
        if keep:               # one row: other blocks still read x
            kw["xout"] = self.xb if one else self.x
        kw.update(read=read, g=g)
        if one:
            hy.lin_row(w, self.x, out, W, eps, rows=rows, bias=bias, epi=epi,
                       hyper=kw)
            if keep:
                self.x, self.xb = self.xb, self.x
            return
        hy.hyper_rows(self.x, self.h, T, W, K, eps, rows=rows, **kw)
        hy.gemm_rows(self.h, w, out, T, K, N, epi, bias=bias)

    def linear(self, w, src, out, T: int, bias=None):
        """out[T, N] fp32 = w . src + bias, rows of src as wide as w's."""
        N, K = w.shape
        if self.one_row(w, T):
            hy.lin_row(w, None, out, 0, 0.0, hin=src, bias=bias)
        else:
            hy.gemm_rows(src, w, out, T, K, N, hy.EPI_F32, bias=bias)

    def normed_linear(self, w, staged, out, T: int, src, W: int, g, gate=None,
                      ldg: int = 0, groups: int = 1):
        """out[T, N] fp32 = w . (norm(src) sigmoid(gate)), src [T, W], or
        with the norm over each of `groups` equal parts."""
        (N, K), eps = w.shape, self.cfg.norm_eps
        if self.one_row(w, T):
            hy.lin_row(w, src, out, W, eps, g=g, gate=gate, ldg=ldg,
                       groups=groups)
        else:
            if groups > 1:
                hy.group_rows(src, g, staged, T, W, K, eps, groups)
            else:
                hy.norm_rows(src, g, staged, T, W, K, eps, gate=gate, ldg=ldg)
            hy.gemm_rows(staged, w, out, T, K, N, hy.EPI_F32)

    def conv_project(self, w, kernel, ring, b: Rows, out, narrow=False):
        """out[T, N] fp32 = w . (v + conv(v)), v the residual with what is
        pending on it; the staged input stays in self.h.  True where a
        `narrow` w (up to 64 rows) ran as the other operand: out[N, T]."""
        (N, K), W, eps, T = w.shape, self.W, self.cfg.norm_eps, b.T
        kw = self._pending()
        keep = bool(kw)
        if keep:               # earlier rows are read again: write beside
            kw["xout"] = self.xb
        conv = (kernel, ring, b.slot, b.pos)
        if self.one_row(w, T):
            res = {"res": kw.pop("y")} if keep else {}
            hy.lin_row(w, self.x, out, W, eps, hout=self.h, conv=conv, **res,
                       **kw)
        else:
            hy.conv_rows(self.x, self.h, b, W, K, eps, conv, **kw)
        if keep:
            self.x, self.xb = self.xb, self.x
        if self.one_row(w, T):
            return False
        if narrow and N <= 64 < T:
            hy.gemm_rows(w, self.h, out, N, K, T, hy.EPI_F32, N=T)
            return True
        hy.gemm_rows(self.h, w, out, T, K, N, hy.EPI_F32)
        return False

    def poly_linear(self, w, z, W: int, coef, staged, out, T: int):
        """out[T, N] fp32 = w . polynorm(z), rows of W values in z."""
        (N, K), eps = w.shape, self.cfg.norm_eps
        if self.one_row(w, T):
            hy.lin_row(w, z, out, W, eps, act=coef)
        else:
            hy.poly_rows(z, K, coef, staged, T, W, eps)
            hy.gemm_rows(staged, w, out, T, K, N, hy.EPI_F32)

    def _head(self, out: torch.Tensor, n: int, rows=None):
        """Final norm, head and soft cap of n rows -> out [n, vocab]."""
        if self.streams:
            self.read_streams(self.head, out, n, self.read_all, self.g_final,
                              rows=rows)
            return
        self.project(self.head, self.h, out, n, self.g_final, rows=rows,
                     cap=self.cfg.logit_softcap or 0.0)

    # ------------------------------------------------------------------
    # mixed-batch step
    # ------------------------------------------------------------------
    def open_sequence(self) -> Sequence:
        return self.cache.open()

    def close_sequence(self, seq: Sequence) -> None:
        self.cache.close(seq)

    def step(self, entries: List[StepEntry], layer_hook=None) -> torch.Tensor:
        """Run the entries' tokens as one batch and return the wanted
        logits, [wanted, vocab] fp32 on the device, in entry order.  Pages
        are reserved for the whole step first; CacheFull leaves everything
        as it was.  A step beyond the scratch size runs as several
        batches."""
        entries = [StepEntry(e.seq, np.asarray(e.tokens, np.int32).ravel(),
                             [int(k) for k in e.want]) for e in entries]
        if len({id(e.seq) for e in entries}) != len(entries):
            raise ValueError("a sequence appears twice in one step")
        missing = 0
        for e in entries:
            n = len(e.tokens)
            if n == 0:
                raise ValueError("empty ids")
            if e.tokens.min() < 0 or e.tokens.max() >= self.cfg.vocab_size:
                raise ValueError("token id outside the vocabulary")
            if any(not 0 <= k < n for k in e.want):
                raise ValueError("wanted place outside the tokens")
            if e.seq.length + n > self.max_seq:
                raise ValueError(f"sequence {e.seq.length}+{n} exceeds "
                                 f"max_seq {self.max_seq}")
            missing += self.cache.missing(e.seq, e.seq.length + n)
        if missing > self.cache.free_pages:
            raise CacheFull(f"{missing} more pages needed, "
                            f"{self.cache.free_pages} free")
        for e in entries:
            self.cache.reserve(e.seq, e.seq.length + len(e.tokens))
        out = torch.empty(sum(len(e.want) for e in entries),
                          self.cfg.vocab_size, dtype=torch.float32,
                          device=self.device)
        done = 0
        parts, room = [], self.PC
        for e in entries:
            at = 0
            while at < len(e.tokens):
                n = min(room, len(e.tokens) - at)
                parts.append((e.seq, e.tokens[at:at + n],
                              [k - at for k in e.want if at <= k < at + n]))
                at += n
                room -= n
                if room == 0:
                    done += self._run_parts(parts, out[done:], layer_hook)
                    parts, room = [], self.PC
        if parts:
            self._run_parts(parts, out[done:], layer_hook)
        return out

    def _run_parts(self, parts, out, layer_hook) -> int:
        order = sorted(range(len(parts)), key=lambda k: len(parts[k][1]) > 1)
        T = sum(len(p[1]) for p in parts)
        nd = sum(len(p[1]) == 1 for p in parts)
        row0, r = {}, 0
        for k in order:
            row0[k] = r
            r += len(parts[k][1])
        cols: Dict[str, list] = {n: [] for n in (
            "ids", "slot", "pos", "seg_row0", "seg_len", "seg_slot",
            "seg_pos0", "seg_chunk0", "chunk_row0", "chunk_len",
            "chunk_seg")}
        for k in order:
            seq, tok, _ = parts[k]
            n = len(tok)
            cols["ids"].append(tok)
            cols["slot"].append(np.full(n, seq.slot, np.int32))
            cols["pos"].append(np.arange(seq.length, seq.length + n,
                                         dtype=np.int32))
            cols["seg_row0"].append(row0[k])
            cols["seg_len"].append(n)
            cols["seg_slot"].append(seq.slot)
            cols["seg_pos0"].append(seq.length)
            if n > 1:
                run = len(cols["seg_chunk0"])
                cols["seg_chunk0"].append(len(cols["chunk_row0"]))
                for t in range(0, n, hy.CHUNK):
                    cols["chunk_row0"].append(row0[k] + t)
                    cols["chunk_len"].append(min(hy.CHUNK, n - t))
                    cols["chunk_seg"].append(run)
        nchunk = len(cols["chunk_row0"])
        # query tiles of the runs, latest (most keys) first
        longest = max([parts[k][0].length + len(parts[k][1])
                       for k in order[nd:]], default=0)
        tiles = {}
        for H in self._tile_pairs:
            t = [(seg, rr) for seg, k in enumerate(order) if seg >= nd
                 for rr in range(0, len(parts[k][1]) * H, hy.TILE)]
            t.sort(key=lambda s: -(parts[order[s[0]]][0].length + s[1] // H))
            cols[f"ts{H}"] = [s for s, _ in t]
            cols[f"tr{H}"] = [rr for _, rr in t]
            tiles[H] = len(t)
        want = [row0[k] + w for k in range(len(parts)) for w in parts[k][2]]
        cols["want"] = want
        flat, off = [], {}
        at = 0
        for name, v in cols.items():
            a = (np.concatenate(v) if v and isinstance(v[0], np.ndarray)
                 else np.asarray(v, dtype=np.int32))
            off[name] = (at, len(a))
            flat.append(a.astype(np.int32, copy=False))
            at += len(a)
        host = np.concatenate(flat)
        assert len(host) <= self._meta.numel()
        self._meta[:at].copy_(torch.from_numpy(host))
        dev = {n: self._meta[a:a + c] for n, (a, c) in off.items()}
        self._sync_table()
        b = Rows(T=T, nd=nd, ids=dev["ids"], slot=dev["slot"],
                 pos=dev["pos"], seg_row0=dev["seg_row0"],
                 seg_len=dev["seg_len"], seg_slot=dev["seg_slot"],
                 seg_pos0=dev["seg_pos0"], nseg=len(parts) - nd,
                 nchunk=nchunk, seg_chunk0=dev["seg_chunk0"],
                 chunk_row0=dev["chunk_row0"], chunk_len=dev["chunk_len"],
                 chunk_seg=dev["chunk_seg"],
                 tiles={H: (dev[f"ts{H}"], dev[f"tr{H}"], n, longest)
                        for H, n in tiles.items()})
        self._layer_stack(b, layer_hook)
        if want:
            self._head(out, len(want), dev["want"])
        for seq, tok, _ in parts:
            seq.length += len(tok)
        return len(want)

    # ------------------------------------------------------------------
    # generation interface (rows of the lockstep group)
    # ------------------------------------------------------------------
    def reset(self):
        self.cache.close_all()
        self.rows: List[Optional[Sequence]] = [None] * self.max_batch
        for t in (self.bt_lens, self.bt_nout, self.rng_ctr, self.bt_gmax,
                  self.bt_pick, self.bt_cnt):
            t.zero_()
        self._host_len = 0
        self._host_lens = [0] * self.max_batch
        self._batch_n = 0

    def _open_row(self, b: int) -> Sequence:
        if self.rows[b] is not None:
            self.cache.close(self.rows[b])
        self.rows[b] = seq = self.cache.open()
        self.bt_slot[b:b + 1].fill_(seq.slot)
        return seq

    def _reserve(self, lens):
        for b, n in enumerate(lens):
            self.cache.reserve(self.rows[b], n)
        self._sync_table()

    def _append_row0(self, ids, pos0: int, want, layer_hook=None):
        ids = np.asarray(ids, dtype=np.int32).ravel()
        if len(ids) == 0:
            raise ValueError("empty ids")
        if pos0 + len(ids) > self.max_seq:
            raise ValueError(f"sequence {pos0}+{len(ids)} exceeds max_seq "
                             f"{self.max_seq}")
        seq = self.rows[0] or self._open_row(0)
        seq.length = pos0        # the device loop advances on its own
        out = self.step([StepEntry(seq, ids, want)], layer_hook)
        self.bt_lens[:1].fill_(pos0 + len(ids))
        self._host_len = pos0 + len(ids)
        return out

    def forward(self, ids: np.ndarray, cache: DeviceCacheHandle,
                pos0: int) -> np.ndarray:
        """Last-position logits (1, V) fp32."""
        if pos0 != cache.seq_len:
            raise ValueError("GPU engine requires sequential positions")
        n = np.asarray(ids).size
        out = self._append_row0(ids, pos0, [n - 1] if n else [])
        self.b_logits.copy_(out[0])
        cache.seq_len = pos0 + n
        return out.cpu().numpy()

    def forward_positions(self, ids: np.ndarray, pos0: int) -> np.ndarray:
        """All-position logits (M, V), continuing from pos0."""
        n = np.asarray(ids).size
        return self._append_row0(ids, pos0, range(n)).cpu().numpy()

    def forward_full(self, ids: np.ndarray,
                     return_hidden_states: bool = False):
        """All-position logits of a fresh sequence; optionally with the
        residual stream after the embedding and after every layer run."""
        self.reset()
        n = np.asarray(ids).size
        if not return_hidden_states:
            return self.forward_positions(ids, 0)
        hidden = [[] for _ in range(len(self.cfg.runs) + 1)]

        def hook(i, x):
            hidden[i + 1].append(x.cpu().numpy())
        out = self._append_row0(ids, 0, range(n), hook)
        return out.cpu().numpy(), [np.concatenate(h) for h in hidden]

    def rewind(self, n: int):
        """Drop the tokens from position n on.  Attention caches can; a
        recurrent state cannot be rolled back, so with recurrent layers
        only the current length (or 0) is possible."""
        if not 0 <= n <= self.max_seq:
            raise ValueError(f"rewind {n} outside [0, {self.max_seq}]")
        if n == 0:
            return self.reset()
        cur = int(self.bt_lens[0].item())
        if n > cur or (n < cur and self.no_rewind):
            raise ValueError(f"cannot rewind from {cur} to {n}: "
                             f"{self.cfg.model_type} carries recurrent state")
        self.rows[0].length = n
        self.bt_lens[:1].fill_(n)
        self._host_len = n

    def _decode_step(self, greedy: bool, min_p: float,
                     temperature: float = 1.0):
        self._decode_batch_step(1, greedy, min_p, temperature)

    def _decode_batch_step(self, B: int, greedy: bool, min_p: float,
                           temperature: float = 1.0):
        """One token for rows [0, B); all state is on the device."""
        b = Rows(T=B, nd=B, ids=self.bt_next, slot=self.bt_slot,
                 pos=self.bt_lens, seg_row0=self._iota, seg_len=self._ones,
                 seg_slot=self.bt_slot, seg_pos0=self.bt_lens)
        x, xb = self.x, self.xb
        self._layer_stack(b)
        self._head(self.bt_logits32, B)
        self.x, self.xb = x, xb      # a captured step ends where it began
        ho.sample(self.bt_logits32[:B] if B > 1 else self.b_logits, min_p,
                  greedy, self.seed, self.rng_ctr, self.bt_gmax,
                  self.bt_pick, self.bt_next, self.bt_ring, self.bt_nout,
                  self.bt_lens, bump_len=True, temperature=temperature,
                  cnt=self.bt_cnt, batch=B)

    def prefill_batch(self, prompts) -> None:
        """Prefill B prompts (ragged lengths) as one mixed step."""
        seqs = [np.asarray(p, dtype=np.int32).ravel() for p in prompts]
        B = len(seqs)
        assert 1 <= B <= self.max_batch
        lens = [len(s) for s in seqs]
        if min(lens) == 0:
            raise ValueError("empty prompt in batch")
        if max(lens) + 1 >= self.max_seq:
            raise ValueError(f"prompt {max(lens)} fills the "
                             f"{self.max_seq} pool")
        self.reset()
        rows = [self._open_row(b) for b in range(B)]
        with trace_range(f"prefill_batch[{B}]"):
            out = self.step([StepEntry(q, s, [len(s) - 1])
                             for q, s in zip(rows, seqs)])
        self.bt_logits32[:B].copy_(out)
        self.bt_lens[:B].copy_(torch.tensor(lens, dtype=torch.int32))
        self._host_lens = lens + [0] * (self.max_batch - B)
        self._batch_n = B

    def prefill_row(self, b: int, ids, greedy: bool = True,
                    min_p: float = 0.1, temperature: float = 1.0):
        """Prefill one sequence into row b and sample its first token (a
        request joining the group between decode chunks)."""
        ids = np.asarray(ids, dtype=np.int32).ravel()
        P = len(ids)
        if P == 0:
            raise ValueError("empty prompt")
        assert 0 <= b < self.max_batch
        if P + 1 >= self.max_seq:
            raise ValueError(f"prompt {P} fills the {self.max_seq} pool")
        logits = self.step([StepEntry(self._open_row(b), ids, [P - 1])])
        self.bt_lens[b:b + 1].fill_(P)
        self.bt_nout[b:b + 1].zero_()
        ho.sample(logits[0], min_p, greedy, self.seed, self.rng_ctr,
                  self.bt_gmax[b:b + 1], self.bt_pick[b:b + 1],
                  self.bt_next[b:b + 1], self.bt_ring[b:b + 1],
                  self.bt_nout[b:b + 1], self.bt_lens[b:b + 1],
                  bump_len=False, temperature=temperature,
                  cnt=self.bt_cnt[b:b + 1], batch=1)
        self._host_lens[b] = P
        self._batch_n = max(self._batch_n, b + 1)

    def compact_row(self, dst: int, src: int):
        """Row dst is finished: its pages and slot are freed and row src
        takes its place (no cache data moves)."""
        if self.rows[dst] is not None:
            self.cache.close(self.rows[dst])
            self.rows[dst] = None
        if dst == src:
            return
        self.rows[dst], self.rows[src] = self.rows[src], None
        for t in (self.bt_slot, self.bt_lens, self.bt_next, self.bt_nout,
                  self.bt_gmax, self.bt_pick, self.bt_cnt):
            t[dst:dst + 1].copy_(t[src:src + 1])
        self.bt_ring[dst].copy_(self.bt_ring[src])
        self._host_lens[dst] = self._host_lens[src]
