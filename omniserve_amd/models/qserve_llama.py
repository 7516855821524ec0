"""The QServe W4A8KV4 Llama on the engine: weights of a QServe checkpoint (ckpt.load_into_runner), the decoder layer as
runtime.DecodeRunner.prefill wires it (llama_w4a8_unpad.py:406-438), KV4 pages from the engine's cache.

Whole prompts run through the prefill writer and the varlen attention over the step's own keys; single tokens, and later portions of
a prompt token by token, through the paged KV4 decode attention.  Steps run eagerly (the captured fast path of a fixed batch is
runtime.DecodeRunner)."""
from __future__ import annotations

import torch

from .. import ckpt
from ..backend import fused_attention_fine_grained_dense as fgd
from ..backend import fused_attention_pure_dense, fused_ext, fused_kernels, layernorm_ops
from ..backend.prefill_attn import flash_attn_varlen_func
from ..runtime import DecodeRunner, LlamaConfig
from .base import EngineModel


def parse_config(c: dict) -> LlamaConfig:
    heads = c["num_attention_heads"]
    return LlamaConfig(hidden=c["hidden_size"], inter=c["intermediate_size"], heads=heads, kv_heads=c.get("num_key_value_heads", heads),
                       head_dim=c.get("head_dim", c["hidden_size"] // heads), layers=c["num_hidden_layers"], vocab=c["vocab_size"],
                       rope_theta=float(c.get("rope_theta", 10000.0)), eps=float(c.get("rms_norm_eps", 1e-5)),
                       group_size=c.get("quantization", {}).get("group_size", -1))


class QServeLlama(EngineModel):
    dtypes = (torch.float16,)
    capturable = False

    def __init__(self, cfg: LlamaConfig, state: dict, device):
        self.cfg, self.device, self.dtype, self.vocab = cfg, torch.device(device), torch.float16, cfg.vocab
        holder = DecodeRunner(cfg, batch=1, context=1, max_new=1, device=self.device, use_graph=False, fused=False)
        ckpt.load_into_runner(holder, state)
        self.layers, self.embed, self.lm_head, self.final_norm = holder.layers, holder.embed, holder.lm_head, holder.final_norm
        self.page_bytes = holder.page_bytes
        self.flags = torch.ones((cfg.kv_heads,), dtype=torch.int32, device=self.device)
        self.rank = torch.arange(cfg.kv_heads, dtype=torch.int32, device=self.device)

    @classmethod
    def from_pretrained(cls, model_dir, config, dtype=None, device="cuda"):
        if dtype not in (None, *cls.dtypes):
            raise ValueError("the W4A8KV4 path runs in float16")
        return cls(parse_config(config), ckpt.load_state_dict(model_dir), device)

    def kv_shapes(self):
        return [(self.cfg.kv_heads, self.cfg.head_dim, self.cfg.head_dim)] * self.cfg.layers

    def page_pools(self, num_pages, device):
        pool = lambda: torch.zeros((num_pages, self.page_bytes), dtype=torch.uint8, device=device)      # noqa: E731
        return [(pool(), pool()) for _ in range(self.cfg.layers)]

    def _layers(self, tokens, attention):
        """The decoder stack on token ids; attention(layer, q, k, v, qkv) -> [T, heads * head_dim].  Returns the residual."""
        c, T, dev = self.cfg, tokens.numel(), self.device
        hq, hk, d, per_chn = c.heads, c.kv_heads, c.head_dim, c.group_size == -1
        f16 = lambda *s: torch.empty(s, dtype=torch.float16, device=dev)      # noqa: E731
        i8 = lambda *s: torch.empty(s, dtype=torch.int8, device=dev)          # noqa: E731
        x, qh, qi, qa = f16(T, c.hidden), i8(T, c.hidden), i8(T, c.inter), i8(T, hq * d)
        qkv, proj, gu = f16(T, (hq + 2 * hk) * d), f16(T, c.hidden), f16(T, 2 * c.inter)
        sn, sa = f16(T), f16(T)
        mn, ma = (f16(T), f16(T)) if per_chn else (None, None)               # g128: no activation sums
        torch.index_select(self.embed, 0, tokens.long(), out=x)
        q, k, v = (qkv[:, a * d:b * d].view(T, b - a, d) for a, b in ((0, hq), (hq, hq + hk), (hq + hk, hq + 2 * hk)))
        for li, L in enumerate(self.layers):
            if li:
                fused_ext.add_rms_norm_general_fuse_sum(qh, x, proj, L["ln1"], mn, sn, c.eps)
            elif per_chn:
                layernorm_ops.rms_norm_general_fuse_sum(qh, x, L["ln1"], mn, sn, c.eps, True)
            else:
                layernorm_ops.rms_norm_general(qh, x, L["ln1"], sn, c.eps, True)
            L["qkv"].forward(qh, sn, mn, qkv)
            o = attention(li, q, k, v, qkv)
            if per_chn:
                fused_kernels.invoke_quant_fuse_sum(qa, o, ma, sa)
            else:
                fused_kernels.invoke_quant(qa, o, sa)
            L["o"].forward(qa, sa, ma, proj)
            fused_ext.add_rms_norm_general_fuse_sum(qh, x, proj, L["ln2"], mn, sn, c.eps)
            L["gate_up"].forward(qh, sn, mn, gu)
            fused_ext.silu_mul_quant_fuse_sum(qi, gu, ma, sa)
            L["down"].forward(qi, sa, ma, proj)
        return x.add_(proj)

    def _pointers(self, table, kv):
        """int64 page addresses [B, 2, blocks] of one layer's pools"""
        t = table.long() * self.page_bytes
        return torch.stack((t + kv[0].data_ptr(), t + kv[1].data_ptr()), dim=1).contiguous()

    def _prompts(self, tokens, lengths, table, cache):
        c, T, L, dev = self.cfg, sum(lengths), max(lengths), self.device
        lens = torch.tensor(lengths, dtype=torch.int32, device=dev)
        cu = torch.zeros((len(lengths) + 1,), dtype=torch.int32, device=dev)
        cu[1:] = torch.cumsum(lens, 0)
        pad = fgd.compute_padding_offsets(cu, L, T)

        def attention(li, q, k, v, qkv):
            fgd.apply_bias_rope_update_kv_cache(qkv, lens, None, pad, self._pointers(table, cache.kv[li]), None, self.flags, self.rank,
                                                c.heads, c.kv_heads, L, self.page_size, c.kv_heads * c.head_dim // 2, 0, 0, 0, 0, 0,
                                                c.kv_heads, 0, c.head_dim, c.rope_theta, 1.0, 1 << 20, True, True, True)
            return flash_attn_varlen_func(q, k, v, cu, cu, L, L, causal=True).view(T, -1)

        return self._layers(tokens, attention)

    def _single(self, tokens, pos, table, cache, max_context):
        c = self.cfg
        lengths = (pos + 1).contiguous()

        def attention(li, q, k, v, qkv):
            return fused_attention_pure_dense.single_query_attention(
                q, k, v, self._pointers(table, cache.kv[li]), lengths, None, 65536, self.page_size, c.kv_heads * c.head_dim // 2,
                max_context, c.head_dim, c.rope_theta, True, True, True).view(tokens.numel(), -1)

        return self._layers(tokens, attention)

    def forward(self, b, cache):
        c, n = self.cfg, b.n_prompt
        x = torch.empty((b.tokens.numel(), c.hidden), dtype=torch.float16, device=self.device)
        entries = b.entry.tolist()
        single = b.pos[n:].tolist()
        first = [(at, m, row) for at, m, pos, row in entries if pos == 0]
        first += [(n + i, 1, b.n_entries + i) for i, p in enumerate(single) if p == 0]      # (a prompt of one token)
        if first:
            rows = torch.cat([torch.arange(at, at + m) for at, m, _ in first]).to(self.device)
            x[rows] = self._prompts(b.tokens[rows], [m for _, m, _ in first], b.block_table[[r for _, _, r in first]], cache)
        for at, m, pos, row in entries:
            for i in range(at, at + m if pos else at):       # a later portion: its tokens one by one
                x[i:i + 1] = self._single(b.tokens[i:i + 1], b.pos[i:i + 1], b.block_table[row:row + 1], cache, pos + i - at + 1)
        at = [n + i for i, p in enumerate(single) if p > 0]
        if at:
            x[at] = self._single(b.tokens[at], b.pos[at], b.block_table[[b.n_entries + i - n for i in at]], cache, b.max_context)
        if not b.rows.numel():
            return None
        h = x[b.rows.long()]
        normed = torch.empty_like(h)
        layernorm_ops.rms_norm(normed, h, self.final_norm, c.eps, False)
        return torch.matmul(normed, self.lm_head.t()).float()
