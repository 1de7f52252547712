"""What every decoder of the framework shares on the generation path: the parts of the reference's
decoder interface that do not depend on the layers (metaseq/models/base_decoder.py:82-100), and
the slot interface of the serving loop on top of three operations a decoder provides -
``prefill_slot`` / ``prefill_slots`` and ``decode_slots``."""
import ctypes
from typing import Optional

import torch
from torch import nn

from . import _capi
from ._capi import check, ptr


def upload(values, dtype, device):
    """A short host list as a device tensor without a blocking copy: through pinned memory and
    stream-ordered.  (A copy from pageable memory makes the host wait for everything queued
    ahead of it - a whole decode step - and leaves the GPU idle while the host goes on.)"""
    t = torch.tensor(values, dtype=dtype)
    if torch.device(device).type != "cuda":
        return t.to(device)
    return t.pin_memory().to(device, non_blocking=True)


class IncrementalDecoder(nn.Module):
    """Base class.  A subclass sets ``_state_key`` (the key of its cache in a caller's
    incremental state) and implements ``prepare_`` (returning the library that selects tokens),
    ``prefill_slot``, ``prefill_slots`` and ``decode_slots``."""

    def make_generation_fast_(self, **unused):
        self.inference = True

    def reorder_incremental_state(self, incremental_state, new_order):
        """No-op, as in the reference (metaseq/models/base_decoder.py:82-93)."""

    def get_normalized_probs(self, logits, log_probs: bool):
        """metaseq/models/base_decoder.py:95-100 (fp32 softmax over the last dimension)."""
        if isinstance(logits, (tuple, list)):
            logits = logits[0]
        if log_probs:
            return torch.log_softmax(logits, dim=-1, dtype=torch.float32)
        return torch.softmax(logits, dim=-1, dtype=torch.float32)

    def get_cache(self, incremental_state):
        if not incremental_state:
            return None
        return incremental_state.get(self._state_key)

    # ------------------------------------------------------------------ slot interface
    # admit_slot / admit_slots take ``lazy=True``: the prompt scores come back as device tensors
    # (None for a one-token prompt) for the caller to read together with everything else
    lazy_admission = True

    def admit_slots(self, cache, requests, lazy=False):
        """``admit_slot`` for several requests with one shared prefill (``prefill_slots``).
        ``requests``: dicts with ``slot``, ``tokens`` and the keyword arguments of
        ``admit_slot``; returns the list of their prompt scores (``lazy``: as fp32 device
        tensors without the leading 0.0, nothing read back yet)."""
        logits = self.prefill_slots(cache, [r["slot"] for r in requests],
                                    [r["tokens"] for r in requests])
        out = []
        for r, lg in zip(requests, logits):
            kw = {k: v for k, v in r.items() if k not in ("slot", "tokens")}
            out.append(self.admit_slot(cache, r["slot"], r["tokens"], _logits=lg, _lazy=True,
                                       **kw))
        if lazy:
            return out
        # every request's kernels are queued: one copy for all the scores
        flat = torch.cat([lp for lp in out if lp is not None]).tolist() if any(
            lp is not None for lp in out) else []
        scores, at = [], 0
        for lp in out:
            n = lp.numel() if lp is not None else 0
            scores.append([0.0] + flat[at:at + n])
            at += n
        return scores

    def admit_slot(self, cache, slot: int, tokens: torch.Tensor, *, banned=(), stop=(),
                   eos=2, mode=0, tok_out=None, score_out=None, temperature=1.0, topp=0.0,
                   noise=None, replicas=(), penalties=None, lprobs_out=None, prompt_topk=0,
                   detail=None, lazy=False, _logits=None, _lazy=False):
        """``prefill_slot`` plus what a request needs from its prompt: the log-probability of
        every prompt token given its prefix (returned as a list, 0.0 for the first token) and
        the choice of the first new token from the last position, written to ``tok_out`` /
        ``score_out`` (int64 / fp32 device tensors, one element per replica) under the selection
        regime ``mode`` (MSA_ROW_* bits).

        With the defaults the choice is greedy on the unscaled logits.  ``temperature`` scales
        the logits (prompt scores included, as the reference's loop does); ``topp`` > 0 with
        ``noise`` (fp32 [1 + len(replicas), V], independent Exp(1) numbers) draws from the
        nucleus.  ``replicas``: further slots that receive a copy of the prompt's keys and values
        and make their own choice (row r of ``noise``, element r of the outputs).

        ``penalties``: dict with ``alphas`` (presence, frequency, presence_src, frequency_src),
        ``counts`` (int64 [R, V], updated with the chosen tokens) and ``counts_src`` (int64
        [R, V] prompt-token counts), R = 1 + len(replicas): the reference's repetition penalties
        on the first choice.  ``lprobs_out`` (fp32 [R, V]) receives the masked, penalised
        log-probabilities the choice was made from.  ``prompt_topk`` > 0 with a dict ``detail``:
        ``detail["prompt_top"]`` = (values, ids), CPU tensors [T - 1, k], the k most likely
        tokens at every prompt position after the first (log-softmax of logits / temperature,
        what the reference records for the prompt with ``need_logprobs``)."""
        lib = self.prepare_()
        _lazy = _lazy or lazy
        # (_logits: the prompt was already prefilled into the slot, by prefill_slots)
        logits = _logits if _logits is not None else self.prefill_slot(cache, slot, tokens)
        T, V = logits.shape
        stream = _capi.stream_ptr()
        scores, lp = [0.0] * T, None
        if T > 1:
            lp = torch.empty(T - 1, dtype=torch.float32, device=logits.device)
            target = tokens.long()[1:].contiguous()
            check(_capi.for_logits(lib, "msa_target_logprob", logits)(
                ptr(logits), logits.stride(0), T - 1, V, float(temperature), ptr(target), ptr(lp),
                stream))
            if not _lazy:   # (_lazy: the caller reads the device tensor once all is queued)
                scores[1:] = lp.tolist()
            if prompt_topk > 0 and detail is not None:
                dist = torch.empty(T - 1, V, dtype=torch.float32, device=logits.device)
                check(_capi.for_logits(lib, "msa_log_softmax", logits)(
                    ptr(logits), 0, logits.stride(0), 1, T - 1, V, float(temperature), ptr(dist),
                    0, V, stream))
                values, ids = dist.topk(min(int(prompt_topk), V), dim=-1)
                detail["prompt_top"] = (values.cpu(), ids.cpu())
                del dist
        for dst in replicas:
            self.copy_slot(cache, slot, dst, length=T)
        R = 1 + len(replicas)
        plain = (float(temperature) == 1.0 and not topp > 0 and noise is None
                 and penalties is None and lprobs_out is None)
        banned, stop = list(banned), list(stop)
        ba = (ctypes.c_int32 * max(1, len(banned)))(*banned)
        sa = (ctypes.c_int32 * max(1, len(stop)))(*stop)
        row_mode = torch.full((R,), mode, dtype=torch.uint8, device=logits.device)
        last = logits[T - 1:T]
        if R > 1:  # every replica reads its own copy of the row (a few hundred KB)
            last = last.expand(R, V).contiguous()
        if plain:
            check(_capi.for_logits(lib, "msa_greedy_select", logits)(
                ptr(last), last.stride(0), R, V, 1.0, ba, len(banned), sa, len(stop), None,
                ptr(row_mode), 0, int(eos), ptr(tok_out), 1, ptr(score_out), 1, None, stream))
        else:
            pen = penalties or {}
            alphas = [float(a) for a in pen.get("alphas", (0.0, 0.0, 0.0, 0.0))]
            for name in ("counts", "counts_src"):
                t = pen.get(name)
                if t is not None and (t.shape != (R, V) or t.dtype != torch.long
                                      or not t.is_contiguous()):
                    raise AssertionError("%s must be contiguous int64 [%d, %d]" % (name, R, V))
            if lprobs_out is not None and (lprobs_out.shape != (R, V)
                                           or lprobs_out.dtype != torch.float32
                                           or lprobs_out.stride(1) != 1):
                raise AssertionError("lprobs_out must be fp32 [%d, %d]" % (R, V))
            check(_capi.for_logits(lib, "msa_sample_topp", logits)(
                ptr(last), last.stride(0), R, V, float(temperature), None, ba, len(banned), sa,
                len(stop), None, ptr(row_mode), 0, int(eos), None, float(topp), ptr(noise),
                ptr(pen.get("counts")), ptr(pen.get("counts_src")), alphas[0], alphas[1],
                alphas[2], alphas[3], None, ptr(lprobs_out), lprobs_out.stride(0) if lprobs_out is
                not None else 0, ptr(tok_out), 1, ptr(score_out), 1, stream))
        return lp if _lazy else scores

    def copy_slot(self, cache, src: int, dst: int, length: Optional[int] = None):
        """Makes slot ``dst`` a copy of slot ``src``: keys, values and length (a replica of a
        request starts from the same prompt).  ``length``: the source's length where the caller
        knows it (reading it from the device waits for everything queued)."""
        n = int(cache.lens[src]) if length is None else int(length)
        cache.copy_row(src, dst, n)
        cache.lens[dst:dst + 1].fill_(n)

    def release_slot(self, cache, slot: int):
        # a fill kernel on a one-element view: ``lens[slot] = -1`` copies a host scalar to the
        # device and makes the caller wait for the work queued ahead of it
        cache.lens[slot:slot + 1].fill_(-1)

    def _sample_rows(self, lib, logits, sampled, banned, stop, finished, eos, tok_out, score_out):
        """Chooses the rows of ``sampled`` (see ``decode_slots``) from the step's logits and
        overwrites their outputs."""
        stream = _capi.stream_ptr()
        B, V = logits.shape
        banned, stop = list(banned), list(stop)
        ba = (ctypes.c_int32 * max(1, len(banned)))(*banned)
        sa = (ctypes.c_int32 * max(1, len(stop)))(*stop)
        lp = sampled.get("lprobs_out")
        for name, dtype in (("counts", torch.long), ("counts_src", torch.long),
                            ("lprobs_out", torch.float32)):
            t = sampled.get(name)
            if t is not None and (t.shape != (B, V) or t.dtype != dtype
                                  or not t.is_contiguous()):
                raise AssertionError("%s must be contiguous [%d, %d]" % (name, B, V))
        pr = sampled.get("penalty_rows")
        if pr is not None and (pr.shape != (B, 4) or pr.dtype != torch.float32
                               or not pr.is_contiguous()):
            raise AssertionError("penalty_rows must be contiguous fp32 [%d, 4]" % B)
        check(_capi.for_logits(lib, "msa_sample_topp", logits)(
            ptr(logits), logits.stride(0), B, V, 1.0, ptr(sampled["temperature"]), ba,
            len(banned), sa, len(stop), ptr(finished), ptr(sampled["row_mode"]), 0, int(eos),
            ptr(sampled["topp"]), 0.0, ptr(sampled.get("noise")),
            ptr(sampled.get("counts")) if pr is not None else None,
            ptr(sampled.get("counts_src")) if pr is not None else None, 0.0, 0.0, 0.0, 0.0,
            ptr(pr), ptr(lp), V if lp is not None else 0, ptr(tok_out), 1, ptr(score_out), 1,
            stream))
