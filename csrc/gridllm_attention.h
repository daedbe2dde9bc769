// Attention kernel templates, shared by the contiguous slot cache and the
// paged cache: where a block of keys lies comes from a KV policy.
#pragma once

#include "gridllm_common.h"

#define LOG2E 1.4426950408889634f

// Where 64 keys (aligned to 64) of a sequence's kv head start, in elements.
// Caches of contiguous slots: [slots, Hk, Smax, D].
template <int D>
struct SlotKV {
    const bf16_t* k;
    const bf16_t* v;
    int Hk, Smax;
    DEV_INLINE long off(int slot, int hk, int key) const {
        return (((long)slot * Hk + hk) * Smax + key) * D;
    }
};

// Caches of pages of 64 keys: [pages, Hk, 64, D]; table[slot][i] is the page
// of keys 64 i .. 64 i + 63.
#define KV_PAGE 64
template <int D>
struct PagedKV {
    const bf16_t* k;
    const bf16_t* v;
    const int* table;
    int Hk, per_slot;
    DEV_INLINE long off(int slot, int hk, int key) const {
        const int page = table[(long)slot * per_slot + (key / KV_PAGE)];
        return (((long)page * Hk + hk) * KV_PAGE + key % KV_PAGE) * D;
    }
};

// Which keys up to its own a query sees. Kernels walk blocks of keys by number
// (decode) or by first key (prefill) and leave out what no row sees.
struct AllKeys {
    DEV_INLINE int blocks(int seq) const { return (seq + 63) >> 6; }
    DEV_INLINE int start(int b, int seq) const { return b << 6; }
    DEV_INLINE int skip(int k0, int q0) const { return k0; }
    DEV_INLINE bool sees(int q, int key) const { return true; }
};

// The last `size` keys, its own included, and the first `keep`.
struct WindowKeys {
    int size, keep;
    // blocks of 64 that hold kept keys, and the first one of the window behind
    // them, for the last of seq positions
    DEV_INLINE int kept(int seq) const { return (min(keep, seq) + 63) >> 6; }
    DEV_INLINE int window(int seq) const {
        return max(kept(seq), max(0, seq - size) >> 6);
    }
    DEV_INLINE int blocks(int seq) const {
        return kept(seq) + ((seq + 63) >> 6) - window(seq);
    }
    DEV_INLINE int start(int b, int seq) const {
        const int k = kept(seq);
        return (b < k ? b : window(seq) + b - k) << 6;
    }
    // first key, from k0 on, of a tile of 32 that rows from q0 on may see
    DEV_INLINE int skip(int k0, int q0) const {
        return k0 < keep ? k0 : max(k0, max(0, q0 - size + 1) & ~31);
    }
    DEV_INLINE bool sees(int q, int key) const {
        return q - key < size || key < keep;
    }
};

// What happens to a head's sums before they are stored. `sink` (nullable, one
// per query head) adds exp(sink) to the softmax denominator; `gate` (nullable,
// row stride gate_ld) multiplies the output by its sigmoid: one per query
// head, or (gate_el) one per element; so does `scale`. out_ld: row stride of
// the output, 0 if the heads fill a row.
struct HeadEpilogue {
    const float* sink;
    const bf16_t* gate;
    int gate_ld;
    int gate_el = 0;
    float scale = 1.f;
    int out_ld = 0;
    DEV_INLINE long at(long row, int head, int Hq, int D) const {
        return row * (out_ld ? out_ld : Hq * D) + head * D;
    }
    DEV_INLINE float element(int row, int col) const {
        if (!gate_el) return 1.f;
        return 1.f / (1.f + __expf(-bf2f(gate[(long)row * gate_ld + col])));
    }
    // M, L: running maximum and sum of the log2-domain softmax. Returns the
    // factor for the accumulated values.
    DEV_INLINE float factor(int row, int head, float M, float L) const {
        float f = 1.f;
        if (sink) {
            const float s2 = sink[head] * LOG2E;
            const float m2 = fmaxf(M, s2);
            f = (M == -INFINITY) ? 0.f : exp2f(M - m2);
            L = L * f + exp2f(s2 - m2);
        }
        f = L > 0.f ? f / L * scale : 0.f;
        if (gate && !gate_el)
            f /= 1.f + __expf(-bf2f(gate[(long)row * gate_ld + head]));
        return f;
    }
};

// ===========================================================================
// GQA decode attention (flash-decode style).
//   q:   [B, Hq, D] bf16 (one new token per sequence)
//   kc/vc: [B, Hk, Smax, D] bf16
//   seqlen: [B] int32 (number of valid keys, including the current token)
//   out: [B, Hq, D] bf16
//   ws (nsplit>1): f32 [B, Hk, G, nsplit, D+2]  (unnormalized acc, m, l)
//
// Block = 256 thr = 4 waves, one block per (b, hk, split). Each wave owns
// key-blocks of 64 (one key per lane), keeps per-(g) online-softmax state,
// then the 4 waves combine in LDS. G = Hq/Hk (q-heads per kv-head) so each
// K/V row is read once and reused for all G query heads.
// Constraints: D in {64, 128}; G <= 8; D % 8 == 0.
// ===========================================================================

#define MAXG 8

// A kv head with more than MAXG query heads is served by `ngrp` blocks of G
// query heads each. Sequence lengths are given as seqlen + seq_add.
template <int D, int G, class KV, class Keys>
__global__ void __launch_bounds__(256, 3)
k_attn_decode(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
              const KV kv,
              const int* __restrict__ seqlen, int seq_add,
              const int* __restrict__ slot_map,
              float* __restrict__ ws,
              int ngrp, int nsplit, float scale, const HeadEpilogue epi,
              const Keys keys) {
    const int Hg = kv.Hk * ngrp;
    const int split = blockIdx.x % nsplit;
    const int hg = (blockIdx.x / nsplit) % Hg;
    const int hk = hg / ngrp;
    const int b = blockIdx.x / (nsplit * Hg);
    const int bc = slot_map ? slot_map[b] : b;   // cache slot for this row
    const int lane = threadIdx.x & 63;
    const int wid = threadIdx.x >> 6;

    __shared__ float q_lds[G * D];
    __shared__ float red[4][G * (D > 64 ? D : 64)];
    __shared__ float wml[4][G][2];            // per-wave m, l

    const int seq = seqlen[b] + seq_add;
    // split range, 64-aligned chunks
    const int chunks = keys.blocks(seq);
    const int per = (chunks + nsplit - 1) / nsplit;
    const int c0 = split * per;
    const int c1 = min(chunks, c0 + per);

    // stage q (scaled) into LDS as f32
    const int Hq = Hg * G;
    for (int i = threadIdx.x; i < G * D; i += 256) {
        int g = i / D, d = i % D;
        // log2-domain softmax: fold log2(e) into the q prescale so every
        // exp becomes a native v_exp_f32 exp2 (identical values:
        // exp2((x-m)*log2e) == exp(x-m))
        q_lds[i] = bf2f(q[((long)b * Hq + hg * (long)G + g) * D + d])
                   * (scale * 1.4426950408889634f);
    }
    __syncthreads();

    // per-wave online softmax state.
    // P.V layout: the wave reads RPI = 64/(D/8) V-rows per b128-load
    // iteration — lane covers row-group rg = lane/DV and d = (lane%DV)*8
    // + 0..7 — so a 64-key block takes 64/RPI wide-load iterations instead
    // of 64 row-at-a-time u32 iterations (which measured as a serial
    // L2-latency chain, 3.2 TB/s). Each lane holds PARTIAL sums over its
    // row group; one shfl_xor ladder at the end totals them.
    float m[G], l[G];
    constexpr int DV = D / 8;          // lanes per V row
    constexpr int RPI = 64 / DV;       // V rows per iteration
    float facc[G][8];
#pragma unroll
    for (int g = 0; g < G; ++g) {
        m[g] = -INFINITY;
        l[g] = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) facc[g][i] = 0.f;
    }
    const int rg = lane / DV;
    const int d8 = (lane % DV) * 8;

    int cb = c0 + wid;
    long next = cb < c1 ? kv.off(bc, hk, keys.start(cb, seq)) : 0;
    for (; cb < c1; cb += 4) {
        const int kb = keys.start(cb, seq);
        const bf16_t* kblk = kv.k + next;
        const bf16_t* vblk = kv.v + next;
        if (cb + 4 < c1) next = kv.off(bc, hk, keys.start(cb + 4, seq));
        const int j = kb + lane;
        const bool valid = j < seq && keys.sees(seq - 1, j);
        float s[G];
#pragma unroll
        for (int g = 0; g < G; ++g) s[g] = 0.f;
        if (valid) {
            const bf16_t* krow = kblk + lane * D;
#pragma unroll
            for (int dd = 0; dd < D; dd += 8) {
                uint4 kv = *(const uint4*)(krow + dd);
                float kf[8];
                unpack8(kv, kf);
#pragma unroll
                for (int g = 0; g < G; ++g) {
                    float a = 0.f;
#pragma unroll
                    for (int i = 0; i < 8; ++i) a += kf[i] * q_lds[g * D + dd + i];
                    s[g] += a;
                }
            }
        }
        // online softmax update per g; store p into LDS (reuse red[] rows)
#pragma unroll
        for (int g = 0; g < G; ++g) {
            float sv = valid ? s[g] : -INFINITY;
            float bmax = wave_reduce_max(sv);
            float mn = fmaxf(m[g], bmax);
            // guard: all-invalid block -> bmax=-inf, mn may stay -inf
            float alpha = (m[g] == -INFINITY) ? 0.f : exp2f(m[g] - mn);
            float p = (sv == -INFINITY) ? 0.f : exp2f(sv - mn);
            l[g] = l[g] * alpha + wave_reduce_sum(p);
            if (mn != m[g]) {          // defer-rescale: skip when max held
#pragma unroll
                for (int i = 0; i < 8; ++i) facc[g][i] *= alpha;
            }
            m[g] = mn;
            red[wid][g * 64 + lane] = p;      // per-wave scratch: p for 64 keys
        }
        // wave-local LDS visibility (no cross-wave traffic here)
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        // accumulate P·V: RPI rows per iteration, one b128 load per lane
        const int jmax = min(64, seq - kb);
        for (int jb = 0; jb < jmax; jb += RPI) {
            const int j2 = jb + rg;
            const uint4 vv = *(const uint4*)(
                vblk + min(j2, jmax - 1) * D + d8);
            float vf[8];
            unpack8(vv, vf);
#pragma unroll
            for (int g = 0; g < G; ++g) {
                const float p = (j2 < jmax) ? red[wid][g * 64 + j2] : 0.f;
#pragma unroll
                for (int i = 0; i < 8; ++i)
                    facc[g][i] = fmaf(p, vf[i], facc[g][i]);
            }
        }
    }

    // total each lane's row-group partials: after the ladder every lane
    // holds the full sum for its d = d8 + 0..7 slice
#pragma unroll
    for (int g = 0; g < G; ++g)
#pragma unroll
        for (int i = 0; i < 8; ++i)
#pragma unroll
            for (int off = 32; off >= DV; off >>= 1)
                facc[g][i] += __shfl_xor(facc[g][i], off, WAVE);

    // cross-wave combine in LDS
#pragma unroll
    for (int g = 0; g < G; ++g) {
        wml[wid][g][0] = m[g];
        wml[wid][g][1] = l[g];
    }
    __syncthreads();
#pragma unroll
    for (int g = 0; g < G; ++g) {
        float M = fmaxf(fmaxf(wml[0][g][0], wml[1][g][0]),
                        fmaxf(wml[2][g][0], wml[3][g][0]));
        float f = (m[g] == -INFINITY) ? 0.f : exp2f(m[g] - M);
        if (lane < DV)
#pragma unroll
            for (int i = 0; i < 8; ++i)
                red[wid][g * D + d8 + i] = facc[g][i] * f;
        if (lane == g % 64) wml[wid][g][1] = l[g] * f;  // scaled l (one lane writes)
    }
    __syncthreads();

    // final reduction over 4 waves + output
    for (int i = threadIdx.x; i < G * D; i += 256) {
        const int g = i / D, d = i % D;
        float a = red[0][g * D + d] + red[1][g * D + d] +
                  red[2][g * D + d] + red[3][g * D + d];
        float L = wml[0][g][1] + wml[1][g][1] + wml[2][g][1] + wml[3][g][1];
        float M = fmaxf(fmaxf(wml[0][g][0], wml[1][g][0]),
                        fmaxf(wml[2][g][0], wml[3][g][0]));
        if (nsplit == 1) {
            out[epi.at(b, hg * G + g, Hq, D) + d] =
                f2bf(a * epi.factor(b, hg * G + g, M, L) *
                     epi.element(b, (hg * G + g) * D + d));
        } else {
            float* wsp = ws + (((long)b * Hq + hg * G + g) * nsplit + split) * (D + 2);
            wsp[d] = a;
            if (d == 0) {
                wsp[D] = M;
                wsp[D + 1] = L;
            }
        }
    }
}

// ===========================================================================
// GQA decode attention, ONE WAVE per (b, hk[, split]) — the large-batch
// variant. At serving batches B*Hk >= ~2048 the chip holds every block
// resident (16 waves/CU), so per-wave independence beats the 4-wave
// cooperative block: no q-staging barrier, no cross-wave LDS combine, no
// idle waves when seq/64 < 4. Same math as k_attn_decode; V phase reads
// RPI rows per b128 iteration with an end shfl ladder.
// ===========================================================================

template <int D, int G, class KV, class Keys>
__global__ void __launch_bounds__(64, 3)
k_attn_decode1(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
               const KV kv,
               const int* __restrict__ seqlen, int seq_add,
               const int* __restrict__ slot_map,
               float* __restrict__ ws,
               int ngrp, int nsplit, float scale, const HeadEpilogue epi,
               const Keys keys) {
    const int Hg = kv.Hk * ngrp;
    const int split = blockIdx.x % nsplit;
    const int hg = (blockIdx.x / nsplit) % Hg;
    const int hk = hg / ngrp;
    const int b = blockIdx.x / (nsplit * Hg);
    const int bc = slot_map ? slot_map[b] : b;
    const int lane = threadIdx.x;

    __shared__ float q_lds[G * D];
    __shared__ float p_lds[G * 64];

    const int seq = seqlen[b] + seq_add;
    const int chunks = keys.blocks(seq);
    const int per = (chunks + nsplit - 1) / nsplit;
    const int c0 = split * per;
    const int c1 = min(chunks, c0 + per);

    const int Hq = Hg * G;
    for (int i = lane; i < G * D; i += 64)
        q_lds[i] = bf2f(q[((long)b * Hq + hg * (long)G + i / D) * D
                          + i % D]) * (scale * 1.4426950408889634f);
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");

    float m[G], l[G];
    constexpr int DV = D / 8;
    constexpr int RPI = 64 / DV;
    float facc[G][8];
#pragma unroll
    for (int g = 0; g < G; ++g) {
        m[g] = -INFINITY;
        l[g] = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) facc[g][i] = 0.f;
    }
    const int rg = lane / DV;
    const int d8 = (lane % DV) * 8;

    long next = c0 < c1 ? kv.off(bc, hk, keys.start(c0, seq)) : 0;
    for (int cb = c0; cb < c1; ++cb) {
        const int kb = keys.start(cb, seq);
        const bf16_t* kblk = kv.k + next;
        const bf16_t* vblk = kv.v + next;
        if (cb + 1 < c1) next = kv.off(bc, hk, keys.start(cb + 1, seq));
        const int j = kb + lane;
        const bool valid = j < seq && keys.sees(seq - 1, j);
        float s[G];
#pragma unroll
        for (int g = 0; g < G; ++g) s[g] = 0.f;
        if (valid) {
            const bf16_t* krow = kblk + lane * D;
#pragma unroll
            for (int dd = 0; dd < D; dd += 8) {
                uint4 kv = *(const uint4*)(krow + dd);
                float kf[8];
                unpack8(kv, kf);
#pragma unroll
                for (int g = 0; g < G; ++g) {
                    float a = 0.f;
#pragma unroll
                    for (int i = 0; i < 8; ++i)
                        a += kf[i] * q_lds[g * D + dd + i];
                    s[g] += a;
                }
            }
        }
#pragma unroll
        for (int g = 0; g < G; ++g) {
            float sv = valid ? s[g] : -INFINITY;
            float bmax = wave_reduce_max(sv);
            float mn = fmaxf(m[g], bmax);
            float alpha = (m[g] == -INFINITY) ? 0.f : exp2f(m[g] - mn);
            float p = (sv == -INFINITY) ? 0.f : exp2f(sv - mn);
            l[g] = l[g] * alpha + wave_reduce_sum(p);
            if (mn != m[g]) {          // defer-rescale: skip when max held
#pragma unroll
                for (int i = 0; i < 8; ++i) facc[g][i] *= alpha;
            }
            m[g] = mn;
            p_lds[g * 64 + lane] = p;
        }
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        // P.V: RPI rows per b128 iteration; p read from same-wave LDS
        // (an LDS hop, not shfl: it bounds how far the scheduler can
        // interleave the K and V phases — shfl spilled 1.5 KB here)
        const int jmax = min(64, seq - kb);
        for (int jb = 0; jb < jmax; jb += RPI) {
            const int j2 = jb + rg;
            const uint4 vv = *(const uint4*)(
                vblk + min(j2, jmax - 1) * D + d8);
            float vf[8];
            unpack8(vv, vf);
#pragma unroll
            for (int g = 0; g < G; ++g) {
                const float p = (j2 < jmax) ? p_lds[g * 64 + j2] : 0.f;
#pragma unroll
                for (int i = 0; i < 8; ++i)
                    facc[g][i] = fmaf(p, vf[i], facc[g][i]);
            }
        }
    }

#pragma unroll
    for (int g = 0; g < G; ++g)
#pragma unroll
        for (int i = 0; i < 8; ++i)
#pragma unroll
            for (int off = 32; off >= DV; off >>= 1)
                facc[g][i] += __shfl_xor(facc[g][i], off, WAVE);

    if (lane < DV) {
#pragma unroll
        for (int g = 0; g < G; ++g) {
            if (nsplit == 1) {
                const float f = epi.factor(b, hg * G + g, m[g], l[g]);
#pragma unroll
                for (int i = 0; i < 8; ++i)
                    out[epi.at(b, hg * G + g, Hq, D) + d8 + i] =
                        f2bf(facc[g][i] * f *
                             epi.element(b, (hg * G + g) * D + d8 + i));
            } else {
                float* wsp = ws + (((long)b * Hq + hg * G + g) * nsplit
                                   + split) * (D + 2);
#pragma unroll
                for (int i = 0; i < 8; ++i) wsp[d8 + i] = facc[g][i];
                if (lane == 0) {
                    wsp[D] = m[g];
                    wsp[D + 1] = l[g];
                }
            }
        }
    }
}

// Combine split-S partials: grid = B*Hq blocks, D threads.
__global__ void
k_attn_combine(bf16_t* __restrict__ out, const float* __restrict__ ws,
               int Hq, int D, int nsplit, const HeadEpilogue epi) {
    const long bh = blockIdx.x;               // b*Hq + hq
    const int d = threadIdx.x;
    const float* base = ws + bh * (long)nsplit * (D + 2);
    float M = -INFINITY;
    for (int s = 0; s < nsplit; ++s) M = fmaxf(M, base[s * (D + 2) + D]);
    float num = 0.f, den = 0.f;
    for (int s = 0; s < nsplit; ++s) {
        const float* p = base + s * (long)(D + 2);
        float ms = p[D];
        float f = (ms == -INFINITY) ? 0.f : exp2f(ms - M);
        num += f * p[d];
        den += f * p[D + 1];
    }
    const int b = (int)(bh / Hq), h = (int)(bh % Hq);
    out[epi.at(b, h, Hq, D) + d] =
        f2bf(num * epi.factor(b, h, M, den) * epi.element(b, h * D + d));
}
// ===========================================================================
// GQA prefill attention — flash-style on MFMA (bf16), reads K/V straight
// from the slot cache (no permuted host-side views).
//   q:   [T, Hq, D] bf16 (roped)
//   kc/vc: [slots, Hk, Smax, D] bf16
//   out: [T, Hq, D] bf16
// Workgroup = 4 waves; wave w owns 32 q-rows (q0 + w*32) of ONE q-head;
// K/V walked in 32-row tiles with online softmax (guide App. B prefill).
//
// Layout trick (guide §5.5 "swapped QK^T"): S^T = mfma(A=K, B=Q) puts a
// whole q-row's scores in ONE lane (C col = lane&31 = q), so the softmax
// row-reduce is 15 in-register fmax + one shfl_xor(32) — no LDS. P is then
// routed to the PV MFMA's B-operand layout through a per-wave LDS scratch
// (paired b32 writes -> b128 fragment reads, same-wave lgkmcnt wait only),
// and O^T = mfma(A=V^T, B=P) accumulates with V staged TRANSPOSED in LDS
// (transpose once per tile, cooperative; A-fragments then read b128-clean).
// mfma_f32_32x32x16_bf16 maps (guide §3):
//   A[i][k]: lane l holds i = l&31, k = (l>>5)*8 + 0..7
//   B[k][j]: lane l holds j = l&31, same k chunk
//   C/D[i][j]: col j = l&31, row i = (reg&3) + 8*(reg>>2) + 4*(l>>5)
// Constraints: D in {64, 128}; Hq % Hk == 0.
// ===========================================================================

// Shared body: one 128-q-row tile of one q-head for one sequence.
// q0 = first q row of this tile; vt/plds = caller's LDS buffers.
// row0 = row of q[0] in the epilogue's gate.
template <int D, class KV, class Keys = AllKeys>
__device__ __forceinline__ void
attn_prefill_tile(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
                  const KV& kv,
                  int T, int Hq, int G, int slot,
                  int s_total, int causal_off, float scale, int q0,
                  bf16_t* vt, bf16_t* plds_all, const HeadEpilogue& epi,
                  int row0, const Keys keys = Keys()) {
    constexpr int NS = D / 16;     // 16-wide d slices (QK^T fragments)
    constexpr int NT = D / 32;     // 32-wide d tiles (output / V^T)
    constexpr int VST = 40;        // padded k-stride of V^T tile (16B-mult)

    const int lane = threadIdx.x & 63;
    const int wid = threadIdx.x >> 6;
    const int hi = lane >> 5;
    const int ln = lane & 31;
    const int hq = blockIdx.y;
    const int hk = hq / G;
    const int qw = q0 + wid * 32;

    // Q fragments: lane holds Q[qw+ln][s*16 + hi*8 + 0..7] (B operand)
    bf16x8 qf[NS];
    {
        const bf16_t* qrow =
            q + ((long)min(qw + ln, T - 1) * Hq + hq) * D + hi * 8;
#pragma unroll
        for (int s = 0; s < NS; ++s) qf[s] = *(const bf16x8*)(qrow + s * 16);
    }

    const int q_abs = causal_off + qw + ln;   // this lane's absolute q pos
    float m = -INFINITY, l = 0.f;
    f32x16 acc[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) acc[t][r] = 0.f;

    // causal upper bound for the workgroup's LAST q-row
    const int kmax = min(s_total, causal_off + q0 + 128);

    const int qfirst = causal_off + q0;
    for (int k0 = keys.skip(0, qfirst); k0 < kmax;
         k0 = keys.skip(k0 + 32, qfirst)) {
        const long blk = kv.off(slot, hk, k0);   // 32 keys lie together
        const int klast = s_total - 1 - k0;
        // ---- stage V^T tile (cooperative transpose) --------------------
        __syncthreads();               // previous tile's vt readers done
        {
            constexpr int CPR = D / 8;            // b128 chunks per V row
            for (int c = threadIdx.x; c < 32 * CPR; c += 256) {
                const int kr = c / CPR;
                const int d8 = (c % CPR) * 8;
                uint4 v = *(const uint4*)(
                    kv.v + blk + min(kr, klast) * D + d8);
                const bf16_t* pv = (const bf16_t*)&v;
#pragma unroll
                for (int j = 0; j < 8; ++j) vt[(d8 + j) * VST + kr] = pv[j];
            }
        }
        __syncthreads();

        // ---- S^T = K·Q^T (K fragments straight from HBM/L2) ------------
        f32x16 s_acc;
#pragma unroll
        for (int r = 0; r < 16; ++r) s_acc[r] = 0.f;
        {
            const bf16_t* krow =
                kv.k + blk + min(ln, klast) * D + hi * 8;
#pragma unroll
            for (int s = 0; s < NS; ++s) {
                const bf16x8 kf = *(const bf16x8*)(krow + s * 16);
                s_acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
                    kf, qf[s], s_acc, 0, 0, 0);
            }
        }

        // ---- mask + online softmax (lane owns one q-row) ---------------
        float sv[16], tmax = -INFINITY;
        const float scl2 = scale * 1.4426950408889634f;   // log2 domain
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const int kg = k0 + (r & 3) + 8 * (r >> 2) + 4 * hi;
            const bool ok = (kg < s_total) && (kg <= q_abs) &&
                            keys.sees(q_abs, kg);
            sv[r] = ok ? s_acc[r] * scl2 : -INFINITY;
            tmax = fmaxf(tmax, sv[r]);
        }
        tmax = fmaxf(tmax, __shfl_xor(tmax, 32, WAVE));
        const float mn = fmaxf(m, tmax);
        const float alpha = (m == -INFINITY) ? 0.f : exp2f(m - mn);
        float p[16], psum = 0.f;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            p[r] = (sv[r] == -INFINITY) ? 0.f : exp2f(sv[r] - mn);
            psum += p[r];
        }
        psum += __shfl_xor(psum, 32, WAVE);
        l = l * alpha + psum;
        m = mn;

        // ---- P -> PV B-fragment layout via per-wave LDS scratch --------
        // (kpos, q=ln) lands where slice sidx = kpos>>4, lane
        // lr = ln + 32*((kpos>>3)&1), word i = kpos&7 will read it; regs
        // pair (r, r+1) = (kpos, kpos+1) -> one packed b32 write.
        bf16_t* ps = plds_all + wid * (2 * 64 * 8);
#pragma unroll
        for (int r = 0; r < 16; r += 2) {
            const int kpos = (r & 3) + 8 * (r >> 2) + 4 * hi;
            const int sidx = kpos >> 4;
            const int lr = ln + 32 * ((kpos >> 3) & 1);
            u32 w = (u32)f2bf(p[r]) | ((u32)f2bf(p[r + 1]) << 16);
            *(u32*)(ps + (sidx * 64 + lr) * 8 + (kpos & 7)) = w;
        }
        // rescale output accumulators while the P writes land
#pragma unroll
        for (int t = 0; t < NT; ++t)
#pragma unroll
            for (int r = 0; r < 16; ++r) acc[t][r] *= alpha;
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");

        // ---- O^T += V^T · P --------------------------------------------
        bf16x8 pf[2];
#pragma unroll
        for (int s = 0; s < 2; ++s)
            pf[s] = *(const bf16x8*)(ps + (s * 64 + lane) * 8);
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const bf16_t* vrow = vt + (t * 32 + ln) * VST + hi * 8;
#pragma unroll
            for (int s = 0; s < 2; ++s) {
                const bf16x8 vf = *(const bf16x8*)(vrow + s * 16);
                acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
                    vf, pf[s], acc[t], 0, 0, 0);
            }
        }
    }

    // ---- normalize + store: lane holds O^T[*][q=ln] — one q-row --------
    if (qw + ln < T) {
        const float inv = epi.factor(row0 + qw + ln, hq, m, l);
        bf16_t* orow = out + epi.at(qw + ln, hq, Hq, D);
#pragma unroll
        for (int t = 0; t < NT; ++t) {
#pragma unroll
            for (int g = 0; g < 4; ++g) {
                const int d = t * 32 + 8 * g + 4 * hi;
                float f[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) f[i] = acc[t][4 * g + i] * inv;
                if (epi.gate_el) {
                    float z[4];
                    ld4(epi.gate + (long)(row0 + qw + ln) * epi.gate_ld +
                        hq * D + d, z);
#pragma unroll
                    for (int i = 0; i < 4; ++i) f[i] /= 1.f + __expf(-z[i]);
                }
                st4(orow + d, f);
            }
        }
    }
}
