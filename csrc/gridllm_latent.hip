// gfx950 kernels of latent attention: softmax attention whose keys and values
// are made from one latent per token, c [KR], and a rotated key part shared by
// all heads, r [R]. A token's cached row is [c | r]; pages of 64 rows.
//
// Per head, score = (q_n . W_uk c + q_r . r) scale and value = W_uv c. Two ways
// to the same result:
//  * absorbed (decode rows, short portions, the exact mode): q_l = W_uk^T q_n
//    meets the latents themselves, and W_uv is applied to the weighted sum of
//    latents. All heads read the same cached rows.
//  * expanded (prompt portions): W_uk c and W_uv c of the whole sequence are
//    made once per step by a library GEMM, and attention runs on those; per
//    score and key that is KR / dim times less work.
//
// Sizes are padded by the host with zero weights: KR to 64, 128, 256 or 512, R
// to 64 or 128, head sizes (unrotated keys and values alike) to P = 64, 128 or
// 256. A query row is [H][P + R], its last R rotated where it is read.

#include "gridllm_tiles.h"

// Online softmax: the reference m of the exponents moves only when the maximum
// has grown by more than this (in powers of two), so that sums are rarely
// scaled again; weights then stay below 2^8.
#define MAX_LAG 8.f

// out = x / rms(x) * w over a row, one wave; W columns, mean over Wtrue
template <class T>
DEV_INLINE void wave_norm(T* out, const T* x, const float* w, int W, int Wtrue,
                          float eps) {
    const int lane = threadIdx.x & 63;
    float ss = 0.f;
    for (int c = lane * 8; c < W; c += 512) {
        float f[8];
        ld8(x + c, f);
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += f[i] * f[i];
    }
    const float rs = 1.f / sqrtf(wave_reduce_sum(ss) / (float)Wtrue + eps);
    for (int c = lane * 8; c < W; c += 512) {
        float f[8], g[8];
        ld8(x + c, f);
        ld8(w + c, g);
#pragma unroll
        for (int i = 0; i < 8; ++i) f[i] *= rs * g[i];
        st8(out + c, f);
    }
}

// ===========================================================================
// From a projection row [q latent QR | latent KR | rotated part R | ...],
// stride ld: the normed query latent, and the token's cached row (normed
// latent, rotated part). One wave per token and half.
// ===========================================================================
template <class T>
__global__ void __launch_bounds__(256)
k_latent_rows(const T* __restrict__ rows, T* __restrict__ cq,
              T* __restrict__ lat, const int* __restrict__ table, int per_slot,
              const int* __restrict__ pos, const int* __restrict__ slot,
              const float* __restrict__ qw, const float* __restrict__ kw,
              const Rotation rot, int N, int QR, int qtrue, int KR, int ktrue,
              int R, int ld_, float eps) {
    const long item = blockIdx.x * 4L + (threadIdx.x >> 6);
    const int n = (int)(item >> 1), lane = threadIdx.x & 63;
    if (n >= N) return;
    const T* row = rows + (long)n * ld_;
    if (!(item & 1)) {
        wave_norm(cq + (long)n * QR, row, qw, QR, qtrue, eps);
        return;
    }
    const int p = pos[n], blk = p / PAGE;
    if (blk >= per_slot) return;
    const long page = table[(long)slot[n] * per_slot + blk];
    T* dst = lat + (page * PAGE + p % PAGE) * (KR + R);
    wave_norm(dst, row + QR, kw, KR, ktrue, eps);
    if (lane * 8 < R) {
        float f[8];
        ld8(row + QR + KR + lane * 8, f);
        rotate8(f, lane * 8, p, rot);
        st8(dst + KR + lane * 8, f);
    }
}

// ===========================================================================
// Per-head product: out[r, h, n] = sum_k x[r, h, k] w[h, n, k], times
// sigmoid(gate[r, h]) if there is a gate. x rows have stride ldx and heads
// stride hx; out is [rows][H][N]. Block: RT * 16 rows x 64 columns of a head.
// ===========================================================================
template <int RT>
__global__ void __launch_bounds__(256)
k_head_gemm(bf16_t* __restrict__ out, const bf16_t* __restrict__ x,
            const bf16_t* __restrict__ w, const bf16_t* __restrict__ gate,
            int gate_ld, int rows, int H, int N, int K, long ldx, int hx) {
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int fr = lane & 15, kg = (lane >> 4) * 8;
    const int nb = N / 64;
    const int h = blockIdx.x / nb, n0 = (blockIdx.x % nb) * 64 + wid * 16;
    const int r0 = blockIdx.y * RT * 16;
    const bf16_t* wr = w + ((long)h * N + n0 + fr) * K + kg;
    const bf16_t* xr[RT];
    f32x4 acc[RT];
#pragma unroll
    for (int t = 0; t < RT; ++t) {
        xr[t] = x + min(r0 + t * 16 + fr, rows - 1) * ldx + (long)h * hx + kg;
        acc[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    }
#pragma unroll 4
    for (int k = 0; k < K; k += 32) {
        const bf16x8 a = *(const bf16x8*)(wr + k);
#pragma unroll
        for (int t = 0; t < RT; ++t)
            acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                a, *(const bf16x8*)(xr[t] + k), acc[t], 0, 0, 0);
    }
#pragma unroll
    for (int t = 0; t < RT; ++t) {
        const int r = r0 + t * 16 + fr;
        if (r >= rows) continue;
        float s = 1.f;
        if (gate) s = sigmoidf_(bf2f(gate[(long)r * gate_ld + h]));
        const float f[4] = {acc[t][0] * s, acc[t][1] * s, acc[t][2] * s,
                            acc[t][3] * s};
        st4(out + ((long)r * H + h) * N + n0 + (lane >> 4) * 4, f);
    }
}

// exact mode: one block per row and head
__global__ void __launch_bounds__(256)
k_head_gemm_f32(float* __restrict__ out, const float* __restrict__ x,
                const float* __restrict__ w, const float* __restrict__ gate,
                int gate_ld, int H, int N, int K, long ldx, int hx) {
    __shared__ float xs[512];
    const int r = blockIdx.x / H, h = blockIdx.x % H;
    for (int k = threadIdx.x; k < K; k += 256)
        xs[k] = x[r * ldx + (long)h * hx + k];
    __syncthreads();
    const float s = gate ? sigmoidf_(gate[(long)r * gate_ld + h]) : 1.f;
    for (int n = threadIdx.x; n < N; n += 256) {
        const float* wr = w + ((long)h * N + n) * K;
        float a = 0.f;
        for (int k = 0; k < K; k += 4) {
            const float4 v = *(const float4*)(wr + k);
            a += v.x * xs[k] + v.y * xs[k + 1] + v.z * xs[k + 2] +
                 v.w * xs[k + 3];
        }
        out[((long)r * H + h) * N + n] = a * s;
    }
}

// ===========================================================================
// Absorbed attention. Row n of a step sees the keys 0 .. pos[n] of slot[n].
//   ql: [N][H][KR] absorbed queries; q: [N][H][P + R] for the rotated part
//   out: [N][H][KR] weighted sums of latents, or partial ones and their
//   log2-domain maxima and sums, f32 [N][H][nsplit][KR + 2], if nsplit > 1
// Block: a row, HG times 16 heads, a split of the keys. Tiles of 32 cached rows
// go through LDS (16-byte pieces XOR-swizzled by the row), once as keys
// (row-wise fragments) and once as values (transposed reads); one tile is ahead
// in a block of 4 waves, of which a CU takes two, and two tiles in a block of 8
// waves. Four waves share 16 heads. Scores: a wave takes 16 keys over half of
// the row, the halves meet in LDS, and every wave then forms the weights of all
// 32 keys, which are its A fragment, against a quarter of the latent columns.
// ===========================================================================
template <int KR, int R, int HG>
__global__ void __launch_bounds__(256 * HG, 2)
k_latent_decode(bf16_t* __restrict__ out, const bf16_t* __restrict__ ql,
                const bf16_t* __restrict__ q, const bf16_t* __restrict__ lat,
                const int* __restrict__ table, int per_slot,
                const int* __restrict__ pos, const int* __restrict__ slot,
                float* __restrict__ ws, const Rotation rot, int N, int H,
                int P, int nsplit, float scale) {
    constexpr int D = KR + R, CH = D / 8;         // 16-byte pieces of a row
    constexpr int WAVES = 4 * HG;
    constexpr int LOADS = (CH / 2 + WAVES - 1) / WAVES;   // of a wave, 64 each
    constexpr int SQ = D / 64;                    // score steps of a half
    constexpr int NT = KR / 64;                   // 16-column tiles of a wave
    constexpr int U = 5, NH = (NT + 1) / 2;
    constexpr int NB = HG + 1;                    // tiles in LDS
    // (the last turn of loads may be half empty: those lanes load piece 0)
    __shared__ __attribute__((aligned(16)))
    bf16_t tile[NB][LOADS * WAVES * 512];
    __shared__ __attribute__((aligned(16))) float red[2][HG][16][32];
    // blocks of the same row and split, but other heads, on the same XCD
    const int hgs = (H + 16 * HG - 1) / (16 * HG);
    const int item = (int)(blockIdx.x >> 3) / hgs * 8 + (blockIdx.x & 7);
    if (item >= N * nsplit) return;
    const int n = item / nsplit, split = item % nsplit;
    const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6;
    const int g = wv >> 2, wid = wv & 3;
    const int h0 = ((int)(blockIdx.x >> 3) % hgs * HG + g) * 16;
    const int fr = lane & 15, kg = (lane >> 4) * 8;
    const int p = pos[n];
    const int seq = min(p + 1, per_slot * PAGE);
    const int tiles = (seq + 31) >> 5;
    const int per = (tiles + nsplit - 1) / nsplit;
    const int t0 = split * per, t1 = min(tiles, t0 + per);
    const int* tab = table + (long)slot[n] * per_slot;

    int off[LOADS];                   // of this thread's pieces in a tile
#pragma unroll
    for (int i = 0; i < LOADS; ++i) {
        const int pc = (i * WAVES + wv) * 64 + lane;
        const int row = pc / CH, c = pc % CH;
        off[i] = row < 32 ? row * D + (c ^ (row & 7)) * 8 : 0;
    }
    auto issue = [&](int t, int page) {
        const bf16_t* src = lat + ((long)page * PAGE + (t & 1) * 32) * D;
#pragma unroll
        for (int i = 0; i < LOADS; ++i)
            load_lds16(src + off[i],
                       tile[(t - t0) % NB] + (i * WAVES + wv) * 512);
    };
#pragma unroll
    for (int i = 0; i < NB - 1; ++i)
        if (t0 + i < t1) issue(t0 + i, tab[(t0 + i) >> 1]);
    int page = tab[min(t0 + NB - 1, tiles - 1) >> 1];

    // queries: head h0 + fr, this wave's half of the row
    const int dbeg = (wid >> 1) * (D / 2) + kg, krow = (wid & 1) * 16 + fr;
    const long qrow = (long)n * H + min(h0 + fr, H - 1);
    bf16x8 qf[SQ];
#pragma unroll
    for (int s = 0; s < SQ; ++s) {
        const int d = dbeg + s * 32;
        if (D / 2 + s * 32 + 32 <= KR || d < KR) {
            qf[s] = *(const bf16x8*)(ql + qrow * KR + d);
        } else {
            float f[8];
            ld8(q + qrow * (P + R) + P + d - KR, f);
            rotate8(f, d - KR, p, rot);
            qf[s] = to_bf16x8(f);
        }
    }

    float m = -INFINITY, l = 0.f;     // of head fr; l over this lane's keys
    f32x4 acc[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t) acc[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const float scale2 = scale * LOG2E;
    for (int t = t0; t < t1; ++t) {
        const bf16_t* kv = tile[(t - t0) % NB];
        if (NB == 3 && t + 1 < t1)
            asm volatile("s_waitcnt vmcnt(%0)" :: "i"(LOADS * (NB - 2))
                         : "memory");
        else
            asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        lds_barrier();                // tile is there, another one is free
        if (t + NB - 1 < t1) {
            issue(t + NB - 1, page);
            page = tab[min(t + NB, tiles - 1) >> 1];
        }
        f32x4 sc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s0 = 0; s0 < SQ; s0 += U) {     // U reads in flight
            bf16x8 kf[U];
#pragma unroll
            for (int i = 0; i < U; ++i)
                if (s0 + i < SQ)
                    kf[i] = *(const bf16x8*)(
                        kv + krow * D +
                        (((dbeg + (s0 + i) * 32) >> 3) ^ (krow & 7)) * 8);
#pragma unroll
            for (int i = 0; i < U; ++i)
                if (s0 + i < SQ)
                    sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                        qf[s0 + i], kf[i], sc, 0, 0, 0);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = (lane >> 4) * 4 + r;         // swizzled, too
            red[wid >> 1][g][row][krow ^ ((row & 7) * 4)] = sc[r];
        }
        auto values = [&](int c) {               // columns of tile c
            const int d = wid * (KR / 4) + c * 16 + (fr & 3) * 4;
            bf16x8 v;
#pragma unroll
            for (int j = 0; j < 2; ++j) {
                const int row = kg + (fr >> 2) + j * 4;
                const bf16x4 x = read_transposed(
                    kv + row * D + ((d >> 3) ^ (row & 7)) * 8 + (d & 7));
#pragma unroll
                for (int i = 0; i < 4; ++i) v[j * 4 + i] = x[i];
            }
            return v;
        };
        bf16x8 vf[NH];                           // half of them ahead of time
#pragma unroll
        for (int c = 0; c < NH; ++c) vf[c] = values(c);
        lds_barrier();
        float s8[8], hi8[8], mx = -INFINITY;
#pragma unroll
        for (int i = 0; i < 8; i += 4) {
            const int c = (kg + i) ^ ((fr & 7) * 4);
            ld4(&red[0][g][fr][c], s8 + i);
            ld4(&red[1][g][fr][c], hi8 + i);
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            s8[i] = t * 32 + kg + i < seq ? (s8[i] + hi8[i]) * scale2
                                          : -INFINITY;
            mx = fmaxf(mx, s8[i]);
        }
        mx = max_across16(mx);                   // finite: a tile has a key
        if (__any(mx > m + MAX_LAG)) {
            const float mn = mx > m + MAX_LAG ? mx : m;
            const float alpha = fast_exp2(m - mn);
            l *= alpha;
            m = mn;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const float a = __shfl(alpha, (lane >> 4) * 4 + r, WAVE);
#pragma unroll
                for (int c = 0; c < NT; ++c) acc[c][r] *= a;
            }
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            s8[i] = fast_exp2(s8[i] - m);
            l += s8[i];
        }
        const bf16x8 pf = to_bf16x8(s8);
#pragma unroll
        for (int c = 0; c < NT; ++c)
            acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                pf, c < NH ? vf[c] : values(c), acc[c], 0, 0, 0);
    }
    l += __shfl_xor(l, 16, WAVE);
    l += __shfl_xor(l, 32, WAVE);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int hd = (lane >> 4) * 4 + r;
        const float lr = __shfl(l, hd, WAVE), mr = __shfl(m, hd, WAVE);
        if (h0 + hd >= H) continue;
        const long row = (long)n * H + h0 + hd;
        const int c0 = wid * (KR / 4) + fr;
        if (nsplit == 1) {
            const float inv = 1.f / lr;
#pragma unroll
            for (int c = 0; c < NT; ++c)
                out[row * KR + c0 + c * 16] = f2bf(acc[c][r] * inv);
        } else {
            float* wp = ws + (row * nsplit + split) * (KR + 2);
#pragma unroll
            for (int c = 0; c < NT; ++c) wp[c0 + c * 16] = acc[c][r];
            if (wid == 0 && fr == 0) {
                wp[KR] = mr;
                wp[KR + 1] = lr;
            }
        }
    }
}

// One wave per row and head (x) and 64 latent columns (y); nsplit <= 64.
__global__ void __launch_bounds__(64)
k_latent_combine(bf16_t* __restrict__ out, const float* __restrict__ ws,
                 int KR, int nsplit) {
    const float* base = ws + blockIdx.x * (long)nsplit * (KR + 2);
    const int lane = threadIdx.x, c = blockIdx.y * 64 + lane;
    float m = -INFINITY, l = 0.f;              // of split `lane`
    if (lane < nsplit) {
        m = base[lane * (KR + 2) + KR];
        l = base[lane * (KR + 2) + KR + 1];
    }
    const float f = exp2f(m - wave_reduce_max(m));   // split 0 has a key
    const float inv = 1.f / wave_reduce_sum(f * l);
    float a = 0.f;
    constexpr int U = 8;
    for (int s0 = 0; s0 < nsplit; s0 += U) {
        float v[U];
#pragma unroll
        for (int u = 0; u < U; ++u)
            v[u] = base[min(s0 + u, nsplit - 1) * (KR + 2) + c];
#pragma unroll
        for (int u = 0; u < U; ++u)
            a += s0 + u < nsplit ? __shfl(f, s0 + u, WAVE) * v[u] : 0.f;
    }
    out[blockIdx.x * (long)KR + c] = f2bf(a * inv);
}

// exact mode: one block per row and head, any position
__global__ void __launch_bounds__(256)
k_latent_attn_f32(float* __restrict__ out, const float* __restrict__ ql,
                  const float* __restrict__ q, const float* __restrict__ lat,
                  const int* __restrict__ table, int per_slot,
                  const int* __restrict__ pos, const int* __restrict__ slot,
                  const Rotation rot, int H, int P, int KR, int R,
                  float scale) {
    __shared__ float qs[640], sc[256], red[4];
    const int n = blockIdx.x / H, h = blockIdx.x % H, D = KR + R;
    const int* tab = table + (long)slot[n] * per_slot;
    const int p = pos[n], seq = min(p + 1, per_slot * PAGE);
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    for (int c = threadIdx.x; c < KR; c += 256)
        qs[c] = ql[((long)n * H + h) * KR + c];
    for (int c = threadIdx.x * 8; c < R; c += 2048) {
        float f[8];
        ld8(q + ((long)n * H + h) * (P + R) + P + c, f);
        rotate8(f, c, p, rot);
        for (int i = 0; i < 8; ++i) qs[KR + c + i] = f[i];
    }
    __syncthreads();
    float m = -INFINITY, l = 0.f, acc[2] = {0.f, 0.f};
    for (int k0 = 0; k0 < seq; k0 += 256) {
        const int j = k0 + threadIdx.x;
        float s = -INFINITY;
        if (j < seq) {
            const float* kr = lat + ((long)tab[j / PAGE] * PAGE + j % PAGE) * D;
            s = 0.f;
            for (int i = 0; i < D; i += 4) {
                const float4 v = *(const float4*)(kr + i);
                s += v.x * qs[i] + v.y * qs[i + 1] + v.z * qs[i + 2] +
                     v.w * qs[i + 3];
            }
            s *= scale;
        }
        float mx = wave_reduce_max(s);
        if (lane == 0) red[wid] = mx;
        __syncthreads();
        mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
        const float mn = fmaxf(m, mx);
        const float alpha = m == -INFINITY ? 0.f : expf(m - mn);
        const float w = j < seq ? expf(s - mn) : 0.f;
        sc[threadIdx.x] = w;
        m = mn;
        __syncthreads();                       // red read, sc written
        const float ps = wave_reduce_sum(w);
        if (lane == 0) red[wid] = ps;
        const int jn = min(256, seq - k0);
        acc[0] *= alpha;
        acc[1] *= alpha;
        for (int t = 0; t < jn; ++t) {
            const int jj = k0 + t;
            const float* v =
                lat + ((long)tab[jj / PAGE] * PAGE + jj % PAGE) * D;
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                const int c = threadIdx.x + i * 256;
                if (c < KR) acc[i] += sc[t] * v[c];
            }
        }
        __syncthreads();
        l = l * alpha + red[0] + red[1] + red[2] + red[3];
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
        const int c = threadIdx.x + i * 256;
        if (c < KR) out[((long)n * H + h) * KR + c] = acc[i] / l;
    }
}

// ===========================================================================
// Expanded attention.
// ===========================================================================
// Cached rows of the portions' sequences, one after the other. Item (int4):
// {page number within the sequence, slot, first row of dst, rows}; rows from
// there to the end of the page's 64 (or what dst keeps of them, `.w >> 8`
// rows) become zero.
__global__ void __launch_bounds__(256)
k_latent_gather(bf16_t* __restrict__ dst, const bf16_t* __restrict__ lat,
                const int* __restrict__ table, int per_slot,
                const int4* __restrict__ items, int D) {
    const int4 it = items[blockIdx.x];
    const int have = (it.w & 255) * D / 8, all = (it.w >> 8) * D / 8;
    const uint4* src = (const uint4*)(
        lat + (long)table[(long)it.y * per_slot + it.x] * PAGE * D);
    uint4* d = (uint4*)(dst + (long)it.z * D);
    for (int i = threadIdx.x; i < all; i += 256)
        d[i] = i < have ? src[i] : make_uint4(0, 0, 0, 0);
}

// One 128-row tile of a portion and head. meta (8 ints): {first token of the
// portion, its length, first row of its sequence in the gathered rows, first
// row of the tile, start position}. e: [rows][H][2 P], keys | values; lat: the
// gathered rows, whose last R are the rotated part. A wave owns 32 query rows.
// S^T = K Q^T puts a query row's scores into one lane pair; the weights become
// the B operand of O^T = V^T P by one swap of lane halves.
template <int P, int R>
__global__ void __launch_bounds__(256, P > 128 ? 1 : 2)
k_latent_prefill(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
                 const bf16_t* __restrict__ e, const bf16_t* __restrict__ lat,
                 int lat_ld, const int* __restrict__ meta, int ntiles,
                 const Rotation rot, int H, float scale,
                 const bf16_t* __restrict__ gate, int gate_ld) {
    constexpr int KD = P + R, KC = KD / 8, VC = P / 8;
    constexpr int LOADS = 32 * (KC + VC) / 256;
    constexpr int NS = KD / 16, NT = P / 32;
    __shared__ __attribute__((aligned(16))) bf16_t tile[2][32 * (KD + P)];
    // neighbouring work (tiles of one head) on the same XCD, longest first
    const int total = ntiles * H, per = (total + 7) >> 3;
    const int i0 = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per || i0 >= total) return;
    const int h = i0 / ntiles;
    const int* mt = meta + (ntiles - 1 - i0 % ntiles) * 8;
    const int q_off = mt[0], len = mt[1], key_off = mt[2], q0 = mt[3];
    const int start = mt[4];
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int hi = lane >> 5, ln = lane & 31;
    const int qw = q0 + wid * 32;
    const int qrow = min(qw + ln, len - 1);
    const int q_abs = start + qw + ln;          // of this lane
    const int kmax = start + min(q0 + 128, len);

    bf16x8 qf[NS];
    {
        const bf16_t* qr = q + ((long)(q_off + qrow) * H + h) * KD + hi * 8;
#pragma unroll
        for (int s = 0; s < NS; ++s) {
            if (s * 16 < P) {
                qf[s] = *(const bf16x8*)(qr + s * 16);
            } else {
                float f[8];
                ld8(qr + s * 16, f);
                rotate8(f, s * 16 - P + hi * 8, start + qrow, rot);
                qf[s] = to_bf16x8(f);
            }
        }
    }

    const bf16_t* src[LOADS];
    int step[LOADS];
#pragma unroll
    for (int i = 0; i < LOADS; ++i) {
        const int pc = i * 256 + threadIdx.x;
        const bool is_k = pc < 32 * KC;
        const int pr = is_k ? pc : pc - 32 * KC;
        const int row = is_k ? pr / KC : pr / VC;
        const int c = ((is_k ? pr % KC : pr % VC) ^ (row & 7)) * 8;
        if (is_k && c >= P) {
            src[i] = lat + (long)(key_off + row) * lat_ld + lat_ld - R + c - P;
            step[i] = 32 * lat_ld;
        } else {
            src[i] = e + ((long)(key_off + row) * H + h) * 2 * P +
                     (is_k ? c : P + c);
            step[i] = 64 * H * P;
        }
    }
    auto issue = [&](int buf) {
#pragma unroll
        for (int i = 0; i < LOADS; ++i) {
            load_lds16(src[i], tile[buf] + (i * 256 + wid * 64) * 8);
            src[i] += step[i];
        }
    };

    float m = -INFINITY, l = 0.f;
    f32x16 acc[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) acc[t][r] = 0.f;
    const float scale2 = scale * LOG2E;
    issue(0);
    for (int k0 = 0; k0 < kmax; k0 += 32) {
        const bf16_t* kt = tile[(k0 >> 5) & 1];
        const bf16_t* vt = kt + 32 * KD;
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        lds_barrier();              // tile is there, the other one is free
        if (k0 + 32 < kmax) issue(((k0 >> 5) + 1) & 1);
        if (k0 > start + qw + 31) continue;     // ahead of all of this wave
        f32x16 sv;
#pragma unroll
        for (int r = 0; r < 16; ++r) sv[r] = 0.f;
#pragma unroll
        for (int s = 0; s < NS; ++s)
            sv = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
                *(const bf16x8*)(kt + ln * KD +
                                 ((s * 2 + hi) ^ (ln & 7)) * 8),
                qf[s], sv, 0, 0, 0);
        float mx = -INFINITY;
        if (k0 + 31 <= start + qw) {
#pragma unroll
            for (int r = 0; r < 16; ++r) mx = fmaxf(mx, sv[r]);
        } else {
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const int key = k0 + (r & 3) + 8 * (r >> 2) + 4 * hi;
                if (key > q_abs) sv[r] = -INFINITY;
                mx = fmaxf(mx, sv[r]);
            }
        }
        mx = max_across32(mx) * scale2;         // finite: a key is visible
        if (__any(mx > m + MAX_LAG)) {
            const float mn = mx > m + MAX_LAG ? mx : m;
            const float alpha = fast_exp2(m - mn);
            l *= alpha;
            m = mn;
#pragma unroll
            for (int t = 0; t < NT; ++t)
#pragma unroll
                for (int r = 0; r < 16; ++r) acc[t][r] *= alpha;
        }
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            sv[r] = fast_exp2(fmaf(sv[r], scale2, -m));
            l += sv[r];                         // this lane's keys
        }
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            // lane half hi holds keys 8 g + 4 hi + 0..3; it needs 8 hi + 0..7
            u32 w[4];
#pragma unroll
            for (int i = 0; i < 2; ++i) {
                const u32x2 x = __builtin_amdgcn_permlane32_swap(
                    pack2(sv[8 * s + 2 * i], sv[8 * s + 2 * i + 1]),
                    pack2(sv[8 * s + 4 + 2 * i], sv[8 * s + 5 + 2 * i]),
                    false, false);
                w[i] = x[0];
                w[2 + i] = x[1];
            }
            bf16x8 pf;
            __builtin_memcpy(&pf, w, 16);
            const int vrow = s * 16 + hi * 8 + ((lane & 15) >> 2);
#pragma unroll
            for (int t = 0; t < NT; ++t) {
                const int d = t * 32 + (lane & 16) + (lane & 3) * 4;
                bf16x8 v;
#pragma unroll
                for (int j = 0; j < 2; ++j) {
                    const int row = vrow + j * 4;
                    const bf16x4 x = read_transposed(
                        vt + row * P + ((d >> 3) ^ (row & 7)) * 8 + (d & 7));
#pragma unroll
                    for (int i = 0; i < 4; ++i) v[j * 4 + i] = x[i];
                }
                acc[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
                    v, pf, acc[t], 0, 0, 0);
            }
        }
    }
    l += __shfl_xor(l, 32, WAVE);
    if (qw + ln >= len) return;
    float inv = 1.f / l;
    if (gate)
        inv *= sigmoidf_(bf2f(gate[(long)(q_off + qrow) * gate_ld + h]));
    bf16_t* orow = out + ((long)(q_off + qrow) * H + h) * P;
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int g = 0; g < 4; ++g)
            *(uint2*)(orow + t * 32 + 8 * g + 4 * hi) = make_uint2(
                pack2(acc[t][4 * g] * inv, acc[t][4 * g + 1] * inv),
                pack2(acc[t][4 * g + 2] * inv, acc[t][4 * g + 3] * inv));
}

// ===========================================================================
// Entry points. f32 != 0 selects the exact mode. 0 = success.
// ===========================================================================
static bool sizes_ok(int KR, int R) {
    return (KR == 64 || KR == 128 || KR == 256 || KR == 512) &&
           (R == 64 || R == 128);
}

extern "C" {

int gn_latent_rows(void* stream, int f32, const void* rows, void* cq,
                   void* lat, const void* table, int per_slot, const void* pos,
                   const void* slot, const void* qw, const void* kw,
                   const void* cos_, const void* sin_, int nrot, int N, int QR,
                   int qtrue, int KR, int ktrue, int R, int ld_, float eps) {
    if (N < 1 || QR % 64 || !sizes_ok(KR, R) || nrot < 1) return -100;
    hipStream_t st_ = (hipStream_t)stream;
    const Rotation rot{(const float*)cos_, (const float*)sin_, R / 2, nrot};
#define GO(T) k_latent_rows<T><<<(N * 2 + 3) / 4, 256, 0, st_>>>( \
        (const T*)rows, (T*)cq, (T*)lat, (const int*)table, per_slot, \
        (const int*)pos, (const int*)slot, (const float*)qw, \
        (const float*)kw, rot, N, QR, qtrue, KR, ktrue, R, ld_, eps)
    if (f32) GO(float); else GO(bf16_t);
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gn_head_gemm(void* stream, int f32, void* out, const void* x,
                 const void* w, const void* gate, int gate_ld, int rows,
                 int H, int N, int K, long ldx, int hx) {
    if (rows < 1 || H < 1 || N % 64 || K % 64 || K > 512) return -100;
    hipStream_t st_ = (hipStream_t)stream;
    if (f32) {
        k_head_gemm_f32<<<(unsigned)((long)rows * H), 256, 0, st_>>>(
            (float*)out, (const float*)x, (const float*)w, (const float*)gate,
            gate_ld, H, N, K, ldx, hx);
        LAUNCH_CHECK();
        return 0;
    }
#define GO(RT) k_head_gemm<RT><<<dim3(H * (N / 64), \
        (rows + 16 * RT - 1) / (16 * RT)), 256, 0, st_>>>((bf16_t*)out, \
        (const bf16_t*)x, (const bf16_t*)w, (const bf16_t*)gate, gate_ld, \
        rows, H, N, K, ldx, hx)
    // as many rows per block as still fill the chip
    const long tiles = (long)H * (N / 64) * ((rows + 15) / 16);
    if (rows <= 16 || tiles < 2048) GO(1);
    else if (rows <= 32 || tiles < 4096) GO(2);
    else GO(4);
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gn_latent_decode(void* stream, void* out, const void* ql, const void* q,
                     const void* lat, const void* table, int per_slot,
                     const void* pos, const void* slot, void* ws,
                     const void* cos_, const void* sin_, int nrot, int N,
                     int H, int P, int KR, int R, int nsplit, float scale) {
    if (N < 1 || H < 1 || nsplit < 1 || nsplit > 64 || !sizes_ok(KR, R))
        return -100;
    hipStream_t st_ = (hipStream_t)stream;
    const Rotation rot{(const float*)cos_, (const float*)sin_, R / 2, nrot};
    const int hgb = H > 16 ? 32 : 16;         // heads of a block
    const unsigned grid =
        (unsigned)(((long)N * nsplit + 7) / 8 * 8 * ((H + hgb - 1) / hgb));
#define GO(A, B) if (hgb == 32) GO1(A, B, 2); else GO1(A, B, 1)
#define GO1(A, B, C) k_latent_decode<A, B, C><<<grid, 256 * C, 0, st_>>>( \
        (bf16_t*)out, (const bf16_t*)ql, (const bf16_t*)q, (const bf16_t*)lat, \
        (const int*)table, per_slot, (const int*)pos, (const int*)slot, \
        (float*)ws, rot, N, H, P, nsplit, scale)
#define PICK(B) do { if (KR == 64) { GO(64, B); } \
        else if (KR == 128) { GO(128, B); } \
        else if (KR == 256) { GO(256, B); } else { GO(512, B); } } while (0)
    if (R == 64) PICK(64); else PICK(128);
#undef PICK
#undef GO1
#undef GO
    LAUNCH_CHECK();
    if (nsplit > 1) {
        k_latent_combine<<<dim3(N * H, KR / 64), 64, 0, st_>>>(
            (bf16_t*)out, (const float*)ws, KR, nsplit);
        LAUNCH_CHECK();
    }
    return 0;
}

int gn_latent_attn_f32(void* stream, void* out, const void* ql, const void* q,
                       const void* lat, const void* table, int per_slot,
                       const void* pos, const void* slot, const void* cos_,
                       const void* sin_, int nrot, int N, int H, int P,
                       int KR, int R, float scale) {
    if (N < 1 || H < 1 || !sizes_ok(KR, R)) return -100;
    k_latent_attn_f32<<<(unsigned)((long)N * H), 256, 0,
                        (hipStream_t)stream>>>((float*)out, (const float*)ql,
        (const float*)q, (const float*)lat, (const int*)table, per_slot,
        (const int*)pos, (const int*)slot,
        Rotation{(const float*)cos_, (const float*)sin_, R / 2, nrot}, H, P,
        KR, R, scale);
    LAUNCH_CHECK();
    return 0;
}

int gn_latent_gather(void* stream, void* dst, const void* lat,
                     const void* table, int per_slot, const void* items,
                     int nitems, int D) {
    if (nitems < 1 || D % 64) return -100;
    k_latent_gather<<<nitems, 256, 0, (hipStream_t)stream>>>(
        (bf16_t*)dst, (const bf16_t*)lat, (const int*)table, per_slot,
        (const int4*)items, D);
    LAUNCH_CHECK();
    return 0;
}

int gn_latent_prefill(void* stream, void* out, const void* q, const void* e,
                      const void* lat, int lat_ld, const void* meta,
                      int ntiles, const void* cos_, const void* sin_,
                      int nrot, int H, int P, int R, float scale,
                      const void* gate, int gate_ld) {
    if (ntiles < 1 || H < 1 || (R != 64 && R != 128)) return -100;
    hipStream_t st_ = (hipStream_t)stream;
    const Rotation rot{(const float*)cos_, (const float*)sin_, R / 2, nrot};
    const unsigned grid = (unsigned)((ntiles * H + 7) / 8 * 8);
#define GO(A, B) k_latent_prefill<A, B><<<grid, 256, 0, st_>>>((bf16_t*)out, \
        (const bf16_t*)q, (const bf16_t*)e, (const bf16_t*)lat, lat_ld, \
        (const int*)meta, ntiles, rot, H, scale, (const bf16_t*)gate, gate_ld)
#define PICK(B) do { if (P == 64) GO(64, B); else if (P == 128) GO(128, B); \
        else if (P == 256) GO(256, B); else return -101; } while (0)
    if (R == 64) PICK(64); else PICK(128);
#undef PICK
#undef GO
    LAUNCH_CHECK();
    return 0;
}

}  // extern "C"
