// gfx950 kernels of talking-heads attention whose values are its keys:
//   v_j            the key projection with its bias; the only thing cached
//   k_j            = rot_j(w_k * v_j / rms(v_j)), q_i likewise
//   s_g(i, j)      = cap tanh(q_g . k scale / cap)
//   seen           j <= i in the same chunk of `chunk` positions
//   p_g(i, j)      = exp(s_g) / (1 + sum_j exp(s_g))
//   out_h(i)       = sum_j (sum_g T[h, g] p_g(i, j)) v_j
// with G key/value heads for H query heads.
//
// Cache: v in pages [page][G][64][P], and 1 / rms(v) f32 [page][G][64]. Head
// sizes are padded by the host to P = 64, 128 or 256 with zeros, and a head's
// coordinates ordered so that rotated pairs are neighbours and come first.
//
// Scores are bounded by the cap, so exponents need no running maximum: they
// are taken relative to a constant `rho` (in powers of two), 0 for usual caps.
//
//  * decode (one row a sequence, short portions): one pass over v, each tile
//    read once from memory and used as keys and as values. The mixing commutes
//    with the sum over keys, so a block keeps sum_j e_g(i, j) v_j for every pair
//    of a score head and a value head, and mixes at the end, in f32.
//  * prompt portions: keys and transposed values are laid out once per step;
//    one kernel makes the denominators, the next one takes all heads of 16
//    query rows, mixes the weights of a tile by MFMA and applies them.
//  * plain: one block per row, any size; the exact mode.

#include "gridllm_tiles.h"

#include <type_traits>

typedef __attribute__((ext_vector_type(8))) _Float16 f16x8;
typedef __attribute__((ext_vector_type(4))) _Float16 f16x4;

// s in powers of two: cap tanh(x scale / cap) log2(e) = top - 2 top / (2^(rate
// x) + 1)
struct Cap {
    float rate, top, rho;
};

// `top` is c.top less what the exponent is taken relative to
DEV_INLINE float capped(float x, const Cap c, float top) {
    return top - 2.f * c.top * __builtin_amdgcn_rcpf(
        fast_exp2(x * c.rate) + 1.f);
}

// number of the wave in its block, in a scalar register: what depends on it
// alone then needs no vector registers, and its branches no masks
DEV_INLINE int wave_number() {
    return __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
}

// 8 coordinates of a key, from coordinate c of its value on
template <class T>
DEV_INLINE void key8(float* f, const T* v, float r, const float* w, int c,
                     int p, const Rotation rot) {
    float g[8];
    ld8(v, f);
    ld8(w, g);
#pragma unroll
    for (int i = 0; i < 8; ++i) f[i] *= r * g[i];
    if (c < 2 * rot.half) rotate8(f, c, p, rot);
}

// ===========================================================================
// From a projection row [H*P q | G*P k | ...], stride ld, without its bias:
// normed and rotated q [N][H][P], and the cached rows. P / 8 lanes per head.
// ===========================================================================
template <class T>
__global__ void __launch_bounds__(256)
k_talk_rows(const T* __restrict__ rows, T* __restrict__ q,
            T* __restrict__ vc, float* __restrict__ inv,
            const int* __restrict__ table, int per_slot,
            const int* __restrict__ pos, const int* __restrict__ slot,
            const float* __restrict__ bias, const float* __restrict__ qw,
            const Rotation rot, int N, int H, int G, int P, int ld_, int dim,
            float eps) {
    const int sub = P / 8;
    const long item = (blockIdx.x * 256L + threadIdx.x) / sub;
    const int n = (int)min(item / (H + G), (long)N - 1);
    const int hd = (int)(item % (H + G));
    const int c = (int)(threadIdx.x % sub) * 8;
    float f[8], g[8];
    ld8(rows + (long)n * ld_ + hd * P + c, f);
    ld8(bias + hd * P + c, g);
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        f[i] += g[i];
        ss += f[i] * f[i];
    }
    for (int off = sub / 2; off > 0; off >>= 1)
        ss += __shfl_xor(ss, off, WAVE);
    const float rs = 1.f / sqrtf(ss / (float)dim + eps);
    if (item >= (long)N * (H + G)) return;
    const int p = pos[n];
    if (hd < H) {
        ld8(qw + c, g);
#pragma unroll
        for (int i = 0; i < 8; ++i) f[i] *= rs * g[i];
        if (c < 2 * rot.half) rotate8(f, c, p, rot);
        st8(q + ((long)n * H + hd) * P + c, f);
        return;
    }
    const int blk = p / PAGE;
    if (blk >= per_slot) return;
    const long at = ((long)table[(long)slot[n] * per_slot + blk] * G + hd - H)
                    * PAGE + p % PAGE;
    st8(vc + at * P + c, f);
    if (c == 0) inv[at] = rs;
}

// the value of the lane 8 further on, in rounds of 16
DEV_INLINE float from_8_lanes_on(float x) {
    return __uint_as_float(__builtin_amdgcn_update_dpp(
        0, __float_as_uint(x), 0x128 /* row_ror:8 */, 0xf, 0xf, true));
}

// keys a query at position p sees: from here on, up to p
DEV_INLINE int first_seen(int p, int chunk) { return p / chunk * chunk; }

// tiles of 32 keys of a split
DEV_INLINE void split_tiles(int p, int chunk, int nsplit, int split, int* t0,
                            int* t1) {
    const int a = first_seen(p, chunk) >> 5, b = (p >> 5) + 1;
    const int per = (b - a + nsplit - 1) / nsplit;
    *t0 = a + split * per;
    *t1 = min(b, *t0 + per);
}

// ===========================================================================
// Decode. Block: a row and a split of its keys; tiles of 32 keys of all G value
// heads go through LDS (16-byte pieces XOR-swizzled by the row), the next one
// in flight. Scores: up to 16 heads of one value head against 16 keys are one
// item, and a wave has one or two of the same heads; the weights meet in LDS,
// and a wave then has all heads' weights against CW columns of one value head.
//   ws (nsplit > 1): sums [N][nsplit][G][H][P], and behind them the weights'
//   sums [N][nsplit][H]
// ===========================================================================
template <int P, int GP, int HB, int R>
struct DecodeShape {
    static constexpr int WAVES =
        GP > 8 ? 16 : GP * P / 16 < 8 ? GP * P / 16 : 8;
    static constexpr int CW = GP * P / WAVES;     // columns of a wave
    static constexpr int PLD = 40;
    static constexpr int TILE = GP * 32 * P;
    static_assert(P % CW == 0, "a wave has columns of one value head");
    // LDS in bytes: two tiles and weights; then in f32 sums, 1 / rms of two
    // tiles and, if it fits, the rotation of one
    static constexpr int ELEMS = 2 * TILE + HB * 16 * PLD;
    static constexpr int FIXED = ELEMS * 2 + (HB * 32 + GP * 64) * 4;
    static constexpr int TABLE = 32 * R * 4;
    static constexpr bool TAB = FIXED + TABLE <= 160 * 1024;
    static constexpr int BYTES = FIXED + (TAB ? TABLE : 0);
};

template <int P, int GP, int HB, int R>
__global__ void __launch_bounds__((DecodeShape<P, GP, HB, R>::WAVES * 64))
k_talk_decode(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
              const bf16_t* __restrict__ vc, const float* __restrict__ inv,
              const int* __restrict__ table, int per_slot,
              const int* __restrict__ pos, const int* __restrict__ slot,
              float* __restrict__ ws, const float* __restrict__ kw,
              const float* __restrict__ talk, const Rotation rot, int N,
              int H, int G, int chunk, int nsplit, const Cap cap) {
    typedef DecodeShape<P, GP, HB, R> Sh;
    constexpr int WAVES = Sh::WAVES, CW = Sh::CW, CH = P / 8;
    constexpr int NS = P / 32, RS = R / 32, NT = CW / 16, PLD = Sh::PLD;
    constexpr int LOADS = GP * 32 * CH / (WAVES * 64);
    extern __shared__ __attribute__((aligned(16))) bf16_t smem[];
    bf16_t* const pb = smem + 2 * Sh::TILE;
    float* const ls = (float*)(smem + Sh::ELEMS);   // [2][HB * 16]
    float* const ivs = ls + HB * 32;                // [2][GP][32]
    float* const tabs = ivs + GP * 64;              // cos, sin [32][R / 2]
    const int n = blockIdx.x / nsplit, split = blockIdx.x % nsplit;
    const int lane = threadIdx.x & 63, wv = wave_number();
    const int fr = lane & 15, gq = lane >> 4;
    const int rep = H / G, rbn = (rep + 15) >> 4, items = 2 * G * rbn;
    const int per = (items + WAVES - 1) / WAVES;    // 1 or 2
    const int p = min(pos[n], per_slot * PAGE - 1);
    const int lo = first_seen(p, chunk);
    int t0, t1;
    split_tiles(p, chunk, nsplit, split, &t0, &t1);
    const int* tab = table + (long)slot[n] * per_slot;

    auto issue = [&](int t, long page) {
        const bf16_t* src = vc + page * G * PAGE * P + (t & 1) * 32 * P;
        bf16_t* dst = smem + (t & 1) * Sh::TILE;
#pragma unroll
        for (int i = 0; i < LOADS; ++i) {
            const int pc = (i * WAVES + wv) * 64 + lane;
            const int kv = pc / (32 * CH), row = pc / CH % 32, c = pc % CH;
            if (kv < G)                            // the same for a wave
                load_lds16(src + ((long)kv * PAGE + row) * P +
                               (c ^ (row & 7)) * 8,
                           dst + (i * WAVES + wv) * 512);
        }
        const int kv = wv * 8 + (lane >> 3);       // 8 value heads a wave
        if (wv * 8 < GP && kv < G)
            load_lds16((const bf16_t*)(inv + (page * G + kv) * PAGE +
                                       (t & 1) * 32 + (lane & 7) * 4),
                       (bf16_t*)(ivs + (t & 1) * GP * 32 + wv * 256));
    };
    // rotation of a tile's positions; 16-byte pieces swizzled by the row
    constexpr int PIECES = R / 8, TWIST = PIECES % 8 ? 3 : 7;
    auto issue_rotation = [&](int t) {
        if (!Sh::TAB) return;
#pragma unroll
        for (int i = 0; i < (PIECES + WAVES - 1) / WAVES; ++i) {
            const int w = i * WAVES + wv, pc = w * 64 + lane;
            const int row = pc / PIECES, c = pc % PIECES;
            const float* src = row < 32 ? rot.cos_ : rot.sin_;
            if (w < PIECES)
                load_lds16((const bf16_t*)(
                               src + (long)(t * 32 + (row & 31)) * (R / 2) +
                               (c ^ (row & TWIST)) * 4),
                           (bf16_t*)(tabs + w * 256));
        }
    };
    int page = tab[min(t0, t1 - 1) >> 1];
    if (t0 < t1) {
        issue(t0, page);
        issue_rotation(t0);
        page = tab[min(t0 + 1, t1 - 1) >> 1];
    }
    // this wave's scores: up to 16 heads of one value head, 16 or 32 keys.
    // Behind the rotated part the keys' weights go into the queries.
    const int sg = min(wv * per >> 1, G * rbn - 1), kv = sg / rbn;
    const int hr = sg % rbn * 16 + fr, h = kv * rep + min(hr, rep - 1);
    const int mine = min(per, items - wv * per);
    bf16x8 qf[NS];
    float kwf[RS][8];
#pragma unroll
    for (int s = 0; s < NS; ++s) {
        const int c = s * 32 + gq * 8;
        float f[8], g[8];
        ld8(q + ((long)n * H + h) * P + c, f);
        ld8(kw + c, g);
#pragma unroll
        for (int i = 0; i < 8; ++i)
            if (s < RS) kwf[s][i] = g[i]; else f[i] *= g[i];
        qf[s] = to_bf16x8(f);
    }
    const bool few = rep <= 8;
    for (int i = threadIdx.x; i < HB * 16 * PLD / 2; i += WAVES * 64)
        ((u32*)pb)[i] = 0;
    if (threadIdx.x < HB * 32) ls[threadIdx.x] = 0.f;

    const int vh = wv * CW / P, part = wv * CW % P;   // value head, column
    float l[2] = {0.f, 0.f};
    f32x4 acc[HB][NT];
#pragma unroll
    for (int b = 0; b < HB; ++b)
#pragma unroll
        for (int c = 0; c < NT; ++c) acc[b][c] = (f32x4){0.f, 0.f, 0.f, 0.f};

    for (int t = t0; t < t1; ++t) {
        const bf16_t* tile = smem + (t & 1) * Sh::TILE;
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        lds_barrier();              // tile is there, the other one is free
        if (t + 1 < t1) issue(t + 1, page);
        page = tab[min(t + 2, t1 - 1) >> 1];
        // raw scores of 16 keys
        auto score = [&](int kb) {
            const int row = kb * 16 + fr;
            f32x4 sc = {0.f, 0.f, 0.f, 0.f};
            bf16x8 kf[NS];
#pragma unroll
            for (int s = 0; s < NS; ++s)
                kf[s] = *(const bf16x8*)(tile + (kv * 32 + row) * P +
                                         ((s * 4 + gq) ^ (row & 7)) * 8);
#pragma unroll
            for (int s = 0; s < RS; ++s) {
                const int c = s * 32 + gq * 8;
                float f[8];
#pragma unroll
                for (int i = 0; i < 8; ++i)
                    f[i] = (float)kf[s][i] * kwf[s][i];
                if (Sh::TAB) {
                    const int at = (row * PIECES + ((s * 4 + gq) ^
                                                    (row & TWIST))) * 4;
                    rotate_by(f, tabs + at, tabs + 128 * PIECES + at);
                } else {
                    rotate8(f, c, t * 32 + row, rot);
                }
                kf[s] = to_bf16x8(f);
            }
#pragma unroll
            for (int s = 0; s < NS; ++s)
                sc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[s], qf[s], sc,
                                                             0, 0, 0);
            return sc;
        };
        // weights of head hk from its scores against 16 keys
        auto weigh = [&](f32x4 sc, int kb, int hk, float* sum) {
            float e[4], iv[4];
            const int key = t * 32 + kb * 16 + gq * 4;
            ld4(ivs + (t & 1) * GP * 32 + kv * 32 + kb * 16 + gq * 4, iv);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                e[r] = fast_exp2(capped(sc[r] * iv[r], cap,
                                        cap.top - cap.rho));
                e[r] = (u32)(key + r - lo) <= (u32)(p - lo) ? e[r] : 0.f;
                *sum += e[r];
            }
            if (hk < rep)
                *(uint2*)(pb + (kv * rep + hk) * PLD + kb * 16 + gq * 4) =
                    make_uint2(pack2(e[0], e[1]), pack2(e[2], e[3]));
        };
        if (mine == 2) {
            f32x4 a = score(0);
            const f32x4 b = score(1);
            if (few) {            // the second 16 keys into idle lanes
#pragma unroll
                for (int r = 0; r < 4; ++r) {
                    const float x = from_8_lanes_on(b[r]);
                    a[r] = fr < 8 ? a[r] : x;
                }
                weigh(a, fr >> 3, fr & 7, l);
            } else {
                weigh(a, 0, hr, l);
                weigh(b, 1, hr, l + 1);
            }
        } else if (mine == 1) {
            weigh(score(wv & 1), wv & 1, hr, l);
        }
        lds_barrier();              // weights are there
        if (t + 1 < t1) issue_rotation(t + 1);
        if (vh >= G) continue;
        bf16x8 pf[HB];
#pragma unroll
        for (int b = 0; b < HB; ++b)
            pf[b] = *(const bf16x8*)(pb + (b * 16 + fr) * PLD + gq * 8);
#pragma unroll
        for (int c = 0; c < NT; ++c) {
            const int d = part + c * 16 + (fr & 3) * 4;
            bf16x8 v;
#pragma unroll
            for (int j = 0; j < 2; ++j) {
                const int row = gq * 8 + (fr >> 2) + j * 4;
                const bf16x4 x = read_transposed(
                    tile + (vh * 32 + row) * P + ((d >> 3) ^ (row & 7)) * 8 +
                    (d & 7));
#pragma unroll
                for (int i = 0; i < 4; ++i) v[j * 4 + i] = x[i];
            }
#pragma unroll
            for (int b = 0; b < HB; ++b)
                acc[b][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                    pf[b], v, acc[b][c], 0, 0, 0);
        }
    }
    lds_barrier();                  // ls is cleared, also without a tile
    if (mine > 0) {
        float s[2] = {l[0], l[1]};
#pragma unroll
        for (int i = 0; i < 2; ++i) {
            s[i] += __shfl_xor(s[i], 16, WAVE);
            s[i] += __shfl_xor(s[i], 32, WAVE);
        }
        if (few && mine == 2) s[1] = from_8_lanes_on(s[0]);
        if (gq == 0 && hr < rep) {
            ls[(mine == 1 ? wv & 1 : 0) * HB * 16 + h] = s[0];
            if (mine == 2) ls[HB * 16 + h] = s[1];
        }
    }
    __syncthreads();
    if (nsplit > 1) {
        const long at = (long)n * nsplit + split;
        float* wl = ws + (long)N * nsplit * G * H * P + at * H;
        for (int h = threadIdx.x; h < H; h += WAVES * 64)
            wl[h] = ls[h] + ls[HB * 16 + h];
        if (vh >= G || t0 >= t1) return;
        float* wo = ws + (at * G + vh) * H * P + part + fr;
#pragma unroll
        for (int b = 0; b < HB; ++b)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int g = b * 16 + gq * 4 + r;
                if (g < H)
#pragma unroll
                    for (int c = 0; c < NT; ++c)
                        wo[g * P + c * 16] = acc[b][c][r];
            }
        return;
    }
    if (vh >= G) return;
    float nrm[HB][4];
#pragma unroll
    for (int b = 0; b < HB; ++b)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int g = b * 16 + gq * 4 + r;
            nrm[b][r] = 1.f / (exp2f(-cap.rho) + ls[g] + ls[HB * 16 + g]);
        }
    for (int i = 0; i < rep; ++i) {
        const int h = vh * rep + i;
        float o[NT];
#pragma unroll
        for (int c = 0; c < NT; ++c) o[c] = 0.f;
#pragma unroll
        for (int b = 0; b < HB; ++b)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int g = b * 16 + gq * 4 + r;
                const float x = g < H ? talk[h * H + g] * nrm[b][r] : 0.f;
#pragma unroll
                for (int c = 0; c < NT; ++c) o[c] += x * acc[b][c][r];
            }
#pragma unroll
        for (int c = 0; c < NT; ++c) {
            o[c] += __shfl_xor(o[c], 16, WAVE);
            o[c] += __shfl_xor(o[c], 32, WAVE);
            if (gq == 0)
                out[((long)n * H + h) * P + part + c * 16 + fr] = f2bf(o[c]);
        }
    }
}

// Splits of a row added up, normalised and mixed. Block: a row, a value head,
// 32 columns; 256 threads are 32 score heads by 8 x 4 columns. H <= 64.
__global__ void __launch_bounds__(256)
k_talk_combine(bf16_t* __restrict__ out, const float* __restrict__ ws,
               const float* __restrict__ talk, const int* __restrict__ pos,
               int per_slot, int N, int H, int G, int P, int chunk,
               int nsplit, float rho) {
    __shared__ __attribute__((aligned(16))) float red[4][4][32];
    __shared__ float nrm[64];
    const int n = blockIdx.x, kv = blockIdx.y, rep = H / G;
    const int c0 = blockIdx.z * 32, tid = threadIdx.x;
    const int c = c0 + (tid & 7) * 4, g0 = tid >> 3;
    const int p = min(pos[n], per_slot * PAGE - 1);
    int t0, t1, live = 0;              // splits that have keys come first
    for (; live < nsplit; ++live) {
        split_tiles(p, chunk, nsplit, live, &t0, &t1);
        if (t0 >= t1) break;
    }
    constexpr int U = 8;               // rows in flight
    const float* wl = ws + (long)N * nsplit * G * H * P + (long)n * nsplit * H;
    if (tid < H) {
        float l = exp2f(-rho);
        for (int s0 = 0; s0 < live; s0 += U) {
            float f[U];
#pragma unroll
            for (int u = 0; u < U; ++u)
                f[u] = wl[min(s0 + u, live - 1) * H + tid];
#pragma unroll
            for (int u = 0; u < U; ++u) l += s0 + u < live ? f[u] : 0.f;
        }
        nrm[tid] = 1.f / l;
    }
    float o[2][4] = {};
#pragma unroll
    for (int k = 0; k < 2; ++k) {
        const int g = g0 + k * 32;
        if (g >= H) break;
        const float* src = ws + (((long)n * nsplit * G + kv) * H + g) * P + c;
        for (int s0 = 0; s0 < live; s0 += U) {
            float f[U][4];
#pragma unroll
            for (int u = 0; u < U; ++u)
                ld4(src + (long)min(s0 + u, live - 1) * G * H * P, f[u]);
#pragma unroll
            for (int u = 0; u < U; ++u)
                if (s0 + u < live)
#pragma unroll
                    for (int j = 0; j < 4; ++j) o[k][j] += f[u][j];
        }
    }
    for (int i0 = 0; i0 < rep; i0 += 4) {
        __syncthreads();               // nrm is there, red is free
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            float a[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < 2; ++k) {
                const int g = g0 + k * 32;
                if (g >= H || i0 + i >= rep) continue;
                const float x = talk[(kv * rep + i0 + i) * H + g] * nrm[g];
#pragma unroll
                for (int j = 0; j < 4; ++j) a[j] += x * o[k][j];
            }
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
                for (int off = 8; off < 64; off <<= 1)
                    a[j] += __shfl_xor(a[j], off, WAVE);
            if ((tid & 63) < 8) st4(&red[tid >> 6][i][(tid & 7) * 4], a);
        }
        __syncthreads();
        const int i = tid >> 5, d = tid & 31;
        if (i < 4 && i0 + i < rep)
            out[((long)n * H + kv * rep + i0 + i) * P + c0 + d] =
                f2bf(red[0][i][d] + red[1][i][d] + red[2][i][d] + red[3][i][d]);
    }
}

// ===========================================================================
// Keys [page][G][64][P] and transposed values [page][G][P][64] of the pages
// that a step's portions see. Item (int4): {page number within the sequence,
// slot, page of kx and vx, rows}; rows from there on become zero.
// ===========================================================================
__global__ void __launch_bounds__(256)
k_talk_gather(bf16_t* __restrict__ kx, bf16_t* __restrict__ vx,
              const bf16_t* __restrict__ vc, const float* __restrict__ inv,
              const int* __restrict__ table, int per_slot,
              const float* __restrict__ kw, const Rotation rot,
              const int4* __restrict__ items, int G, int P) {
    __shared__ __attribute__((aligned(16))) bf16_t tile[256 * 72];
    const int4 it = items[blockIdx.x];
    const int kv = blockIdx.y, ch = P / 8;
    const long src =
        ((long)table[(long)it.y * per_slot + it.x] * G + kv) * PAGE;
    const long dst = ((long)it.z * G + kv) * PAGE * P;
    // a wave takes the same 8 columns of 64 rows: column-wise LDS stores of
    // neighbouring rows
    for (int i = threadIdx.x; i < PAGE * ch; i += 256) {
        const int row = i % PAGE, c = i / PAGE * 8;
        uint4 v = make_uint4(0, 0, 0, 0), k = v;
        if (row < it.w) {
            const bf16_t* s = vc + (src + row) * P + c;
            float f[8];
            v = *(const uint4*)s;
            key8(f, s, inv[src + row], kw + c, c, it.x * PAGE + row, rot);
            k = pack8(f);
        }
        *(uint4*)(kx + dst + (long)row * P + c) = k;
        const u32 w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
        for (int j = 0; j < 8; ++j)
            tile[(c + j) * 72 + row] = (bf16_t)(w[j >> 1] >> (j & 1) * 16);
    }
    __syncthreads();
    for (int i = threadIdx.x; i < PAGE * ch; i += 256) {
        const int d = i / 8, c = i % 8 * 8;
        *(uint4*)(vx + dst + (long)d * PAGE + c) =
            *(const uint4*)(tile + d * 72 + c);
    }
}

// A portion's rows: {first token, length, page of kx at which its keys begin,
// first row of the tile, start position, page number of that page, 0, 0}
struct Tile {
    int off, len, page, q0, start, page0;
    DEV_INLINE Tile(const int* m)
        : off(m[0]), len(m[1]), page(m[2]), q0(m[3]), start(m[4]),
          page0(m[5]) {}
    // page of kx that holds position k
    DEV_INLINE long at(int k) const { return page + (k >> 6) - page0; }
};

// ===========================================================================
// lse[n][h] = log2(1 + sum_j exp(s_h(n, j))). Block: 128 rows of a portion, a
// head; a wave owns 32 rows. S^T = K Q^T puts a row's scores into a lane pair.
// ===========================================================================
template <int P>
__global__ void __launch_bounds__(256, 2)
k_talk_lse(float* __restrict__ lse, const bf16_t* __restrict__ q,
           const bf16_t* __restrict__ kx, const int* __restrict__ meta,
           int ntiles, int H, int G, int chunk, const Cap cap) {
    constexpr int NS = P / 16, CH = P / 8, LOADS = 32 * CH / 256;
    __shared__ __attribute__((aligned(16))) bf16_t tile[2][32 * P];
    // neighbouring work (tiles of one head) on the same XCD, longest first
    const int total = ntiles * H, per = (total + 7) >> 3;
    const int i0 = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per || i0 >= total) return;
    const int h = i0 / ntiles, kv = h / (H / G);
    const Tile tl(meta + (i0 % ntiles) * 8);
    const int lane = threadIdx.x & 63, wid = wave_number();
    const int hi = lane >> 5, ln = lane & 31;
    const int qw = min(tl.q0 + wid * 32, tl.len - 1);   // (a wave without rows
    const int qrow = min(qw + ln, tl.len - 1);          // repeats the last)
    const int qa = tl.start + qrow, qlo = first_seen(qa, chunk);
    const int first = tl.start + qw, last = tl.start + min(qw + 31, tl.len - 1);
    const int all_lo = first_seen(last, chunk);     // seen by every row
    const int wave_lo = first_seen(first, chunk);
    bf16x8 qf[NS];
    const bf16_t* qr = q + ((long)(tl.off + qrow) * H + h) * P + hi * 8;
#pragma unroll
    for (int s = 0; s < NS; ++s) qf[s] = *(const bf16x8*)(qr + s * 16);
    auto issue = [&](int k0) {
        const bf16_t* src = kx + ((tl.at(k0) * G + kv) * PAGE + (k0 & 63)) * P;
#pragma unroll
        for (int i = 0; i < LOADS; ++i) {
            const int pc = i * 256 + threadIdx.x;
            const int row = pc / CH, c = pc % CH;
            load_lds16(src + row * P + (c ^ (row & 7)) * 8,
                       tile[(k0 >> 5) & 1] + (i * 256 + wid * 64) * 8);
        }
    };
    const int begin = first_seen(tl.start + tl.q0, chunk) & ~31;
    const int end = tl.start + min(tl.q0 + 127, tl.len - 1);
    const float top = cap.top - cap.rho;
    float l = 0.f;
    issue(begin);
    for (int k0 = begin; k0 <= end; k0 += 32) {
        const bf16_t* kt = tile[(k0 >> 5) & 1];
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        lds_barrier();              // tile is there, the other one is free
        if (k0 + 32 <= end) issue(k0 + 32);
        if (k0 > last || k0 + 31 < wave_lo) continue;
        f32x16 sv;
#pragma unroll
        for (int r = 0; r < 16; ++r) sv[r] = 0.f;
#pragma unroll
        for (int s = 0; s < NS; ++s)
            sv = __builtin_amdgcn_mfma_f32_32x32x16_bf16(
                *(const bf16x8*)(kt + ln * P +
                                 ((s * 2 + hi) ^ (ln & 7)) * 8),
                qf[s], sv, 0, 0, 0);
        if (k0 >= all_lo && k0 + 31 <= first) {
#pragma unroll
            for (int r = 0; r < 16; ++r)
                l += fast_exp2(capped(sv[r], cap, top));
        } else {
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const int key = k0 + (r & 3) + 8 * (r >> 2) + 4 * hi;
                const float e = fast_exp2(capped(sv[r], cap, top));
                l += key >= qlo && key <= qa ? e : 0.f;
            }
        }
    }
    l += __shfl_xor(l, 32, WAVE);
    if (hi == 0 && tl.q0 + wid * 32 + ln < tl.len)
        lse[(long)(tl.off + qrow) * H + h] =
            cap.rho + log2f(exp2f(-cap.rho) + l);
}

// ===========================================================================
// Mixed weights times values. Block: 16 rows of a portion, all heads; wave w
// has heads w * NH .. + NH - 1, which are numbered w * 4 + 0 .. NH - 1 where
// heads are a matrix dimension. Per 32 keys: a wave makes its heads' weights
// (f16, times 2^14) and leaves them in LDS; one MFMA mixes 16 keys of a row for
// 16 output heads; each wave applies its heads' mixed weights. The three steps
// work on three successive tiles between two barriers.
// Weights are normalised, so parts of a row's keys (grid y) just add up.
//   talk: f16 [32][32] in that numbering; fin: factor of the result
//   ws: null, or f32 [parts][rows][H][P] from token `row0` on
//   SAME: the heads of a wave share a value head
// ===========================================================================
#define LIFT 14.f

template <int P, int NH, bool SAME>
__global__ void __launch_bounds__(512, 2)
k_talk_prefill(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
               const bf16_t* __restrict__ kx, const bf16_t* __restrict__ vx,
               const float* __restrict__ lse, const _Float16* __restrict__ talk,
               const int* __restrict__ meta, int H, int G, int chunk,
               const Cap cap, float fin, float* __restrict__ ws, int row0,
               int rows) {
    constexpr int NS = P / 32, NT = P / 16;
    // a row of 32, and 32 or 16 such rows, padded against bank conflicts
    constexpr int LDR = 36, QS = 32 * LDR + 4, HS = 16 * LDR + 4;
    __shared__ __attribute__((aligned(16))) _Float16 pb[2][16 * QS];
    __shared__ __attribute__((aligned(16))) bf16_t wb[2][32 * HS];
    __shared__ __attribute__((aligned(16))) _Float16 tb[2 * 512];
    const Tile tl(meta + (long)blockIdx.x * 8);
    if (tl.len <= tl.q0) return;              // the same for the block
    const int lane = threadIdx.x & 63, wv = wave_number();
    const int fr = lane & 15, gq = lane >> 4, rep = H / G;
    const int nq = min(16, tl.len - tl.q0);
    const int row = tl.off + tl.q0 + min(fr, nq - 1);
    const int first = tl.start + tl.q0, last = first + nq - 1;
    const int qa = first + min(fr, nq - 1), qlo = first_seen(qa, chunk);
    const int all_lo = first_seen(last, chunk);
    const int h0 = wv * NH;
    const bool two = (H + NH - 1) / NH > 4;   // numbers above 16 occur

    bf16x8 qf[NH][NS], kf[2][NS], vf[NT];
    float ls[NH];
    f32x4 acc[NH][NT];
#pragma unroll
    for (int i = 0; i < NH; ++i) {
        const int h = min(h0 + i, H - 1);
        ls[i] = cap.top - lse[(long)row * H + h] + LIFT;
        const bf16_t* qr = q + ((long)row * H + h) * P + gq * 8;
#pragma unroll
        for (int s = 0; s < NS; ++s) qf[i][s] = *(const bf16x8*)(qr + s * 32);
#pragma unroll
        for (int t = 0; t < NT; ++t) acc[i][t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    }
    for (int i = threadIdx.x; i < 512; i += 512)   // in MFMA operand order
        ((u32*)tb)[i] = ((const u32*)talk)[(i >> 8) * 256 + (i & 3) +
                                           (i >> 2 & 15) * 16 +
                                           (i >> 6 & 3) * 4];

    auto load_k = [&](int kv, int k0, int b) {        // 16 keys
        const bf16_t* kr = kx + ((tl.at(k0) * G + kv) * PAGE + (k0 & 63) +
                                 b * 16 + fr) * P + gq * 8;
#pragma unroll
        for (int s = 0; s < NS; ++s) kf[b][s] = *(const bf16x8*)(kr + s * 32);
    };
    auto load_v = [&](int kv, int k0) {
        const bf16_t* vr = vx + ((tl.at(k0) * G + kv) * P + fr) * PAGE +
                           (k0 & 63) + gq * 8;
#pragma unroll
        for (int t = 0; t < NT; ++t)
            vf[t] = *(const bf16x8*)(vr + t * 16 * PAGE);
    };
    const int start = first_seen(first, chunk) & ~31;
    const int tiles = (last - start) / 32 + 1;
    const int per = (tiles + gridDim.y - 1) / gridDim.y * 32;
    const int begin = start + blockIdx.y * per;
    const int tail = min(last & ~31, begin + per - 32);
    // value head of a wave's head (the last head stands in for missing ones:
    // their column of talk is zero, and nobody stores their result)
    auto value_head = [&](int i) { return min(h0 + i, H - 1) / rep; };
    auto other = [&](int i) {                 // not the head's before
        return !SAME && (i == 0 || value_head(i) != value_head(i - 1));
    };
    const int kv0 = value_head(0), now0 = (begin >> 5) & 1;
    for (int i = threadIdx.x; i < 8 * QS; i += 512) ((u32*)pb[now0 ^ 1])[i] = 0;
    for (int i = threadIdx.x; i < 16 * HS; i += 512) ((u32*)wb[now0])[i] = 0;
    if (SAME && begin <= tail) load_v(kv0, begin);
    lds_barrier();
    // Tile k0: weights; tile k0 - 32: mixing; tile k0 - 64: values. Where there
    // is no such tile the weights are zero. Keys take over the registers of
    // the values.
    for (int k0 = begin; k0 <= tail + 64 && begin <= tail; k0 += 32) {
        const int now = (k0 >> 5) & 1, kt = min(k0, tail);
        bf16x8 w[NH];
#pragma unroll
        for (int i = 0; i < NH; ++i) {
            const bf16_t* wr =
                wb[now] + (wv * 4 + i) * HS + fr * LDR + gq * 8;
            w[i] = __builtin_shufflevector(
                *(const bf16x4*)wr, *(const bf16x4*)(wr + 4), 0, 1, 2, 3, 4, 5,
                6, 7);
        }
        if (SAME) {
#pragma unroll
            for (int b = 0; b < 2; ++b) {
#pragma unroll
                for (int t = b * NT / 2; t < (b + 1) * NT / 2; ++t)
#pragma unroll
                    for (int i = 0; i < NH; ++i)
                        acc[i][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                            vf[t], w[i], acc[i][t], 0, 0, 0);
                load_k(kv0, kt, b);
            }
        } else {
#pragma unroll
            for (int i = 0; i < NH; ++i) {
                if (other(i)) load_v(value_head(i), max(k0 - 64, begin));
#pragma unroll
                for (int t = 0; t < NT; ++t)
                    acc[i][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                        vf[t], w[i], acc[i][t], 0, 0, 0);
            }
        }
        u32 pw[8][2] = {};                    // heads 0 | 1 and 2 | 3
        const int base = k0 + gq * 4 - qlo;   // from the first key seen
        const u32 until = k0 <= tail ? qa - qlo + 1 : 0;
        auto weights = [&](auto whole) {
#pragma unroll
            for (int i = 0; i < NH; ++i) {
                if (other(i)) {
                    load_k(value_head(i), kt, 0);
                    load_k(value_head(i), kt, 1);
                }
                f32x4 sc[2];
#pragma unroll
                for (int b = 0; b < 2; ++b) {
                    sc[b] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
                    for (int s = 0; s < NS; ++s)
                        sc[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                            kf[b][s], qf[i][s], sc[b], 0, 0, 0);
                }
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    float e =
                        fast_exp2(capped(sc[j >> 2][j & 3], cap, ls[i]));
                    if (!decltype(whole)::value)
                        e = (u32)(base + (j >> 2) * 16 + (j & 3)) < until
                                ? e : 0.f;
                    const u32 x = __builtin_bit_cast(unsigned short,
                                                     (_Float16)e);
                    pw[j][i >> 1] |= i & 1 ? x << 16 : x;
                }
            }
        };
        if (k0 >= all_lo && k0 + 31 <= first && k0 <= tail)
            weights(std::true_type{});
        else
            weights(std::false_type{});
#pragma unroll
        for (int j = 0; j < 8; ++j)
            *(uint2*)(pb[now] + fr * QS +
                      ((j >> 2) * 16 + gq * 4 + (j & 3)) * LDR + wv * 4) =
                make_uint2(pw[j][0], pw[j][1]);
        if (SAME)                             // for the next turn
            load_v(kv0, min(max(k0 - 32, begin), tail));
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int qi = wv * 2 + (j >> 1), kb = (j & 1) * 16;
            const _Float16* ar =
                pb[now ^ 1] + qi * QS + (kb + fr) * LDR + gq * 8;
            const f16x8 a = __builtin_shufflevector(
                *(const f16x4*)ar, *(const f16x4*)(ar + 4), 0, 1, 2, 3, 4, 5,
                6, 7);
#pragma unroll
            for (int b = 0; b < 2; ++b)
                if (b == 0 || two) {
                    const f32x4 c = __builtin_amdgcn_mfma_f32_16x16x32_f16(
                        a, *(const f16x8*)(tb + b * 512 + lane * 8),
                        (f32x4){0.f, 0.f, 0.f, 0.f}, 0, 0, 0);
                    *(uint2*)(wb[now ^ 1] + (b * 16 + fr) * HS + qi * LDR +
                              kb + gq * 4) =
                        make_uint2(pack2(c[0], c[1]), pack2(c[2], c[3]));
                }
        }
        lds_barrier();
    }
    if (fr >= nq) return;
#pragma unroll
    for (int i = 0; i < NH; ++i)
        if (h0 + i < H && ws) {
            float* o = ws + (((long)blockIdx.y * rows + row - row0) * H + h0 +
                             i) * P + gq * 4;
#pragma unroll
            for (int t = 0; t < NT; ++t)
                *(f32x4*)(o + t * 16) = acc[i][t] * fin;
        } else if (h0 + i < H) {
            bf16_t* o = out + ((long)row * H + h0 + i) * P + gq * 4;
#pragma unroll
            for (int t = 0; t < NT; ++t)
                *(uint2*)(o + t * 16) = make_uint2(
                    pack2(acc[i][t][0] * fin, acc[i][t][1] * fin),
                    pack2(acc[i][t][2] * fin, acc[i][t][3] * fin));
        }
}

// out = the sum of `parts` f32 rows [parts][n], 4 elements a thread
__global__ void __launch_bounds__(256)
k_talk_add(bf16_t* __restrict__ out, const float* __restrict__ ws, long n,
           int parts) {
    const long i = (blockIdx.x * 256L + threadIdx.x) * 4;
    if (i >= n) return;
    float a[4];
    ld4(ws + i, a);
    for (int s = 1; s < parts; ++s) {
        float b[4];
        ld4(ws + s * n + i, b);
#pragma unroll
        for (int j = 0; j < 4; ++j) a[j] += b[j];
    }
    st4(out + i, a);
}

// ===========================================================================
// Plain: one block per row, any sizes that fit LDS, two passes over the keys
// (denominators, then weights). Exponents relative to a running maximum that
// starts at the sink's 0. The exact mode, and bf16 for sizes or caps that the
// kernels above do not take.
//   LDS (f32): q [H][P], sums [H][P], keys [16][P], scores and mixed weights
//   [H][16], maximum and denominator [H]
// ===========================================================================
template <class T>
__global__ void __launch_bounds__(256)
k_talk_plain(T* __restrict__ out, const T* __restrict__ q,
             const T* __restrict__ vc, const float* __restrict__ inv,
             const int* __restrict__ table, int per_slot,
             const int* __restrict__ pos, const int* __restrict__ slot,
             const float* __restrict__ kw, const float* __restrict__ talk,
             const Rotation rot, int H, int G, int P, int chunk, float scale,
             float cap) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    float* const qs = sm;
    float* const os = qs + H * P;
    float* const ks = os + H * P;
    float* const sc = ks + 16 * P;
    float* const wt = sc + H * 16;
    float* const mx = wt + H * 16;
    float* const dn = mx + H;
    const int n = blockIdx.x, tid = threadIdx.x, rep = H / G;
    const int p = min(pos[n], per_slot * PAGE - 1);
    const int lo = first_seen(p, chunk);
    const int* tab = table + (long)slot[n] * per_slot;
    for (int i = tid; i < H * P; i += 256) {
        qs[i] = ld(q + (long)n * H * P + i);
        os[i] = 0.f;
    }
    for (int h = tid; h < H; h += 256) {
        mx[h] = 0.f;
        dn[h] = 1.f;
    }
    auto row_at = [&](int kv, int k) {
        return ((long)tab[k / PAGE] * G + kv) * PAGE + k % PAGE;
    };
    for (int pass = 0; pass < 2; ++pass)
        for (int k0 = lo; k0 <= p; k0 += 16) {
            const int nk = min(16, p + 1 - k0);
            for (int kv = 0; kv < G; ++kv) {
                __syncthreads();
                for (int i = tid; i < nk * P / 8; i += 256) {
                    const int k = i / (P / 8), c = i % (P / 8) * 8;
                    const long r = row_at(kv, k0 + k);
                    float f[8];
                    key8(f, vc + r * P + c, inv[r], kw + c, c, k0 + k, rot);
                    st8(ks + k * P + c, f);
                }
                __syncthreads();
                for (int i = tid >> 2; i < rep * 16; i += 64) {
                    const int h = kv * rep + i / 16, k = min(i % 16, nk - 1);
                    float s = 0.f;
                    for (int c = tid & 3; c < P; c += 4)
                        s += qs[h * P + c] * ks[k * P + c];
                    s += __shfl_xor(s, 1, WAVE);
                    s += __shfl_xor(s, 2, WAVE);
                    if ((tid & 3) == 0)
                        sc[h * 16 + i % 16] = i % 16 < nk
                            ? cap * tanhf(s * scale / cap) : -INFINITY;
                }
            }
            __syncthreads();
            if (pass == 0) {
                for (int h = tid; h < H; h += 256) {
                    float m = mx[h];
                    for (int k = 0; k < nk; ++k)
                        m = fmaxf(m, sc[h * 16 + k]);
                    float l = dn[h] * expf(mx[h] - m);
                    for (int k = 0; k < nk; ++k)
                        l += expf(sc[h * 16 + k] - m);
                    mx[h] = m;
                    dn[h] = l;
                }
                continue;
            }
            for (int i = tid; i < H * 16; i += 256)
                sc[i] = expf(sc[i] - mx[i / 16]) / dn[i / 16];
            __syncthreads();
            for (int i = tid; i < H * 16; i += 256) {
                float w = 0.f;
                for (int g = 0; g < H; ++g)
                    w += talk[i / 16 * H + g] * sc[g * 16 + i % 16];
                wt[i] = w;
            }
            __syncthreads();
            for (int i = tid; i < H * P; i += 256) {
                const int h = i / P;
                float o = os[i];
                for (int k = 0; k < nk; ++k)
                    o += wt[h * 16 + k] *
                         ld(vc + row_at(h / rep, k0 + k) * P + i % P);
                os[i] = o;
            }
        }
    for (int i = tid; i < H * P; i += 256)
        st(out + (long)n * H * P + i, os[i]);
}

// ===========================================================================
// Entry points. f32 != 0 selects the exact mode. 0 = success.
// ===========================================================================
static Rotation rotation(const void* cos_, const void* sin_, int R, int nrot) {
    return Rotation{(const float*)cos_, (const float*)sin_, R / 2, nrot};
}

static bool sizes_ok(int H, int G, int P, int R, int nrot, int chunk) {
    return H > 0 && G > 0 && H % G == 0 &&
           (P == 64 || P == 128 || P == 256) && R % 8 == 0 && R >= 0 &&
           R <= P && nrot > 0 && chunk > 0;
}

// A kernel with more LDS than the default limit asks for it, once.
template <auto Kernel>
static int allow_lds(int bytes) {
    static bool done = false;
    if (done) return 0;
    const hipError_t e = hipFuncSetAttribute(
        (const void*)Kernel, hipFuncAttributeMaxDynamicSharedMemorySize,
        bytes);
    done = e == hipSuccess;
    return (int)e;
}

template <int P, int GP, int HB, int R>
static int go_decode(hipStream_t st, bf16_t* out, const bf16_t* q,
                     const bf16_t* vc, const float* inv, const int* table,
                     int per_slot, const int* pos, const int* slot, float* ws,
                     const float* kw, const float* talk, const Rotation rot,
                     int N, int H, int G, int chunk, int nsplit,
                     const Cap cap) {
    typedef DecodeShape<P, GP, HB, R> Sh;
    if (Sh::BYTES > 160 * 1024) return -102;
    const int e = allow_lds<k_talk_decode<P, GP, HB, R>>(Sh::BYTES);
    if (e) return e;
    k_talk_decode<P, GP, HB, R><<<N * nsplit, Sh::WAVES * 64, Sh::BYTES, st>>>(
        out, q, vc, inv, table, per_slot, pos, slot, ws, kw, talk, rot, N, H,
        G, chunk, nsplit, cap);
    LAUNCH_CHECK();
    if (nsplit > 1) {
        k_talk_combine<<<dim3(N, G, P / 32), 256, 0, st>>>(
            out, ws, talk, pos, per_slot, N, H, G, P, chunk, nsplit, cap.rho);
        LAUNCH_CHECK();
    }
    return 0;
}

extern "C" {

int gt_talk_rows(void* stream, int f32, const void* rows, void* q, void* vc,
                 void* inv, const void* table, int per_slot, const void* pos,
                 const void* slot, const void* bias, const void* qw,
                 const void* cos_, const void* sin_, int nrot, int N, int H,
                 int G, int P, int R, int ld_, int dim, float eps) {
    if (N < 1 || !sizes_ok(H, G, P, R, nrot, 1) || dim < 1 || dim > P ||
        ld_ < (H + G) * P || ld_ % 8) return -100;
    const Rotation rot = rotation(cos_, sin_, R, nrot);
    const long threads = (long)N * (H + G) * (P / 8);
#define GO(T) k_talk_rows<T><<<(unsigned)((threads + 255) / 256), 256, 0, \
        (hipStream_t)stream>>>((const T*)rows, (T*)q, (T*)vc, (float*)inv, \
        (const int*)table, per_slot, (const int*)pos, (const int*)slot, \
        (const float*)bias, (const float*)qw, rot, N, H, G, P, ld_, dim, eps)
    if (f32) GO(float); else GO(bf16_t);
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gt_talk_decode(void* stream, void* out, const void* q, const void* vc,
                   const void* inv, const void* table, int per_slot,
                   const void* pos, const void* slot, void* ws,
                   const void* kw, const void* talk, const void* cos_,
                   const void* sin_, int nrot, int N, int H, int G, int P,
                   int R, int chunk, int nsplit, float rate, float top,
                   float rho) {
    if (N < 1 || !sizes_ok(H, G, P, R, nrot, chunk) || nsplit < 1 ||
        nsplit > 64 || H > 64 || G * P > 1024 ||
        nrot < per_slot * PAGE ||
        (nsplit > 1 && !ws)) return -100;
    const Rotation rot = rotation(cos_, sin_, R, nrot);
    const Cap cap{rate, top, rho};
#define GO(A, B, C, D) return go_decode<A, B, C, D>((hipStream_t)stream, \
        (bf16_t*)out, (const bf16_t*)q, (const bf16_t*)vc, \
        (const float*)inv, (const int*)table, per_slot, (const int*)pos, \
        (const int*)slot, (float*)ws, (const float*)kw, (const float*)talk, \
        rot, N, H, G, chunk, nsplit, cap)
#define HEADS(A, B, D) do { if (H <= 16) GO(A, B, 1, D); \
        else if (H <= 32) GO(A, B, 2, D); else GO(A, B, 4, D); } while (0)
#define VALUES(A, D) do { if (G == 1) HEADS(A, 1, D); \
        else if (G == 2) HEADS(A, 2, D); \
        else if (G <= 4) HEADS(A, 4, D); \
        else if (G <= 8 && A <= 128) HEADS(A, A <= 128 ? 8 : 4, D); \
        else if (A == 64) HEADS(A, A == 64 ? 16 : 4, D); } while (0)
    if (P == 64 && R == 32) VALUES(64, 32);
    if (P == 64 && R == 64) VALUES(64, 64);
    if (P == 128 && R == 32) VALUES(128, 32);
    if (P == 128 && R == 64) VALUES(128, 64);
    if (P == 128 && R == 128) VALUES(128, 128);
    if (P == 256 && R == 64) VALUES(256, 64);
    if (P == 256 && R == 256) VALUES(256, 256);
#undef VALUES
#undef HEADS
#undef GO
    return -101;
}

int gt_talk_gather(void* stream, void* kx, void* vx, const void* vc,
                   const void* inv, const void* table, int per_slot,
                   const void* kw, const void* cos_, const void* sin_,
                   int nrot, const void* items, int nitems, int G, int P,
                   int R) {
    if (nitems < 1 || !sizes_ok(G, G, P, R, nrot, 1)) return -100;
    k_talk_gather<<<dim3(nitems, G), 256, 0, (hipStream_t)stream>>>(
        (bf16_t*)kx, (bf16_t*)vx, (const bf16_t*)vc, (const float*)inv,
        (const int*)table, per_slot, (const float*)kw,
        rotation(cos_, sin_, R, nrot), (const int4*)items, G, P);
    LAUNCH_CHECK();
    return 0;
}

int gt_talk_lse(void* stream, void* lse, const void* q, const void* kx,
                const void* meta, int ntiles, int H, int G, int P, int chunk,
                float rate, float top, float rho) {
    if (ntiles < 1 || !sizes_ok(H, G, P, 0, 1, chunk)) return -100;
    const unsigned grid = (unsigned)(((long)ntiles * H + 7) / 8 * 8);
#define GO(A) k_talk_lse<A><<<grid, 256, 0, (hipStream_t)stream>>>( \
        (float*)lse, (const bf16_t*)q, (const bf16_t*)kx, (const int*)meta, \
        ntiles, H, G, chunk, Cap{rate, top, rho})
    if (P == 64) GO(64); else if (P == 128) GO(128); else GO(256);
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gt_talk_prefill(void* stream, void* out, const void* q, const void* kx,
                    const void* vx, const void* lse, const void* talk,
                    const void* meta, int ntiles, int H, int G, int P,
                    int chunk, float rate, float top, float rho, float fin,
                    void* ws, int parts, int row0, int rows) {
    const int nh = (H + 7) / 8;
    if (ntiles < 1 || !sizes_ok(H, G, P, 0, 1, chunk) || nh > 4 ||
        nh * P > 512 || parts < 1 || (parts > 1) != !!ws || row0 < 0 ||
        rows < 1) return -100;
#define GO1(A, B, C) k_talk_prefill<A, B, C><<<dim3(ntiles, parts), 512, 0, \
        (hipStream_t)stream>>>((bf16_t*)out, (const bf16_t*)q, \
        (const bf16_t*)kx, (const bf16_t*)vx, (const float*)lse, \
        (const _Float16*)talk, (const int*)meta, H, G, chunk, \
        Cap{rate, top, rho}, fin, (float*)ws, row0, rows)
#define GO(A, B) do { if (H / G % B == 0) GO1(A, B, true); \
        else GO1(A, B, false); } while (0)
#define PICK(A) do { if (nh == 1) GO(A, 1); else if (nh == 2) GO(A, 2); \
        else if (nh == 3) GO(A, 3); else GO(A, 4); } while (0)
    if (P == 64) PICK(64);
    else if (P == 128) PICK(128);
    else if (nh == 1) GO(256, 1);
    else GO(256, 2);
#undef PICK
#undef GO
#undef GO1
    LAUNCH_CHECK();
    if (parts > 1) {
        const long n = (long)rows * H * P;
        k_talk_add<<<(unsigned)((n / 4 + 255) / 256), 256, 0,
                     (hipStream_t)stream>>>(
            (bf16_t*)out + (long)row0 * H * P, (const float*)ws, n, parts);
        LAUNCH_CHECK();
    }
    return 0;
}

int gt_talk_plain(void* stream, int f32, void* out, const void* q,
                  const void* vc, const void* inv, const void* table,
                  int per_slot, const void* pos, const void* slot,
                  const void* kw, const void* talk, const void* cos_,
                  const void* sin_, int nrot, int N, int H, int G, int P,
                  int R, int chunk, float scale, float cap) {
    const int bytes = 4 * (2 * H * P + 16 * P + 34 * H);
    if (N < 1 || !sizes_ok(H, G, P, R, nrot, chunk) || bytes > 160 * 1024)
        return -100;
#define GO(T) do { const int e = allow_lds<k_talk_plain<T>>(160 * 1024); \
        if (e) return e; \
        k_talk_plain<T><<<N, 256, bytes, (hipStream_t)stream>>>((T*)out, \
        (const T*)q, (const T*)vc, (const float*)inv, (const int*)table, \
        per_slot, (const int*)pos, (const int*)slot, (const float*)kw, \
        (const float*)talk, rotation(cos_, sin_, R, nrot), H, G, P, chunk, \
        scale, cap); } while (0)
    if (f32) GO(float); else GO(bf16_t);
#undef GO
    LAUNCH_CHECK();
    return 0;
}

}  // extern "C"
