// gfx950 kernels of the layer-list models: a decoder whose layers each name a
// mixer (grouped softmax attention over a paged cache, latent or talking-heads
// attention, mLSTM, gated linear or lightning attention with a matrix memory
// per sequence, or two of these side by side) and a feed-forward (dense gated,
// dense with PolyNorm, or routed experts, with a shared one beside them).
// Latent attention is in gridllm_latent.hip, talking heads in gridllm_talk.hip.
//
// Conventions
//  * T is the element type of activations, weights and the KV cache: bf16, or
//    f32 for the exact mode. The residual stream, norms, scores, gates, router
//    logits and recurrent state are f32 in both.
//  * Widths and head sizes are padded by the host to multiples of 64 with zero
//    weights, so rows are 16-byte aligned and padding stays zero; the true
//    sizes enter only where a mean is taken.
//  * The tokens of a step are ordered decode rows first (one token of a
//    sequence each), then the prompt portions, each a contiguous segment.
//
// Exported extern "C" with an explicit stream; nothing here allocates.

#include "gridllm_attention.h"
#include "gridllm_tiles.h"

// ===========================================================================
// x = embed[token], f32, plus pos_table[position] if there is one, then its
// norm if there are norm weights; xb = the same in T
// ===========================================================================
template <class T>
__global__ void __launch_bounds__(256)
k_embed(float* __restrict__ x, T* __restrict__ xb,
        const T* __restrict__ emb, const T* __restrict__ ptab,
        const long long* __restrict__ tok, const int* __restrict__ pos,
        const float* __restrict__ w, float w_off, int W, int Wtrue, float eps,
        int vocab, int max_pos) {
    __shared__ float red[4];
    const long n = blockIdx.x;
    const long t = min(max(tok[n], 0ll), (long long)vocab - 1);
    const long p = ptab ? min(max(pos[n], 0), max_pos - 1) : 0;
    auto row = [&](int c, float* a) {
        ld8(emb + t * W + c, a);
        if (!ptab) return;
        float b[8];
        ld8(ptab + p * W + c, b);
#pragma unroll
        for (int i = 0; i < 8; ++i) a[i] += b[i];
    };
    float rs = 1.f;
    if (w) {
        float ss = 0.f;
        for (int c = threadIdx.x * 8; c < W; c += 2048) {
            float a[8];
            row(c, a);
#pragma unroll
            for (int i = 0; i < 8; ++i) ss += a[i] * a[i];
        }
        rs = 1.f / sqrtf(block_sum(ss, red) / (float)Wtrue + eps);
    }
    for (int c = threadIdx.x * 8; c < W; c += 2048) {
        float a[8];
        row(c, a);
        if (w) {
            float g[8];
            ld8(w + c, g);
#pragma unroll
            for (int i = 0; i < 8; ++i) a[i] *= rs * (w_off + g[i]);
        }
        st8(x + n * W + c, a);
        if (xb) st8(xb + n * W + c, a);
    }
}

// ===========================================================================
// Norm of a sublayer's output, added to the residual:
//   x += y * (1 / sqrt(mean(y^2) + eps)) * (w_off + w);  xb = T(x)
// TOP > 0 (routed experts): y is sum_k wt[n, k] * ye[n * top + k].
// W <= 8192 (a row is kept in registers); the mean is over Wtrue elements.
// ===========================================================================
// 8 columns of a sublayer's output. A pair of weight zero has no row (its
// expert is an identity).
template <class T, bool MOE>
DEV_INLINE void sublayer8(const T* y, const float* wt, int top, long n, int W,
                          int c, float* v) {
    if (!MOE) {
        ld8(y + n * W + c, v);
        return;
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) v[i] = 0.f;
    for (int k0 = 0; k0 < top; k0 += 4) {       // 4 rows in flight
        float f[4][8], g[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const long r = n * top + min(k0 + k, top - 1);
            g[k] = k0 + k < top ? wt[r] : 0.f;
            if (g[k] != 0.f) ld8(y + r * W + c, f[k]);
        }
#pragma unroll
        for (int k = 0; k < 4; ++k)
            if (g[k] != 0.f)
#pragma unroll
                for (int i = 0; i < 8; ++i) v[i] += g[k] * f[k][i];
    }
}

template <class T, bool MOE>
__global__ void __launch_bounds__(256)
k_post_norm(float* __restrict__ x, T* __restrict__ xb,
            const T* __restrict__ y, const float* __restrict__ wt, int top,
            const float* __restrict__ w, float w_off, int W, int Wtrue,
            float eps) {
    __shared__ float red[4];
    const long n = blockIdx.x;
    float v[4][8];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8;
        if (c < W) {
            sublayer8<T, MOE>(y, wt, top, n, W, c, v[j]);
#pragma unroll
            for (int i = 0; i < 8; ++i) ss += v[j][i] * v[j][i];
        }
    }
    const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)Wtrue + eps);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8;
        if (c < W) {
            float a[8], g[8];
            ld8(x + n * W + c, a);
            ld8(w + c, g);
#pragma unroll
            for (int i = 0; i < 8; ++i) a[i] += v[j][i] * rs * (w_off + g[i]);
            st8(x + n * W + c, a);
            if (xb) st8(xb + n * W + c, a);
        }
    }
}

// ===========================================================================
// Norm behind the sum, and the average over depth:
//   r = norm(alpha * x + y) * (w_off + w)       r: the (sub)layer's result
//   hist null:  x' = r
//   otherwise:  x' = sum_{j < nh} coef[j] hist[j] + coef[nh] r, and r is
//               kept as hist[nh] if `keep`. hist: f32 [layers + 1][N][W]
//   xb = T(x'). The row x may be x' or a row of hist.
// With experts y is their weighted sum plus ident[n] * x (the weight of the
// identity experts, which return the sublayer's input).
// ===========================================================================
template <class T, bool MOE>
__global__ void __launch_bounds__(256)
k_sum_norm(float* xo, T* __restrict__ xb, const float* x,
           const T* __restrict__ y, const float* __restrict__ wt, int top,
           const float* __restrict__ ident, const float* __restrict__ w,
           float w_off, float alpha, float* hist,
           const float* __restrict__ coef, int nh, int keep, long N, int W,
           int Wtrue, float eps) {
    __shared__ float red[4];
    const long n = blockIdx.x;
    if (MOE && ident) alpha += ident[n];
    float v[4][8];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8;
        if (c < W) {
            float a[8];
            sublayer8<T, MOE>(y, wt, top, n, W, c, v[j]);
            ld8(x + n * W + c, a);
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                v[j][i] += alpha * a[i];
                ss += v[j][i] * v[j][i];
            }
        }
    }
    const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)Wtrue + eps);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8;
        if (c < W) {
            float g[8];
            ld8(w + c, g);
#pragma unroll
            for (int i = 0; i < 8; ++i) v[j][i] *= rs * (w_off + g[i]);
            if (hist) {
                if (keep) st8(hist + (nh * N + n) * W + c, v[j]);
                const float cr = coef[nh];
#pragma unroll
                for (int i = 0; i < 8; ++i) v[j][i] *= cr;
                for (int l0 = 0; l0 < nh; l0 += 4) {    // 4 rows in flight
                    float f[4][8];
#pragma unroll
                    for (int l = 0; l < 4; ++l)
                        ld8(hist + (min(l0 + l, nh - 1) * N + n) * W + c, f[l]);
#pragma unroll
                    for (int l = 0; l < 4; ++l) {
                        const float cl = l0 + l < nh ? coef[l0 + l] : 0.f;
#pragma unroll
                        for (int i = 0; i < 8; ++i) v[j][i] += cl * f[l][i];
                    }
                }
            }
            st8(xo + n * W + c, v[j]);
            if (xb) st8(xb + n * W + c, v[j]);
        }
    }
}

// out[r] = norm(x[rows[r]]) in T; rows null = identity
template <class T>
__global__ void __launch_bounds__(256)
k_norm_rows(T* __restrict__ out, const float* __restrict__ x,
            const int* __restrict__ rows, const float* __restrict__ w,
            float w_off, int W, int Wtrue, float eps) {
    __shared__ float red[4];
    const long n = rows ? rows[blockIdx.x] : blockIdx.x;
    float ss = 0.f;
    for (int c = threadIdx.x * 8; c < W; c += 2048) {
        float a[8];
        ld8(x + n * W + c, a);
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += a[i] * a[i];
    }
    const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)Wtrue + eps);
    for (int c = threadIdx.x * 8; c < W; c += 2048) {
        float a[8], g[8];
        ld8(x + n * W + c, a);
        ld8(w + c, g);
#pragma unroll
        for (int i = 0; i < 8; ++i) a[i] *= rs * (w_off + g[i]);
        st8(out + (long)blockIdx.x * W + c, a);
    }
}

// ===========================================================================
// Norm in groups: a row's `groups` equal consecutive parts, each divided by
// its own root mean square, times w (no offset).
//   ADD:  x += norm(y) * wy;  out = norm(x) * w, if there is an out
//   else: out[r] = norm(x[rows[r]]) * w
// Columns from Wtrue on carry zeros. Squares are summed in pieces of GR columns
// (the largest power of two up to 8 that divides a group), which meet in LDS:
// group sums come out the same in every run. W <= 8192.
// ===========================================================================
struct Groups {
    int count, size;
};

// v holds columns c .. c + 7 of j = 0 .. 3; factors 1 / rms by group into rs
template <int GR>
DEV_INLINE void group_factors(const float v[4][8], float* part, float* rs,
                              int W, const Groups gp, float eps) {
    __syncthreads();                       // part and rs are free
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8;
        if (c < W)
#pragma unroll
            for (int i = 0; i < 8; i += GR) {
                float s = 0.f;
#pragma unroll
                for (int k = 0; k < GR; ++k) s += v[j][i + k] * v[j][i + k];
                part[(c + i) / GR] = s;
            }
    }
    __syncthreads();
    const int lane = threadIdx.x & 63, n = gp.size / GR;
    for (int g = threadIdx.x >> 6; g < gp.count; g += 4) {
        float s = 0.f;
        for (int i = lane; i < n; i += 64) s += part[g * n + i];
        s = wave_reduce_sum(s);
        if (lane == 0) rs[g] = 1.f / sqrtf(s / (float)gp.size + eps);
    }
    __syncthreads();
}

// f *= rs of each column's group
template <int GR>
DEV_INLINE void scale_groups(float* f, const float* rs, int c,
                             const Groups gp) {
#pragma unroll
    for (int i = 0; i < 8; i += GR) {
        const float r = rs[min((c + i) / gp.size, gp.count - 1)];
#pragma unroll
        for (int k = 0; k < GR; ++k) f[i + k] *= r;
    }
}

template <class T, bool ADD, int GR>
__global__ void __launch_bounds__(256)
k_group_norm(T* __restrict__ out, float* __restrict__ x,
             const T* __restrict__ y, const int* __restrict__ rows,
             const float* __restrict__ wy, const float* __restrict__ w, int W,
             const Groups gp, float eps) {
    extern __shared__ float part[];        // W / GR, then a factor per group
    float* const rs = part + W / GR;
    const long n = !ADD && rows ? rows[blockIdx.x] : blockIdx.x;
    float v[4][8], a[4][8];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8;
        if (c < W) {
            ld8(x + n * W + c, a[j]);
            if (ADD) ld8(y + n * W + c, v[j]);
        }
    }
    if (ADD) {
        group_factors<GR>(v, part, rs, W, gp, eps);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int c = (j * 256 + threadIdx.x) * 8;
            if (c < W) {
                float g[8];
                ld8(wy + c, g);
                scale_groups<GR>(v[j], rs, c, gp);
#pragma unroll
                for (int i = 0; i < 8; ++i) a[j][i] += v[j][i] * g[i];
                st8(x + n * W + c, a[j]);
            }
        }
        if (!out) return;
    }
    group_factors<GR>(a, part, rs, W, gp, eps);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8;
        if (c < W) {
            float g[8];
            ld8(w + c, g);
            scale_groups<GR>(a[j], rs, c, gp);
#pragma unroll
            for (int i = 0; i < 8; ++i) a[j][i] *= g[i];
            st8(out + (long)blockIdx.x * W + c, a[j]);
        }
    }
}

// ===========================================================================
// Hyper-connections: ns residual streams x_s, f32 [N][ns][W].
//   start: x_s = embed[token] * scale for all s
//   join:  x_t = sum_s mix[s][t] x_s + put[t] y, all from the old ones
// and what the next sublayer reads, if there is one:
//   h = T(norm(sum_s in[s] x_s) * w)
// hc holds mix [from][to], then put. y is a sublayer's output; with experts
// (top > 0) the sum of a token's pairs, and `extra` adds a row times the
// sigmoid of a number per token. S: ns rounded up to a power of two. W <= 2048
// NV; the mean is over Wtrue elements.
// ===========================================================================
template <class T, int NV>
DEV_INLINE void store_normed(T* h, const float u[NV][8], const float* w,
                             long n, int W, int Wtrue, float eps, float* red) {
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j)
        if ((j * 256 + threadIdx.x) * 8 < W)
#pragma unroll
            for (int i = 0; i < 8; ++i) ss += u[j][i] * u[j][i];
    const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)Wtrue + eps);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8;
        if (c < W) {
            float g[8];
            ld8(w + c, g);
#pragma unroll
            for (int i = 0; i < 8; ++i) g[i] *= u[j][i] * rs;
            st8(h + n * W + c, g);
        }
    }
}

template <class T>
__global__ void __launch_bounds__(256)
k_streams_start(float* __restrict__ x, T* __restrict__ h,
                const T* __restrict__ emb, const long long* __restrict__ tok,
                float scale, const float* __restrict__ in,
                const float* __restrict__ w, int ns, int W, int Wtrue,
                float eps, int vocab) {
    __shared__ float red[4];
    const long n = blockIdx.x;
    const long t = min(max(tok[n], 0ll), (long long)vocab - 1);
    float total = 0.f, u[4][8];
    for (int s = 0; s < ns; ++s) total += in[s];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8;
        if (c < W) {
            float a[8];
            ld8(emb + t * W + c, a);
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                a[i] *= scale;
                u[j][i] = total * a[i];
            }
            for (int s = 0; s < ns; ++s) st8(x + (n * ns + s) * W + c, a);
        }
    }
    store_normed<T, 4>(h, u, w, n, W, Wtrue, eps, red);
}

template <class T, int S, int NV, bool MOE>
__global__ void __launch_bounds__(256)
k_streams_join(float* __restrict__ x, T* __restrict__ h,
               const T* __restrict__ y, int top, const T* __restrict__ extra,
               const float* __restrict__ extra_z, int extra_ld,
               const float* __restrict__ hc, const float* __restrict__ in,
               const float* __restrict__ w, int ns, int W, int Wtrue,
               float eps) {
    constexpr bool AHEAD = S * NV <= 8;     // all loads ahead of the stores
    constexpr int NX = AHEAD ? NV : 1;
    __shared__ float red[4];
    const long n = blockIdx.x;
    float* xr = x + n * ns * W;
    const float ge = MOE && extra ? sigmoidf_(extra_z[n * extra_ld]) : 0.f;
    float a[NX][S][8], v[NX][8], u[NV][8];
    auto load = [&](int j, int c) {
#pragma unroll
        for (int s = 0; s < S; ++s)
            if (s < ns) ld8(xr + (long)s * W + c, a[j][s]);
        if (!MOE) {
            ld8(y + n * W + c, v[j]);
            return;
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) v[j][i] = 0.f;
        for (int k0 = 0; k0 < top; k0 += 4) {       // 4 rows in flight
            float f[4][8];
#pragma unroll
            for (int k = 0; k < 4; ++k)
                ld8(y + (n * top + min(k0 + k, top - 1)) * W + c, f[k]);
#pragma unroll
            for (int k = 0; k < 4; ++k)
#pragma unroll
                for (int i = 0; i < 8; ++i)
                    v[j][i] += k0 + k < top ? f[k][i] : 0.f;
        }
        if (extra) {
            float f[8];
            ld8(extra + n * W + c, f);
#pragma unroll
            for (int i = 0; i < 8; ++i) v[j][i] += ge * f[i];
        }
    };
    if (AHEAD)
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int c = (j * 256 + threadIdx.x) * 8;
            if (c < W) load(j % NX, c);
        }
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8, jx = j % NX;
        if (c < W) {
            if (!AHEAD) load(jx, c);
#pragma unroll
            for (int i = 0; i < 8; ++i) u[j][i] = 0.f;
#pragma unroll
            for (int t = 0; t < S; ++t) {
                if (t >= ns) continue;
                const float put = hc[ns * ns + t], read = h ? in[t] : 0.f;
                float r[8];
#pragma unroll
                for (int i = 0; i < 8; ++i) r[i] = put * v[jx][i];
#pragma unroll
                for (int s = 0; s < S; ++s) {
                    if (s >= ns) continue;
                    const float m = hc[s * ns + t];
#pragma unroll
                    for (int i = 0; i < 8; ++i) r[i] += m * a[jx][s][i];
                }
#pragma unroll
                for (int i = 0; i < 8; ++i) u[j][i] += read * r[i];
                st8(xr + (long)t * W + c, r);
            }
        }
    }
    if (h) store_normed<T, NV>(h, u, w, n, W, Wtrue, eps, red);
}

// out[r] = norm(sum_s x_s[rows[r]]) * w; rows null = identity
template <class T>
__global__ void __launch_bounds__(256)
k_streams_norm(T* __restrict__ out, const float* __restrict__ x,
               const int* __restrict__ rows, const float* __restrict__ w,
               int ns, int W, int Wtrue, float eps) {
    __shared__ float red[4];
    const long n = rows ? rows[blockIdx.x] : blockIdx.x;
    float u[4][8];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int c = (j * 256 + threadIdx.x) * 8;
#pragma unroll
        for (int i = 0; i < 8; ++i) u[j][i] = 0.f;
        if (c < W)
            for (int s = 0; s < ns; ++s) {
                float a[8];
                ld8(x + (n * ns + s) * W + c, a);
#pragma unroll
                for (int i = 0; i < 8; ++i) u[j][i] += a[i];
            }
    }
    store_normed<T, 4>(out, u, w, blockIdx.x, W, Wtrue, eps, red);
}

// ===========================================================================
// PolyNorm: out = c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3, powers by element, N
// dividing a row by its root mean square over Ftrue elements (columns behind
// them are zero). NV > 0: a row of up to NV * 2048 columns stays in registers.
// ===========================================================================
template <class T, int NV>
__global__ void __launch_bounds__(256)
k_poly_norm(T* __restrict__ out, const T* __restrict__ z,
            const float* __restrict__ coef, int F, int Ftrue, float eps) {
    __shared__ float red[3][4];
    constexpr int KEEP = NV ? NV : 1;
    const long n = blockIdx.x;
    float v[KEEP][8], ss[3] = {0.f, 0.f, 0.f};
    auto add = [&](const float* f) {
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const float q = f[i] * f[i];
            ss[0] += q;
            ss[1] += q * q;
            ss[2] += q * q * q;
        }
    };
    if (NV) {
#pragma unroll
        for (int j = 0; j < KEEP; ++j) {
            const int c = (j * 256 + threadIdx.x) * 8;
            if (c < F) {
                ld8(z + n * F + c, v[j]);
                add(v[j]);
            }
        }
    } else {
        for (int c = threadIdx.x * 8; c < F; c += 2048) {
            ld8(z + n * F + c, v[0]);
            add(v[0]);
        }
    }
    float k[3];
#pragma unroll
    for (int i = 0; i < 3; ++i) {
        const float s = wave_reduce_sum(ss[i]);
        if ((threadIdx.x & 63) == 0) red[i][threadIdx.x >> 6] = s;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 3; ++i)
        k[i] = coef[i] / sqrtf((red[i][0] + red[i][1] + red[i][2] +
                                red[i][3]) / (float)Ftrue + eps);
    const float k3 = coef[3];
    auto put = [&](float* f, int c) {
#pragma unroll
        for (int i = 0; i < 8; ++i)
            f[i] = k3 + f[i] * (k[0] + f[i] * (k[1] + f[i] * k[2]));
        st8(out + n * F + c, f);
    };
    if (NV) {
#pragma unroll
        for (int j = 0; j < KEEP; ++j) {
            const int c = (j * 256 + threadIdx.x) * 8;
            if (c < F) put(v[j], c);
        }
    } else {
        for (int c = threadIdx.x * 8; c < F; c += 2048) {
            ld8(z + n * F + c, v[0]);
            put(v[0], c);
        }
    }
}

// out = glu(gu[:, :F], gu[:, F:]), f32
__global__ void __launch_bounds__(256)
k_glu_f32(float* __restrict__ out, const float* __restrict__ gu, long n,
          int F, const GluParams p) {
    for (long i = blockIdx.x * 256L + threadIdx.x; i < n * F;
         i += gridDim.x * 256L) {
        const long r = i / F, c = i % F;
        float g = fminf(gu[r * 2 * F + c], p.limit);
        float u = fminf(fmaxf(gu[r * 2 * F + F + c], -p.limit), p.limit);
        const float z = p.alpha * g * (1.f + p.cubic * g * g);
        out[i] = g / (1.f + expf(-z)) * (u + p.shift);
    }
}

// ===========================================================================
// Projection to a few f32 outputs (router logits, recurrence gates):
//   out[n, j] = sum_k x[n, k] w[j, k] + bias[j], bf16 inputs, f32 result.
// One block per 16 rows x 16 NT outputs; its 8 waves split K and add up in
// LDS, each with U steps of loads in flight. Fragments load straight from
// memory (both operands are k-contiguous). K % 32 == 0.
// ===========================================================================
template <int NT>
__global__ void __launch_bounds__(512)
k_proj_f32(float* __restrict__ out, const bf16_t* __restrict__ x,
           const bf16_t* __restrict__ w, const float* __restrict__ bias,
           int M, int N, int K) {
    constexpr int U = NT == 1 ? 6 : 4;
    __shared__ float red[8][16][16 * NT + 1];
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int fr = lane & 15, kg = (lane >> 4) * 8;
    const int m0 = blockIdx.x * 16, n0 = blockIdx.y * 16 * NT;
    const bf16_t* xr = x + (long)min(m0 + fr, M - 1) * K + kg;
    const bf16_t* wr[NT];
    f32x4 acc[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        wr[t] = w + (long)min(n0 + t * 16 + fr, N - 1) * K + kg;
        acc[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    }
    const int steps = K >> 5;
    for (int s0 = wid; s0 < steps; s0 += 8 * U) {
        bf16x8 a[U], b[U][NT];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int s = min(s0 + u * 8, steps - 1);
            a[u] = *(const bf16x8*)(xr + s * 32);
#pragma unroll
            for (int t = 0; t < NT; ++t)
                b[u][t] = *(const bf16x8*)(wr[t] + s * 32);
        }
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (s0 + u * 8 < steps)
#pragma unroll
                for (int t = 0; t < NT; ++t)
                    acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                        a[u], b[u][t], acc[t], 0, 0, 0);
    }
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r)
            red[wid][(lane >> 4) * 4 + r][t * 16 + fr] = acc[t][r];
    __syncthreads();
    for (int e = threadIdx.x; e < 256 * NT; e += 512) {
        const int i = e / (16 * NT), j = e % (16 * NT);
        if (m0 + i >= M || n0 + j >= N) continue;
        float v = bias ? bias[n0 + j] : 0.f;
#pragma unroll
        for (int k = 0; k < 8; ++k) v += red[k][i][j];
        out[(long)(m0 + i) * N + n0 + j] = v;
    }
}

// ===========================================================================
// Attention prologue: rotated (if there are tables) unit-RMS q and k (no
// weight), query temperature, and the write of k and v into the paged cache,
// from one projection row
//   [H*P q | G*P k | G*P v | ...], row stride ld.
// temperature(p) = 1 + coef * ln(floor((p + 1) / every) + 1).
// P / 8 lanes per head. Further waves put SiLU on act_n columns from act_0 on,
// in place (q, k and v of a recurrence in the same row).
// ===========================================================================
template <class T, int P>
__global__ void __launch_bounds__(256)
k_qknorm_kv(T* __restrict__ qkv, T* __restrict__ q_out,
            T* __restrict__ kc, T* __restrict__ vc,
            const int* __restrict__ table, int per_slot,
            const int* __restrict__ pos, const int* __restrict__ slot,
            int N, int H, int G, int ld_, int dim, float eps, float coef,
            int every, const Rotation rot, int act_0, int act_n) {
    constexpr int LPH = P / 8, HW = 64 / LPH;
    const int nh = H + 2 * G;
    const int groups = (nh + HW - 1) / HW, per = groups + (act_n + 511) / 512;
    const long item = blockIdx.x * 4L + (threadIdx.x >> 6);
    if (item >= (long)N * per) return;
    const int n = (int)(item / per), it = (int)(item % per);
    const int lane = threadIdx.x & 63;
    float f[8];
    if (it >= groups) {
        const int c = (it - groups) * 512 + lane * 8;
        if (c >= act_n) return;
        T* z = qkv + (long)n * ld_ + act_0 + c;
        ld8(z, f);
#pragma unroll
        for (int i = 0; i < 8; ++i) f[i] *= sigmoidf_(f[i]);
        st8(z, f);
        return;
    }
    const int h = it * HW + lane / LPH, c = (lane % LPH) * 8;
    if (h >= nh) return;
    ld8(qkv + (long)n * ld_ + (long)h * P + c, f);
    const int p = pos[n];
    T* dst;
    if (h < H) {
        dst = q_out + ((long)n * H + h) * P;
    } else {
        const int blk = p / KV_PAGE;
        if (blk >= per_slot) return;
        const int hk = (h - H) % G;
        const long page = table[(long)slot[n] * per_slot + blk];
        dst = (h < H + G ? kc : vc) +
              ((page * G + hk) * KV_PAGE + p % KV_PAGE) * P;
    }
    if (h < H + G) {
        if (c < 2 * rot.half) rotate8(f, c, p, rot);
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < 8; ++i) ss += f[i] * f[i];
#pragma unroll
        for (int off = LPH / 2; off > 0; off >>= 1)
            ss += __shfl_xor(ss, off, WAVE);
        float s = 1.f / sqrtf(ss / (float)dim + eps);
        if (h < H) s *= 1.f + coef * logf((float)((p + 1) / every) + 1.f);
#pragma unroll
        for (int i = 0; i < 8; ++i) f[i] *= s;
    }
    st8(dst + c, f);
}

// Varlen prefill over the paged cache. meta row (8 ints): {q_off, len, slot,
// q0, start}: rows [q0, q0 + 128) of the portion packed at q_off, whose first
// token stands at position `start`.
template <int D, class Keys>
__global__ void __launch_bounds__(256, D > 128 ? 1 : 2)
k_paged_prefill(bf16_t* __restrict__ out, const bf16_t* __restrict__ q,
                const PagedKV<D> kv, const int* __restrict__ meta, int Hq,
                int G, float scale, const HeadEpilogue epi, const Keys keys) {
    __shared__ __attribute__((aligned(16))) bf16_t vt[D * 40];
    __shared__ __attribute__((aligned(16))) bf16_t plds[4][2 * 64 * 8];
    const int* m = meta + blockIdx.x * 8;
    const int q_off = m[0], len = m[1], start = m[4];
    attn_prefill_tile<D>(out + epi.at(q_off, 0, Hq, D),
                         q + (long)q_off * Hq * D, kv, len, Hq, G, m[2],
                         start + len, start, scale, m[3], vt, &plds[0][0],
                         epi, q_off, keys);
}

// Exact mode: one block per (row, query head), f32 cache, any position.
template <int P>
__global__ void __launch_bounds__(256)
k_attn_rows_f32(float* __restrict__ out, const float* __restrict__ q,
                const float* __restrict__ kc, const float* __restrict__ vc,
                const int* __restrict__ table, int per_slot,
                const int* __restrict__ pos, const int* __restrict__ slot,
                int H, int G, float scale, const float* __restrict__ sink,
                const float* __restrict__ gate, int gate_ld, int gate_el,
                float oscale, int out_ld, const WindowKeys keys) {
    const int n = blockIdx.x / H, h = blockIdx.x % H;
    const int hk = h / (H / G);
    const int* tab = table + (long)slot[n] * per_slot;
    const int seq = min(pos[n] + 1, per_slot * KV_PAGE);
    __shared__ float qs[P], sc[256], red[4], acc_s[256];
    for (int i = threadIdx.x; i < P; i += 256)
        qs[i] = q[((long)n * H + h) * P + i];
    __syncthreads();
    constexpr int NG = 256 / P;
    const int c = threadIdx.x % P, grp = threadIdx.x / P;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    float m = sink ? sink[h] : -INFINITY, l = sink ? 1.f : 0.f, acc = 0.f;
    for (int k0 = keys.skip(0, seq - 1); k0 < seq;
         k0 = keys.skip(k0 + 256, seq - 1)) {
        const int j = k0 + threadIdx.x;
        const bool seen = j < seq && keys.sees(seq - 1, j);
        float s = -INFINITY;
        if (seen) {
            const float* kr = kc + (((long)tab[j / KV_PAGE] * G + hk) * KV_PAGE
                                    + j % KV_PAGE) * P;
            s = 0.f;
            for (int i = 0; i < P; i += 4) {
                const float4 kv = *(const float4*)(kr + i);
                s += kv.x * qs[i] + kv.y * qs[i + 1] + kv.z * qs[i + 2] +
                     kv.w * qs[i + 3];
            }
            s *= scale;
        }
        float mx = wave_reduce_max(s);
        if (lane == 0) red[wid] = mx;
        __syncthreads();
        mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
        const float mn = fmaxf(m, mx);
        const float alpha = (m == -INFINITY) ? 0.f : expf(m - mn);
        const float p = seen ? expf(s - mn) : 0.f;
        sc[threadIdx.x] = p;
        m = mn;
        __syncthreads();                       // red read, sc written
        const float ps = wave_reduce_sum(p);
        if (lane == 0) red[wid] = ps;
        acc *= alpha;
        const int jn = min(256, seq - k0);
        for (int t = grp; t < jn; t += NG) {
            const int jj = k0 + t;
            acc += sc[t] * vc[(((long)tab[jj / KV_PAGE] * G + hk) * KV_PAGE +
                               jj % KV_PAGE) * P + c];
        }
        __syncthreads();
        l = l * alpha + red[0] + red[1] + red[2] + red[3];
        __syncthreads();
    }
    acc_s[threadIdx.x] = acc;
    __syncthreads();
    if (threadIdx.x < P) {
        float a = 0.f;
        for (int g = 0; g < NG; ++g) a += acc_s[g * P + threadIdx.x];
        float f = l > 0.f ? oscale / l : 0.f;
        if (gate)
            f *= sigmoidf_(gate[(long)n * gate_ld +
                                (gate_el ? h * P + threadIdx.x : h)]);
        out[(long)n * out_ld + h * P + threadIdx.x] = a * f;
    }
}

// ===========================================================================
// mLSTM: matrix memory with exponential gates, per head
//   i = cap tanh(zi / cap);  f = logsigmoid(cap tanh(zf / cap))
//   m' = max(f + m, i);  keep = exp(f + m - m');  put = exp(i - m')
//   S = keep S + put v k^T;  n = keep n + put k
//   o = S q / (max(|n . q|, exp(-m')) + 1e-6),  q scaled by dim^-1/2
// The state of a slot is f32 [H][DV + 1][DK]: row r < DV is S[:, r] over the
// key dimension, and row DV is n, which is the memory of the constant value
// 1, so one update serves both. m is f32 [H]. A segment that starts at
// position 0 takes the state as zero whatever the slot holds.
// Projection row: [H*DK q | H*DK k | H*DV v | H*DV out gate | ...], stride ld;
// gate row: [H zi | H zf], f32, biases included.
// ===========================================================================
DEV_INLINE void mlstm_gates(const float* gr, int h, int H, float cap,
                            float& i, float& f) {
    i = cap * tanhf(gr[h] / cap);
    const float z = cap * tanhf(gr[H + h] / cap);
    f = fminf(z, 0.f) - log1pf(expf(-fabsf(z)));
}

// seg (int4): {first token, length, slot, start position}; null: row r is a
// segment of one token at pos[r] of slot[r].
DEV_INLINE int4 segment(const int4* seg, const int* pos, const int* slot,
                        int r) {
    if (seg) return seg[r];
    return make_int4(r, 1, slot[r], pos[r]);
}

// Token by token. Block = (segment, head, `rpb` state rows); LPR lanes hold
// one row of DK as NJ float4 each, and a wave works on 64 / LPR rows at once,
// U of them in flight. The other kinds have neither an input gate nor a
// normaliser row (S is [H][DV][DK]): their memory decays per key channel, gr
// being the logarithm of the decay, f32 [n][H*DK] (gated linear attention), or
// by a constant per head, gr f32 [H] (lightning attention).
enum Rec { MLSTM = 0, CHANNELS = 1, CONSTANT = 2 };

template <class T, int LPR, int NJ, int KIND>
__global__ void __launch_bounds__(256)
k_rec_step(float* __restrict__ o, float* __restrict__ S,
           const float* __restrict__ mst, const T* __restrict__ qkv,
           const float* __restrict__ gr, const int4* __restrict__ segs,
           const int* __restrict__ pos, const int* __restrict__ slot,
           int H, int DK, int DV, int ld_, float qscale, float cap,
           int rpb) {
    constexpr int RW = 64 / LPR;
    constexpr int U = NJ == 1 ? 4 : 2;
    constexpr bool CH = KIND == CHANNELS, GATED = KIND == MLSTM;
    const int R = GATED ? DV + 1 : DV;
    const int4 sg = segment(segs, pos, slot, blockIdx.x);
    const int h = blockIdx.y;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int c0 = (lane % LPR) * 4, rl = lane / LPR;
    const int rbeg = blockIdx.z * rpb, rend = min(R, rbeg + rpb);
    float* Sb = S + ((long)sg.z * H + h) * R * DK;
    float m = !GATED || sg.w == 0 ? 0.f : mst[(long)sg.z * H + h];
    for (int t = 0; t < sg.y; ++t) {
        const long n = sg.x + t;
        const bool fresh = sg.w + t == 0;
        float keep1 = KIND == CONSTANT ? gr[h] : 0.f, put = 1.f;
        if (GATED) {
            float gi, gf;
            mlstm_gates(gr + n * 2 * H, h, H, cap, gi, gf);
            const float mn = fmaxf(gf + m, gi);
            keep1 = expf(gf + m - mn);
            put = expf(gi - mn);
            m = mn;
        }
        const T* row = qkv + n * ld_;
        float qv[NJ][4], kv[NJ][4], keep[CH ? NJ : 1][4];
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
            const int c = c0 + j * LPR * 4;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const bool in = c < DK;
                qv[j][i] = in ? ld(row + h * DK + c + i) * qscale : 0.f;
                kv[j][i] = in ? ld(row + (H + h) * DK + c + i) * put : 0.f;
                if (CH)
                    keep[j][i] =
                        in ? expf(gr[n * H * DK + h * DK + c + i]) : 0.f;
            }
        }
        auto kept = [&](int j, int i) { return CH ? keep[j][i] : keep1; };
        const T* vrow = row + 2 * H * DK + h * DV;
        for (int r0 = rbeg + wid * RW * U; r0 < rend; r0 += 4 * RW * U) {
            float4 s[U][NJ];
            float v[U];
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int r = r0 + u * RW + rl;
                v[u] = r < DV ? ld(vrow + r) : 1.f;
                if (r >= rend) v[u] = 0.f;
#pragma unroll
                for (int j = 0; j < NJ; ++j) {
                    const int c = c0 + j * LPR * 4;
                    s[u][j] = make_float4(0.f, 0.f, 0.f, 0.f);
                    if (!fresh && r < rend && c < DK)
                        s[u][j] = *(const float4*)(Sb + (long)r * DK + c);
                }
            }
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int r = r0 + u * RW + rl;
                float a = 0.f;
#pragma unroll
                for (int j = 0; j < NJ; ++j) {
                    const int c = c0 + j * LPR * 4;
                    float4 z = s[u][j];
                    z.x = kept(j, 0) * z.x + kv[j][0] * v[u];
                    z.y = kept(j, 1) * z.y + kv[j][1] * v[u];
                    z.z = kept(j, 2) * z.z + kv[j][2] * v[u];
                    z.w = kept(j, 3) * z.w + kv[j][3] * v[u];
                    a += z.x * qv[j][0] + z.y * qv[j][1] + z.z * qv[j][2] +
                         z.w * qv[j][3];
                    if (r < rend && c < DK)
                        *(float4*)(Sb + (long)r * DK + c) = z;
                }
#pragma unroll
                for (int off = LPR / 2; off > 0; off >>= 1)
                    a += __shfl_xor(a, off, WAVE);
                if (lane % LPR == 0 && r < rend)
                    o[(n * H + h) * (DV + 4) + r] = a;
            }
        }
    }
}

// o (f32 rows of DV + 4 per token and head: DV sums, n . q, padding)
// -> T out[n, H*DV]: unit RMS per head, times norm, times sigmoid of the
// output gate. Items [0, nseg) are segments of the token-by-token kernel, whose
// o still lacks its denominator and whose m is advanced here; the nplain
// tokens from plain0 on are finished sums. One wave per (item, head). With
// SILU the gate multiplies by itself times its sigmoid.
template <class T, bool SILU>
__global__ void __launch_bounds__(256)
k_rec_out(T* __restrict__ out, const float* __restrict__ o,
            float* __restrict__ mst, const T* __restrict__ qkv,
            const float* __restrict__ gr, const int4* __restrict__ segs,
            const int* __restrict__ pos, const int* __restrict__ slot,
            const float* __restrict__ norm, int nseg, int plain0, int nplain,
            int H, int DK, int DV, int ld_, int dvtrue, float cap,
            float eps) {
    const long item = blockIdx.x * 4L + (threadIdx.x >> 6);
    if (item >= (long)(nseg + nplain) * H) return;
    const int it = (int)(item / H), h = (int)(item % H);
    const int lane = threadIdx.x & 63;
    int4 sg;
    float m = 0.f;
    const bool is_seg = it < nseg;
    if (is_seg) {
        sg = segment(segs, pos, slot, it);
        if (sg.w != 0) m = mst[(long)sg.z * H + h];
    } else {
        sg = make_int4(plain0 + it - nseg, 1, 0, 0);
    }
    for (int t = 0; t < sg.y; ++t) {
        const long n = sg.x + t;
        const float* ob = o + (n * H + h) * (DV + 4);
        float inv = 1.f;
        if (is_seg) {
            float gi, gf;
            mlstm_gates(gr + n * 2 * H, h, H, cap, gi, gf);
            m = fmaxf(gf + m, gi);
            inv = 1.f / (fmaxf(fabsf(ob[DV]), expf(-m)) + 1e-6f);
        }
        float ss = 0.f;
        for (int c = lane * 4; c < DV; c += 256) {
            const float4 v = *(const float4*)(ob + c);
            ss += (v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w) * inv * inv;
        }
        const float rs =
            inv / sqrtf(wave_reduce_sum(ss) / (float)dvtrue + eps);
        const T* g = qkv + n * ld_ + (long)H * (2 * DK + DV) + (long)h * DV;
        T* dst = out + (n * H + h) * DV;
        for (int c = lane * 4; c < DV; c += 256) {
            const float4 v = *(const float4*)(ob + c);
            const float4 w = *(const float4*)(norm + h * DV + c);
            float z[4];
            ld4(g + c, z);
#pragma unroll
            for (int i = 0; i < 4; ++i)
                z[i] = sigmoidf_(z[i]) * (SILU ? z[i] : 1.f);
            const float r[4] = {v.x * rs * w.x * z[0], v.y * rs * w.y * z[1],
                                v.z * rs * w.z * z[2], v.w * rs * w.w * z[3]};
            st4(dst + c, r);
        }
    }
    if (is_seg && lane == 0) mst[(long)sg.z * H + h] = m;
}

// The same for heads that are normed together and have no denominators
// (lightning attention): one block per token, out rows of stride out_ld. NV > 0:
// a row of up to NV * 1024 columns stays in registers.
template <class T, int NV>
__global__ void __launch_bounds__(256)
k_rec_row_out(T* __restrict__ out, const float* __restrict__ o,
              const T* __restrict__ gate, const float* __restrict__ norm,
              int H, int DV, int ld_, int out_ld, int true_cols, float eps) {
    __shared__ float red[4];
    constexpr int KEEP = NV ? NV : 1;
    const long n = blockIdx.x;
    const int cols = H * DV;
    const float* ob = o + n * H * (DV + 4);
    float v[KEEP][4], ss = 0.f;
    auto load = [&](int c, float* f) {
        ld4(ob + (c / DV) * (DV + 4) + c % DV, f);
    };
    auto add = [&](const float* f) {
        ss += f[0] * f[0] + f[1] * f[1] + f[2] * f[2] + f[3] * f[3];
    };
    if (NV) {
#pragma unroll
        for (int j = 0; j < KEEP; ++j) {
            const int c = (j * 256 + threadIdx.x) * 4;
            if (c < cols) {
                load(c, v[j]);
                add(v[j]);
            }
        }
    } else {
        for (int c = threadIdx.x * 4; c < cols; c += 1024) {
            load(c, v[0]);
            add(v[0]);
        }
    }
    const float rs = 1.f / sqrtf(block_sum(ss, red) / (float)true_cols + eps);
    auto put = [&](int c, float* f) {
        float z[4], w[4];
        ld4(gate + n * ld_ + c, z);
        ld4(norm + c, w);
#pragma unroll
        for (int i = 0; i < 4; ++i) f[i] *= rs * w[i] * sigmoidf_(z[i]);
        st4(out + n * out_ld + c, f);
    };
    if (NV) {
#pragma unroll
        for (int j = 0; j < KEEP; ++j) {
            const int c = (j * 256 + threadIdx.x) * 4;
            if (c < cols) put(c, v[j]);
        }
    } else {
        for (int c = threadIdx.x * 4; c < cols; c += 1024) {
            load(c, v[0]);
            put(c, v[0]);
        }
    }
}

// ---------------------------------------------------------------------------
// Prompt portions in chunks of 64 tokens. With F_t the running sum of f
// inside a chunk, a_s = i_s - F_s and M_t = max(m_in, max_{s<=t} a_s):
//   m_t = F_t + M_t
//   S_t = exp(m_in - M_t) S_in + sum_{s<=t} exp(a_s - M_t) v_s k_s^T
// so a chunk's own contribution (state kernel), the state that enters each
// chunk (scan kernel), and the outputs (out kernel) separate; the first and
// the last run over all chunks at once on the matrix cores. Where a product
// takes f32 factors (state, weighted keys) they are split into two bf16 parts.
//
// chunk (int4): {first token, length, segment, -}
// seg   (int4): {slot, start position, first chunk, chunks}
// dS: f32 [chunks][H][DV + 1][DK]; the scan leaves the entering state there as
// (hi | lo << 16) bf16 pairs. scal: f32 [chunks][H][4] = {max a, F total,
// m of the slot before the step, m_in}.
// ---------------------------------------------------------------------------
#define MCH 64
#define MLD 72      // padded row of 64 tokens in LDS

// Lightning attention (CONST) is the case i = 0, f the same for every token: m
// then stays 0. It has no normaliser and no head norm; gr is f by head, f32
// [H]. Score weights are (hi, lo) pairs of bf16, too.

// running sum of f, a, running max of a; lane = token, wave-wide
template <bool CONST>
DEV_INLINE void chunk_scan(const float* gr, int tok0, int clen, int h, int H,
                           float cap, float& F, float& a, float& amax) {
    const int t = threadIdx.x & 63;
    float gi = -INFINITY, gf = 0.f;
    if (t < clen) {
        if (CONST) {
            gi = 0.f;
            gf = gr[h];
        } else {
            mlstm_gates(gr + (long)(tok0 + t) * 2 * H, h, H, cap, gi, gf);
        }
    }
    F = gf;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const float u = __shfl_up(F, off, WAVE);
        if (t >= off) F += u;
    }
    a = gi - F;
    amax = a;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const float u = __shfl_up(amax, off, WAVE);
        if (t >= off) amax = fmaxf(amax, u);
    }
}

template <bool CONST>
__global__ void __launch_bounds__(256)
k_mlstm_chunk_state(float* __restrict__ dS, float* __restrict__ scal,
                    const float* __restrict__ mst,
                    const bf16_t* __restrict__ qkv,
                    const float* __restrict__ gr,
                    const int4* __restrict__ chunks,
                    const int4* __restrict__ segs, int H, int DK, int DV,
                    int ld_, float cap) {
    __shared__ __attribute__((aligned(16))) bf16_t vt[64 * MLD];
    __shared__ __attribute__((aligned(16))) bf16_t kh[64 * MLD];
    __shared__ __attribute__((aligned(16))) bf16_t kl[64 * MLD];
    __shared__ float wgt[MCH];
    const int4 ch = chunks[blockIdx.x];
    const int h = blockIdx.y;
    const int nd = DK / 64;
    const int d0 = (blockIdx.z % nd) * 64, v0 = (blockIdx.z / nd) * 64;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    if (wid == 0) {
        float F, a, amax;
        chunk_scan<CONST>(gr, ch.x, ch.y, h, H, cap, F, a, amax);
        const float A = __shfl(amax, 63, WAVE);
        wgt[lane] = lane < ch.y ? expf(a - A) : 0.f;
        if (blockIdx.z == 0 && lane == 63) {
            const int4 sg = segs[ch.z];
            float* sp = scal + ((long)blockIdx.x * H + h) * 4;
            sp[0] = A;
            sp[1] = F;
            sp[2] = CONST || sg.y == 0 ? 0.f : mst[(long)sg.x * H + h];
        }
    }
    __syncthreads();
    for (int i = threadIdx.x; i < 512; i += 256) {
        const int t = i & 63, c8 = (i >> 6) * 8;   // a wave spans 64 tokens
        const bf16_t* row = qkv + (long)(ch.x + min(t, ch.y - 1)) * ld_;
        float f[8];
        ld8(row + (H + h) * DK + d0 + c8, f);
        const uint4 vv = *(const uint4*)(row + 2 * H * DK + h * DV + v0 + c8);
        const bf16_t* pv = (const bf16_t*)&vv;
        const float w = wgt[t];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float x = f[j] * w;
            const bf16_t hi = f2bf(x);
            kh[(c8 + j) * MLD + t] = hi;
            kl[(c8 + j) * MLD + t] = f2bf(x - bf2f(hi));
            vt[(c8 + j) * MLD + t] = pv[j];
        }
    }
    __syncthreads();
    const int R = CONST ? DV : DV + 1;
    float* Db = dS + ((long)blockIdx.x * H + h) * R * DK;
    const int fr = lane & 15, kg = (lane >> 4) * 8;
    f32x4 acc[4];
#pragma unroll
    for (int c = 0; c < 4; ++c) acc[c] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
        const bf16x8 a =
            *(const bf16x8*)(vt + (wid * 16 + fr) * MLD + ks * 32 + kg);
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const int at = (c * 16 + fr) * MLD + ks * 32 + kg;
            acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                a, *(const bf16x8*)(kh + at), acc[c], 0, 0, 0);
            acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                a, *(const bf16x8*)(kl + at), acc[c], 0, 0, 0);
        }
    }
#pragma unroll
    for (int c = 0; c < 4; ++c)
#pragma unroll
        for (int r = 0; r < 4; ++r)
            Db[(long)(v0 + wid * 16 + (lane >> 4) * 4 + r) * DK + d0 + c * 16 +
               fr] = acc[c][r];
    if (!CONST && v0 == 0 && threadIdx.x < 64) {
        float s = 0.f;
        for (int t = 0; t < MCH; ++t)
            s += bf2f(kh[lane * MLD + t]) + bf2f(kl[lane * MLD + t]);
        Db[(long)DV * DK + d0 + lane] = s;
    }
}

template <bool CONST>
__global__ void __launch_bounds__(256)
k_mlstm_chunk_scan(float* __restrict__ dS, float* __restrict__ scal,
                   float* __restrict__ S, float* __restrict__ mst,
                   const int4* __restrict__ segs, int H, int DK, int DV) {
    const int4 sg = segs[blockIdx.x];
    const int h = blockIdx.y;
    const long size = (long)(CONST ? DV : DV + 1) * DK;
    const long e = (blockIdx.z * 256L + threadIdx.x) * 4;
    if (e >= size) return;
    float* Sb = S + ((long)sg.x * H + h) * size + e;
    float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
    if (sg.y != 0) s = *(const float4*)Sb;
    float m = scal[((long)sg.z * H + h) * 4 + 2];
    const long cs = (long)H * size;
    float* Db = dS + ((long)sg.z * H + h) * size + e;
    constexpr int U = 8;
    for (int c = 0; c < sg.w; c += U) {
        float4 d[U];
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (c + u < sg.w) d[u] = *(const float4*)(Db + (c + u) * cs);
#pragma unroll
        for (int u = 0; u < U; ++u) {
            if (c + u >= sg.w) break;
            float* sp = scal + ((long)(sg.z + c + u) * H + h) * 4;
            const float A = sp[0], Ft = sp[1];
            if (e == 0) sp[3] = m;
            uint4 pk;
            const float sv[4] = {s.x, s.y, s.z, s.w};
            u32* pp = (u32*)&pk;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const bf16_t hi = f2bf(sv[i]);
                pp[i] = (u32)hi | ((u32)f2bf(sv[i] - bf2f(hi)) << 16);
            }
            *(uint4*)(Db + (c + u) * cs) = pk;
            const float M = fmaxf(m, A);
            const float keep = expf(m - M), put = expf(A - M);
            s.x = keep * s.x + put * d[u].x;
            s.y = keep * s.y + put * d[u].y;
            s.z = keep * s.z + put * d[u].z;
            s.w = keep * s.w + put * d[u].w;
            m = Ft + M;
        }
    }
    *(float4*)Sb = s;
    if (!CONST && e == 0) mst[(long)sg.x * H + h] = m;
}

// 8 (hi | lo << 16) pairs -> the two bf16 fragments
DEV_INLINE void split8(const u32* p, bf16x8& hi, bf16x8& lo) {
    const uint4 x = ((const uint4*)p)[0], y = ((const uint4*)p)[1];
    uint4 a, b;
    a.x = (x.x & 0xffffu) | (x.y << 16);  b.x = (x.x >> 16) | (x.y & 0xffff0000u);
    a.y = (x.z & 0xffffu) | (x.w << 16);  b.y = (x.z >> 16) | (x.w & 0xffff0000u);
    a.z = (y.x & 0xffffu) | (y.y << 16);  b.z = (y.x >> 16) | (y.y & 0xffff0000u);
    a.w = (y.z & 0xffffu) | (y.w << 16);  b.w = (y.z >> 16) | (y.w & 0xffff0000u);
    hi = *(bf16x8*)&a;
    lo = *(bf16x8*)&b;
}

// Block = (chunk, head, 128 value columns); a wave owns 16 tokens.
template <bool CONST>
__global__ void __launch_bounds__(256, 2)
k_mlstm_chunk_out(float* __restrict__ o, const float* __restrict__ dS,
                  const float* __restrict__ scal,
                  const bf16_t* __restrict__ qkv,
                  const float* __restrict__ gr,
                  const int4* __restrict__ chunks, int H, int DK, int DV,
                  int ld_, float qscale, float cap) {
    __shared__ __attribute__((aligned(16))) bf16_t vt[128 * MLD];
    __shared__ __attribute__((aligned(16))) bf16_t ps[64 * MLD];
    __shared__ __attribute__((aligned(16))) bf16_t pl[CONST ? 64 * MLD : 8];
    __shared__ float sa[MCH], sM[MCH], sm[MCH], sin_[MCH], snq[MCH];
    const int4 ch = chunks[blockIdx.x];
    const int h = blockIdx.y, v0 = blockIdx.z * 128;
    const int nv = min(128, DV - v0);
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    if (wid == 0) {
        float F, a, amax;
        chunk_scan<CONST>(gr, ch.x, ch.y, h, H, cap, F, a, amax);
        const float m_in = scal[((long)blockIdx.x * H + h) * 4 + 3];
        const float M = fmaxf(m_in, amax);
        sa[lane] = a;
        sM[lane] = M;
        sm[lane] = F + M;
        sin_[lane] = expf(m_in - M);
    }
    for (int i = threadIdx.x; i < 64 * (nv / 8); i += 256) {
        const int t = i & 63, c8 = (i >> 6) * 8;
        const uint4 vv = *(const uint4*)(
            qkv + (long)(ch.x + min(t, ch.y - 1)) * ld_ + 2 * H * DK + h * DV +
            v0 + c8);
        const bf16_t* pv = (const bf16_t*)&vv;
#pragma unroll
        for (int j = 0; j < 8; ++j) vt[(c8 + j) * MLD + t] = pv[j];
    }
    __syncthreads();
    const int fr = lane & 15, kg = (lane >> 4) * 8, r0 = wid * 16;
    const u32* Sb = (const u32*)dS +
                    ((long)blockIdx.x * H + h) * (CONST ? DV : DV + 1) * DK;
    const bf16_t* qr = qkv + (long)(ch.x + min(r0 + fr, ch.y - 1)) * ld_ +
                       h * DK + kg;

    // ---- scores of this wave's tokens against the chunk's keys, and n . q
    f32x4 sc[4];
    const bf16_t* kr[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        sc[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
        kr[j] = qkv + (long)(ch.x + min(j * 16 + fr, ch.y - 1)) * ld_ +
                (H + h) * DK + kg;
    }
    float nq = 0.f;
    for (int k0 = 0; k0 < DK; k0 += 32) {
        const bf16x8 a = *(const bf16x8*)(qr + k0);
        if (!CONST) {
            float qf[8];
            unpack8(*(const uint4*)&a, qf);
            const u32* np = Sb + (long)DV * DK + k0 + kg;
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                const u32 w = np[i];
                nq += qf[i] * (__uint_as_float(w << 16) +
                               __uint_as_float(w & 0xffff0000u));
            }
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (j <= wid)
                sc[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                    a, *(const bf16x8*)(kr[j] + k0), sc[j], 0, 0, 0);
    }
    if (!CONST) {
        nq += __shfl_xor(nq, 16, WAVE);
        nq += __shfl_xor(nq, 32, WAVE);
        if (lane < 16) snq[r0 + lane] = nq;
    }
    float den[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        if (j > (wid | 1)) continue;
        const int key = j * 16 + fr;
        const float ak = sa[key];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = r0 + (lane >> 4) * 4 + r;
            const float p = (key <= row && key < ch.y)
                ? sc[j][r] * qscale * expf(ak - sM[row]) : 0.f;
            den[r] += p;
            ps[row * MLD + key] = f2bf(p);
            if (CONST)
                pl[row * MLD + key] = f2bf(p - bf2f(f2bf(p)));
        }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int off = 8; off > 0; off >>= 1)
            den[r] += __shfl_xor(den[r], off, WAVE);
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");   // own rows only

    // ---- what the entering state gives, then the chunk's own values
    f32x4 acc[8];
#pragma unroll
    for (int c = 0; c < 8; ++c) acc[c] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < DK; k0 += 32) {
        const bf16x8 a = *(const bf16x8*)(qr + k0);
#pragma unroll
        for (int c = 0; c < 8; ++c) {
            if (c * 16 >= nv) continue;
            bf16x8 hi, lo;
            split8(Sb + (long)(v0 + c * 16 + fr) * DK + k0 + kg, hi, lo);
            acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, hi, acc[c],
                                                             0, 0, 0);
            acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, lo, acc[c],
                                                             0, 0, 0);
        }
    }
    float inv[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int row = r0 + (lane >> 4) * 4 + r;
        const float in = sin_[row] * qscale;
        inv[r] = 1.f;
        if (!CONST) {
            const float d = den[r] + in * snq[row];
            inv[r] = 1.f / (fmaxf(fabsf(d), expf(-sm[row])) + 1e-6f);
        }
#pragma unroll
        for (int c = 0; c < 8; ++c) acc[c][r] *= in;
    }
    for (int ks = 0; ks <= (wid >> 1); ++ks) {
        const int at = (r0 + fr) * MLD + ks * 32 + kg;
        const bf16x8 a = *(const bf16x8*)(ps + at);
        bf16x8 al;
        if (CONST) al = *(const bf16x8*)(pl + at);
#pragma unroll
        for (int c = 0; c < 8; ++c) {
            if (c * 16 >= nv) continue;
            const bf16x8 v =
                *(const bf16x8*)(vt + (c * 16 + fr) * MLD + ks * 32 + kg);
            acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, v, acc[c],
                                                             0, 0, 0);
            if (CONST)
                acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                    al, v, acc[c], 0, 0, 0);
        }
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        const int row = r0 + (lane >> 4) * 4 + r;
        if (row >= ch.y) continue;
        float* ob = o + ((long)(ch.x + row) * H + h) * (DV + 4) + v0 + fr;
#pragma unroll
        for (int c = 0; c < 8; ++c)
            if (c * 16 < nv) ob[c * 16] = acc[c][r] * inv[r];
    }
}

// ===========================================================================
// Gated linear attention: S_t = diag(a_t) S_{t-1} + k_t v_t^T, o_t = S_t^T q_t
// with a_t = sigmoid(z_t)^(1 / tau) per key channel, q scaled by dim^-1/2.
// b holds the running sum of log a inside a chunk, f32 [n][H*DK] (a decode row
// is a chunk of its own). State and projection rows are laid out as mLSTM's,
// without the normaliser row.
// ===========================================================================

// b of one chunk for 256 channels: z = W2 u + bias with w = W2^T, f32 [R][C].
// The first items are U each of the first nd tokens, chunks of their own; then
// come the chunks ({first token, length, ..}).
template <int U>
__global__ void __launch_bounds__(256)
k_gla_decay(float* __restrict__ b, const float* __restrict__ u,
            const float* __restrict__ w, const float* __restrict__ bias,
            const int4* __restrict__ chunks, int nd, int R, int C,
            float inv_tau) {
    const int it = blockIdx.x, singles = (nd + U - 1) / U;
    int4 ch = make_int4(it * U, min(U, nd - it * U), 0, 0);
    if (it >= singles) ch = chunks[it - singles];
    const int c = blockIdx.y * 256 + threadIdx.x;
    if (c >= C) return;
    const float b0 = bias[c];
    float sum = 0.f;
    for (int t0 = 0; t0 < ch.y; t0 += U) {
        float z[U];
        const float* ur[U];
#pragma unroll
        for (int i = 0; i < U; ++i) {
            z[i] = b0;
            ur[i] = u + (long)(ch.x + min(t0 + i, ch.y - 1)) * R;
        }
        for (int rb = 0; rb < R; rb += 8) {    // 8 loads in flight
            float wv[8];
#pragma unroll
            for (int k = 0; k < 8; ++k)
                wv[k] = rb + k < R ? w[(long)(rb + k) * C + c] : 0.f;
#pragma unroll
            for (int k = 0; k < 8; ++k)
                if (rb + k < R)
#pragma unroll
                    for (int i = 0; i < U; ++i) z[i] += ur[i][rb + k] * wv[k];
        }
#pragma unroll
        for (int i = 0; i < U; ++i) {
            if (t0 + i >= ch.y) break;
            const float la =
                (fminf(z[i], 0.f) - log1pf(expf(-fabsf(z[i])))) * inv_tau;
            sum = it < singles ? la : sum + la;
            b[(long)(ch.x + t0 + i) * C + c] = sum;
        }
    }
}

// Prompt portions in chunks of 64 tokens, as mLSTM's: with b_t the sum of log
// decays up to token t and T the last token,
//   S_t = diag(exp(b_t)) S_in + sum_{s<=t} diag(exp(b_t - b_s)) k_s v_s^T
// Decays enter products as differences that are never positive where the span
// is unbounded, and as (hi, lo) pairs of bf16.
DEV_INLINE void split_bf16(float x, bf16_t& hi, bf16_t& lo) {
    hi = f2bf(x);
    lo = f2bf(x - bf2f(hi));
}

// A chunk's own contribution to the state. Block = (chunk, head, 64 key
// channels and every so many-th 64 value columns).
__global__ void __launch_bounds__(256)
k_gla_chunk_state(float* __restrict__ dS, const bf16_t* __restrict__ qkv,
                  const float* __restrict__ b, const int4* __restrict__ chunks,
                  int H, int DK, int DV, int ld_) {
    __shared__ __attribute__((aligned(16))) bf16_t vt[64 * MLD];
    __shared__ __attribute__((aligned(16))) bf16_t kh[64 * MLD];
    __shared__ __attribute__((aligned(16))) bf16_t kl[64 * MLD];
    const int4 ch = chunks[blockIdx.x];
    const int h = blockIdx.y;
    const int nd = DK / 64, nv = gridDim.z / nd;
    const int d0 = (blockIdx.z % nd) * 64;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const float* bl = b + (long)(ch.x + ch.y - 1) * H * DK + h * DK + d0;
    for (int i = threadIdx.x; i < 512; i += 256) {
        const int t = i & 63, c8 = (i >> 6) * 8;   // a wave spans 64 tokens
        const long n = ch.x + min(t, ch.y - 1);
        const bf16_t* row = qkv + n * ld_;
        float f[8], bt[8], bT[8];
        ld8(row + (H + h) * DK + d0 + c8, f);
        ld8(b + n * H * DK + h * DK + d0 + c8, bt);
        ld8(bl + c8, bT);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float x = t < ch.y ? f[j] * __expf(bT[j] - bt[j]) : 0.f;
            split_bf16(x, kh[(c8 + j) * MLD + t], kl[(c8 + j) * MLD + t]);
        }
    }
    float* Db = dS + ((long)blockIdx.x * H + h) * DV * DK;
    const int fr = lane & 15, kg = (lane >> 4) * 8;
    for (int v0 = blockIdx.z / nd * 64; v0 < DV; v0 += nv * 64) {
        __syncthreads();                 // readers of the last columns are done
        for (int i = threadIdx.x; i < 512; i += 256) {
            const int t = i & 63, c8 = (i >> 6) * 8;
            const uint4 vv = *(const uint4*)(
                qkv + (long)(ch.x + min(t, ch.y - 1)) * ld_ + 2 * H * DK +
                h * DV + v0 + c8);
            const bf16_t* pv = (const bf16_t*)&vv;
#pragma unroll
            for (int j = 0; j < 8; ++j) vt[(c8 + j) * MLD + t] = pv[j];
        }
        __syncthreads();
        f32x4 acc[4];
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[c] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            const bf16x8 a =
                *(const bf16x8*)(vt + (wid * 16 + fr) * MLD + ks * 32 + kg);
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                const int at = (c * 16 + fr) * MLD + ks * 32 + kg;
                acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                    a, *(const bf16x8*)(kh + at), acc[c], 0, 0, 0);
                acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                    a, *(const bf16x8*)(kl + at), acc[c], 0, 0, 0);
            }
        }
#pragma unroll
        for (int c = 0; c < 4; ++c)
#pragma unroll
            for (int r = 0; r < 4; ++r)
                Db[(long)(v0 + wid * 16 + (lane >> 4) * 4 + r) * DK + d0 +
                   c * 16 + fr] = acc[c][r];
    }
}

// The state that enters each chunk, left in dS as (hi | lo << 16) bf16 pairs;
// the slot's state is advanced.
__global__ void __launch_bounds__(256)
k_gla_chunk_scan(float* __restrict__ dS, float* __restrict__ S,
                 const float* __restrict__ b, const int4* __restrict__ chunks,
                 const int4* __restrict__ segs, int H, int DK, int DV) {
    const int4 sg = segs[blockIdx.x];
    const int h = blockIdx.y;
    const long size = (long)DV * DK;
    const long e = (blockIdx.z * 256L + threadIdx.x) * 4;
    if (e >= size) return;
    float* Sb = S + ((long)sg.x * H + h) * size + e;
    float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
    if (sg.y != 0) s = *(const float4*)Sb;
    const long cs = (long)H * size;
    float* Db = dS + ((long)sg.z * H + h) * size + e;
    const float* bc = b + h * DK + (int)(e % DK);
    constexpr int U = 8;
    for (int c = 0; c < sg.w; c += U) {
        float4 d[U], k[U];
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (c + u < sg.w) {
                const int4 ch = chunks[sg.z + c + u];
                d[u] = *(const float4*)(Db + (c + u) * cs);
                k[u] = *(const float4*)(bc + (long)(ch.x + ch.y - 1) * H * DK);
            }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            if (c + u >= sg.w) break;
            uint4 pk;
            const float sv[4] = {s.x, s.y, s.z, s.w};
            u32* pp = (u32*)&pk;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                bf16_t hi, lo;
                split_bf16(sv[i], hi, lo);
                pp[i] = (u32)hi | ((u32)lo << 16);
            }
            *(uint4*)(Db + (c + u) * cs) = pk;
            s.x = __expf(k[u].x) * s.x + d[u].x;
            s.y = __expf(k[u].y) * s.y + d[u].y;
            s.z = __expf(k[u].z) * s.z + d[u].z;
            s.w = __expf(k[u].w) * s.w + d[u].w;
        }
    }
    *(float4*)Sb = s;
}

// 8 values f[i] exp(e[i]) as the (hi, lo) pair of bf16 fragments
DEV_INLINE void decayed8(const bf16_t* p, const float* e, bf16x8& hi,
                         bf16x8& lo) {
    float f[8];
    ld8(p, f);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
        const float x = f[i] * __expf(e[i]);
        hi[i] = (__bf16)x;
        lo[i] = (__bf16)(x - (float)hi[i]);
    }
}

// hi . hi + hi . lo + lo . hi
DEV_INLINE f32x4 mfma_split(bf16x8 ah, bf16x8 al, bf16x8 bh, bf16x8 bl,
                            f32x4 c) {
    c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, bh, c, 0, 0, 0);
    c = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, bl, c, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, bh, c, 0, 0, 0);
}

// Block = (chunk, head, every gridDim.z-th 128 value columns); wave w owns
// tokens 16 w .. 16 w + 15. Scores refer to b at the end of the 16 tokens
// before: queries then decay by exp(b_t - ref) and older keys by
// exp(ref - b_s), both at most 1. Keys of the same 16 tokens grow by
// exp(ref - b_s) instead, unless a channel loses so much in 16 tokens that
// this could overflow; then these scores are taken pair by pair.
#define GLA_SPAN 60.f
__global__ void __launch_bounds__(256, 2)
k_gla_chunk_out(float* __restrict__ o, const float* __restrict__ dS,
                const bf16_t* __restrict__ qkv, const float* __restrict__ b,
                const int4* __restrict__ chunks, int H, int DK, int DV,
                int ld_, float qscale) {
    __shared__ __attribute__((aligned(16))) bf16_t vt[128 * MLD];
    __shared__ __attribute__((aligned(16))) bf16_t ph[64 * MLD];
    __shared__ __attribute__((aligned(16))) bf16_t pl[64 * MLD];
    const int4 ch = chunks[blockIdx.x];
    const int h = blockIdx.y;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int fr = lane & 15, kg = (lane >> 4) * 8, r0 = wid * 16;
    const long C = (long)H * DK;
    const int last = ch.y - 1;
    const float* bh = b + (long)ch.x * C + h * DK;     // row t at t * C
    const bf16_t* qh = qkv + (long)ch.x * ld_ + h * DK;
    const bf16_t* kh = qh + C;
    const int tq = min(r0 + fr, last);
    const float* ref = r0 ? bh + min(r0 - 1, last) * C : nullptr;

    // ---- does a channel lose too much within these 16 tokens?
    float span = 0.f;
    for (int c = lane; c < DK; c += 64)
        span = fmaxf(span, (ref ? ref[c] : 0.f) -
                               bh[min(r0 + 15, last) * C + c]);
    const bool pairwise = wave_reduce_max(span) > GLA_SPAN;

    // ---- scores
    f32x4 sc[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) sc[j] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int jmax = pairwise ? wid - 1 : wid;
    for (int k0 = 0; k0 < DK; k0 += 32) {
        const int c = k0 + kg;
        float rf[8], e[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) rf[i] = 0.f;
        if (ref) ld8(ref + c, rf);
        ld8(bh + tq * C + c, e);
#pragma unroll
        for (int i = 0; i < 8; ++i) e[i] -= rf[i];
        bf16x8 ah, al;
        decayed8(qh + (long)tq * ld_ + c, e, ah, al);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            if (j > jmax) continue;
            const int s = min(j * 16 + fr, last);
            ld8(bh + s * C + c, e);
#pragma unroll
            for (int i = 0; i < 8; ++i) e[i] = rf[i] - e[i];
            bf16x8 th, tl;
            decayed8(kh + (long)s * ld_ + c, e, th, tl);
            sc[j] = mfma_split(ah, al, th, tl, sc[j]);
        }
    }
    if (pairwise) {
        const int s = min(r0 + fr, last);
        const bf16_t* kr = kh + (long)s * ld_;
        const float* bs = bh + s * C;
        f32x4 d = {0.f, 0.f, 0.f, 0.f};
        for (int c = 0; c < DK; c += 4) {
            float kf[4], e[4];
            ld4(kr + c, kf);
            ld4(bs + c, e);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = min(r0 + (lane >> 4) * 4 + r, last);
                float qf[4], f[4];
                ld4(qh + (long)t * ld_ + c, qf);
                ld4(bh + t * C + c, f);
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    d[r] += qf[i] * kf[i] * __expf(fminf(f[i] - e[i], 0.f));
            }
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
            if (j == wid) sc[j] = d;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        if (j > (wid | 1)) continue;
        const int key = j * 16 + fr;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = r0 + (lane >> 4) * 4 + r;
            const float p = key <= row && key <= last ? sc[j][r] * qscale : 0.f;
            split_bf16(p, ph[row * MLD + key], pl[row * MLD + key]);
        }
    }
    // (rows of ph and pl are read by the wave that wrote them)

    const u32* Sb = (const u32*)dS + ((long)blockIdx.x * H + h) * DV * DK;
    for (int v0 = blockIdx.z * 128; v0 < DV; v0 += gridDim.z * 128) {
        const int nv = min(128, DV - v0);
        __syncthreads();                 // readers of the last columns are done
        for (int i = threadIdx.x; i < 64 * (nv / 8); i += 256) {
            const int t = i & 63, c8 = (i >> 6) * 8;
            const uint4 vv = *(const uint4*)(
                qkv + (long)(ch.x + min(t, last)) * ld_ + 2 * C + h * DV + v0 +
                c8);
            const bf16_t* pv = (const bf16_t*)&vv;
#pragma unroll
            for (int j = 0; j < 8; ++j) vt[(c8 + j) * MLD + t] = pv[j];
        }
        __syncthreads();
        // ---- what the entering state gives, then the chunk's own values
        f32x4 acc[8];
#pragma unroll
        for (int c = 0; c < 8; ++c) acc[c] = (f32x4){0.f, 0.f, 0.f, 0.f};
        for (int k0 = 0; k0 < DK; k0 += 32) {
            float e[8];
            ld8(bh + tq * C + k0 + kg, e);
            bf16x8 ah, al;
            decayed8(qh + (long)tq * ld_ + k0 + kg, e, ah, al);
#pragma unroll
            for (int c = 0; c < 8; ++c) {
                if (c * 16 >= nv) continue;
                bf16x8 hi, lo;
                split8(Sb + (long)(v0 + c * 16 + fr) * DK + k0 + kg, hi, lo);
                acc[c] = mfma_split(ah, al, hi, lo, acc[c]);
            }
        }
#pragma unroll
        for (int c = 0; c < 8; ++c)
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[c][r] *= qscale;
        for (int ks = 0; ks <= (wid >> 1); ++ks) {
            const int at = (r0 + fr) * MLD + ks * 32 + kg;
            const bf16x8 ah = *(const bf16x8*)(ph + at);
            const bf16x8 al = *(const bf16x8*)(pl + at);
#pragma unroll
            for (int c = 0; c < 8; ++c) {
                if (c * 16 >= nv) continue;
                const bf16x8 v =
                    *(const bf16x8*)(vt + (c * 16 + fr) * MLD + ks * 32 + kg);
                acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                    ah, v, acc[c], 0, 0, 0);
                acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                    al, v, acc[c], 0, 0, 0);
            }
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int row = r0 + (lane >> 4) * 4 + r;
            if (row > last) continue;
            float* ob = o + ((long)(ch.x + row) * H + h) * (DV + 4) + v0 + fr;
#pragma unroll
            for (int c = 0; c < 8; ++c)
                if (c * 16 < nv) ob[c * 16] = acc[c][r];
        }
    }
}

// ===========================================================================
// Routed experts.
//   route:   top experts of every token by f32 logits (ties: lower index),
//            their weights, by softmax or (plain) sigmoids; counts per expert
//            and each pair's rank. The choice may add a correction per expert
//            to the softmax scores and be confined to the best of equal groups;
//            router outputs beyond the experts are identities, whose weights
//            are summed up apart
//   scatter: pairs (token * top + k) sorted by expert, and the tile list
//            {expert, first sorted row, rows, -}; entry max_tiles holds the
//            number of tiles
//   gemm:    rows of one expert against its weights, once for the up
//            projection (gathers token rows, times the pairs' weights if these
//            go with the input; squared ReLU or a gated unit) and once for the
//            down projection (writes each pair's row back in pair order)
// The (weighted) sum over a token's pairs is taken in k_post_norm, k_sum_norm
// or k_streams_join.
// ===========================================================================
//
// A wave routes `tpw` tokens, one expert per lane and VPL experts deep. The
// place of an expert among a token's logits is the number of larger ones, so
// the chosen fall out of one pass over the lanes. Counts are gathered per
// block in LDS and added up once per block and expert.
template <int VPL>
__global__ void __launch_bounds__(256)
k_moe_route(int* __restrict__ idx, float* __restrict__ wt,
            int* __restrict__ rank, int* __restrict__ counts,
            const float* __restrict__ z, int ldz,
            const float* __restrict__ corr, float* __restrict__ ident, int N,
            int E, int experts, int top, int groups, int keep, float eps,
            float scale, int sigmoid, int tpw) {
    __shared__ int cnt[VPL * 64], base[VPL * 64];
    __shared__ float cs[4][VPL * 64], gm[4][VPL * 64];
    for (int e = threadIdx.x; e < VPL * 64; e += 256) cnt[e] = 0;
    __syncthreads();
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int n0 = (blockIdx.x * 4 + wid) * tpw;
    for (int n = n0; n < min(N, n0 + tpw); ++n) {
        float v[VPL], s[VPL];          // choice score, score
        int place[VPL];
        float mx = -INFINITY;
#pragma unroll
        for (int i = 0; i < VPL; ++i) {
            const int e = i * 64 + lane;
            v[i] = e < E ? z[(long)n * ldz + e] : -INFINITY;
            if (v[i] != v[i]) v[i] = -INFINITY;   // keeps the choice in range
            place[i] = 0;
            mx = fmaxf(mx, v[i]);
        }
        mx = wave_reduce_max(mx);
        float total = 0.f;
#pragma unroll
        for (int i = 0; i < VPL; ++i) {
            s[i] = i * 64 + lane >= E ? 0.f
                   : sigmoid ? sigmoidf_(v[i]) : expf(v[i] - mx);
            total += s[i];
        }
        total = sigmoid ? 1.f : wave_reduce_sum(total);
#pragma unroll
        for (int i = 0; i < VPL; ++i) {
            const int e = i * 64 + lane;
            s[i] /= total;
            if (corr && e < E) {
                v[i] = s[i] + corr[e];
                if (v[i] != v[i]) v[i] = -INFINITY;
            }
        }
        if (groups > 1) {
            // a group's score is its largest; the others' experts drop out
            const int gs = E / groups;
            asm volatile("" ::: "memory");
#pragma unroll
            for (int i = 0; i < VPL; ++i) cs[wid][i * 64 + lane] = v[i];
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // own wave's
            for (int g = lane; g < groups; g += 64) {
                float a = -INFINITY;
#pragma unroll 4
                for (int j = 0; j < gs; ++j) a = fmaxf(a, cs[wid][g * gs + j]);
                gm[wid][g] = a;
            }
            asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
#pragma unroll
            for (int i = 0; i < VPL; ++i) {
                const int e = i * 64 + lane;
                if (e >= E) continue;
                const int own = e / gs;
                const float a = gm[wid][own];
                int ahead = 0;
#pragma unroll 4
                for (int g = 0; g < groups; ++g) {
                    const float b = gm[wid][g];
                    ahead += b > a || (b == a && g < own);
                }
                if (ahead >= keep) v[i] = -INFINITY;
            }
        }
#pragma unroll
        for (int j = 0; j < VPL; ++j) {
            const int last = min(64, E - j * 64);
#pragma unroll 8
            for (int l = 0; l < last; ++l) {
                const float o = __uint_as_float(
                    __builtin_amdgcn_readlane(__float_as_uint(v[j]), l));
#pragma unroll
                for (int i = 0; i < VPL; ++i)
                    place[i] += i > j ? o >= v[i] : i < j ? o > v[i]
                        : o > v[i] || (o == v[i] && l < lane);
            }
        }
        float sum = 0.f;
#pragma unroll
        for (int i = 0; i < VPL; ++i)
            sum += place[i] < top && i * 64 + lane < E ? s[i] : 0.f;
        sum = wave_reduce_sum(sum);
        float same = 0.f;
#pragma unroll
        for (int i = 0; i < VPL; ++i) {
            const int e = i * 64 + lane;
            if (place[i] >= top || e >= E) continue;
            const long at = (long)n * top + place[i];
            const float w = sigmoid ? s[i] : s[i] / (sum + eps) * scale;
            idx[at] = e;
            wt[at] = e < experts ? w : 0.f;
            if (e >= experts) same += w;
            rank[at] = atomicAdd(cnt + e, 1);       // within the block
        }
        if (ident) {
            same = wave_reduce_sum(same);
            if (lane == 0) ident[n] = same;
        }
    }
    __syncthreads();
    for (int e = threadIdx.x; e < E; e += 256)
        base[e] = cnt[e] ? atomicAdd(counts + e, cnt[e]) : 0;
    __syncthreads();
    const long p0 = (long)blockIdx.x * 4 * tpw * top;
    const long p1 = min((long)N * top, p0 + 4L * tpw * top);
    for (long at = p0 + threadIdx.x; at < p1; at += 256)
        rank[at] += base[idx[at]];
}

__global__ void __launch_bounds__(256)
k_moe_scatter(int* __restrict__ sorted, int4* __restrict__ tiles,
              const int* __restrict__ idx, const int* __restrict__ rank,
              const int* __restrict__ counts, int pairs, int E, int bm,
              int max_tiles) {          // E: experts that have weights
    __shared__ int off[1025], toff[1025];
    for (int e = threadIdx.x; e < E; e += 256) off[e + 1] = counts[e];
    if (threadIdx.x == 0) off[0] = toff[0] = 0;
    __syncthreads();
    if (threadIdx.x < 64) {            // one wave scans, 64 experts a turn
        int base = 0, tbase = 0;
        for (int e0 = 0; e0 < E; e0 += 64) {
            const int e = e0 + threadIdx.x;
            int c = e < E ? off[e + 1] : 0;
            int t = (c + bm - 1) / bm;
#pragma unroll
            for (int s = 1; s < 64; s <<= 1) {
                const int a = __shfl_up(c, s, WAVE);
                const int b = __shfl_up(t, s, WAVE);
                if ((int)threadIdx.x >= s) { c += a; t += b; }
            }
            if (e < E) { off[e + 1] = base + c; toff[e + 1] = tbase + t; }
            base += __shfl(c, 63, WAVE);
            tbase += __shfl(t, 63, WAVE);
        }
    }
    __syncthreads();
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i < pairs && idx[i] < E) {
        const int at = off[idx[i]] + rank[i];
        if (at >= 0 && at < pairs) sorted[at] = i;
    }
    if (blockIdx.x == 0) {
        for (int e = threadIdx.x; e < E; e += 256) {
            const int n = off[e + 1] - off[e];
            for (int t = 0; t * bm < n; ++t)
                if (toff[e] + t < max_tiles)
                    tiles[toff[e] + t] = make_int4(e, off[e] + t * bm,
                                                   min(bm, n - t * bm), 0);
        }
        if (threadIdx.x == 0)
            tiles[max_tiles] = make_int4(min(toff[E], max_tiles), 0, 0, 0);
    }
}

DEV_INLINE float sq_relu(float v) {
    v = fmaxf(v, 0.f);
    return v * v;
}

// Work item of this block: tiles of neighbouring numbers (the columns of one
// row tile, then the next row tile of the expert) go to the same XCD, whose L2
// then holds the rows and weights they share. Blocks are dealt to the 8 XCDs
// in turn, and only the tiles in use are counted. Returns false if none is
// left for the block.
DEV_INLINE bool moe_work(const int4* tiles, int max_tiles, int ntn, int4& tl,
                         int& nt) {
    const int total = tiles[max_tiles].x * ntn;
    const int per = (total + 7) >> 3;
    const int i = (blockIdx.x & 7) * per + (blockIdx.x >> 3);
    if ((int)(blockIdx.x >> 3) >= per || i >= total) return false;
    tl = tiles[i / ntn];
    nt = i % ntn;
    return true;
}

// 128 rows x 128 columns per block, 4 waves of 64 x 64, both
// operands through LDS by global_load_lds (source addresses pre-swizzled so
// that the lane-linear image reads back without bank conflicts), NB buffers.
// With few rows per expert the same pipeline streams the weights.
// ACT != 0 (up projection): row r of the tile is token sorted[row0 + r] / top,
// output in sorted order through squared ReLU (1) or, with weight rows in turns
// of 16 gate | 16 up, the gated unit `glu` in N / 2 columns (2); pw (nullable):
// a weight per pair on the unit's input. ACT 0: row r is sorted row row0 + r and
// its output goes to pair order. The MFMA computes W x^T, so a lane ends up with
// 4 neighbouring columns of one row.
// K % 64 == 0, N % 64 == 0 (ACT 2: N % 128 == 0).
template <int ACT, int NB>
__global__ void __launch_bounds__(256, 2)
k_moe_gemm(bf16_t* __restrict__ out, const bf16_t* __restrict__ x,
           const bf16_t* __restrict__ w, const int4* __restrict__ tiles,
           const int* __restrict__ sorted, int top, int N, int K, int ntn,
           int max_tiles, const GluParams glu, const float* __restrict__ pw) {
    constexpr int BK = 64, TB = 256 * BK, GL = 8;
    constexpr bool UP = ACT != 0;
    const int NO = ACT == 2 ? N / 2 : N;
    __shared__ __attribute__((aligned(16))) bf16_t lds[NB * TB];
    int4 tl;
    int nti;
    if (!moe_work(tiles, max_tiles, ntn, tl, nti)) return;
    const int n0 = nti * 128;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int fr = lane & 15, kg = (lane >> 4) * 8;
    const int lrow = lane >> 3, lkb = (lane & 7) * 16;
    const char* src[GL];
#pragma unroll
    for (int i = 0; i < GL; ++i) {     // pieces of 8 rows: 16 of x, 16 of w
        const int piece = (i < 4 ? wid * 4 + i : 16 + wid * 4 + i - 4);
        const int row = (piece & 15) * 8 + lrow;
        const bf16_t* p;
        if (piece < 16) {
            const int r = tl.y + min(row, tl.z - 1);
            p = x + (long)(UP ? sorted[r] / top : r) * K;
        } else {
            p = w + ((long)tl.x * N + min(n0 + row, N - 1)) * K;
        }
        src[i] = (const char*)p + (lkb ^ ((row & 7) << 4));
    }
    auto issue = [&](int buf, int kt) {
#pragma unroll
        for (int i = 0; i < GL; ++i) {
            const int piece = (i < 4 ? wid * 4 + i : 16 + wid * 4 + i - 4);
            __builtin_amdgcn_global_load_lds(
                (const __attribute__((address_space(1))) unsigned int*)
                    (src[i] + (long)kt * BK * 2),
                (__attribute__((address_space(3))) unsigned int*)
                    (lds + buf * TB + piece * 512), 16, 0, 0);
        }
    };
    f32x4 acc[4][4];
#pragma unroll
    for (int a = 0; a < 4; ++a)
#pragma unroll
        for (int b = 0; b < 4; ++b) acc[a][b] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int nt = K / BK;
    const int wr = (wid >> 1) * 64, wc = (wid & 1) * 64;
#pragma unroll
    for (int u = 0; u < NB - 1; ++u)
        if (u < nt) issue(u, u);
    for (int kt = 0; kt < nt; ++kt) {
        if (kt + NB - 1 < nt)
            asm volatile("s_waitcnt vmcnt(%0)" :: "i"(GL * (NB - 2)) : "memory");
        else
            asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __builtin_amdgcn_s_barrier();
        if (kt + NB - 1 < nt) issue((kt + NB - 1) % NB, kt + NB - 1);
        const char* xb = (const char*)(lds + (kt % NB) * TB);
        const char* wb = xb + 128 * BK * 2;
#pragma unroll
        for (int kc = 0; kc < 2; ++kc) {
            bf16x8 b[4];
#pragma unroll
            for (int c = 0; c < 4; ++c) {
                const int row = wc + c * 16 + fr;
                b[c] = *(const bf16x8*)(wb + row * 128 +
                    (((kc * 32 + kg) * 2) ^ ((row & 7) << 4)));
            }
#pragma unroll
            for (int a = 0; a < 4; ++a) {
                const int row = wr + a * 16 + fr;
                const bf16x8 av = *(const bf16x8*)(xb + row * 128 +
                    (((kc * 32 + kg) * 2) ^ ((row & 7) << 4)));
#pragma unroll
                for (int c = 0; c < 4; ++c)
                    acc[a][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                        b[c], av, acc[a][c], 0, 0, 0);
            }
        }
    }
#pragma unroll
    for (int a = 0; a < 4; ++a) {
        const int m = wr + a * 16 + fr;
        if (m >= tl.z) continue;
        bf16_t* orow = out + (UP ? (long)tl.y + m : sorted[tl.y + m]) *
                                 (long)NO;
        const float wi = ACT == 2 && pw ? pw[sorted[tl.y + m]] : 1.f;
#pragma unroll
        for (int c = 0; c < 4; c += ACT == 2 ? 2 : 1) {
            const int n = (ACT == 2 ? (n0 + wc + c * 16) / 2
                                    : n0 + wc + c * 16) + (lane >> 4) * 4;
            float f[4];
#pragma unroll
            for (int r = 0; r < 4; ++r)
                f[r] = ACT == 2 ? glu_act(wi * acc[a][c][r],
                                          wi * acc[a][(c + 1) & 3][r], glu)
                     : ACT == 1 ? sq_relu(acc[a][c][r]) : acc[a][c][r];
            if (n < NO) st4(orow + n, f);
        }
    }
}

// A few rows: up to 16 against 16 columns per block, K split over the 4 waves,
// so that a handful of experts still fills the chip. (16 output columns: 32
// weight rows if gated.)
template <int ACT>
__global__ void __launch_bounds__(256)
k_moe_gemm_few(bf16_t* __restrict__ out, const bf16_t* __restrict__ x,
               const bf16_t* __restrict__ w, const int4* __restrict__ tiles,
               const int* __restrict__ sorted, int top, int N, int K,
               int ntn, int max_tiles, const GluParams glu,
               const float* __restrict__ pw) {
    constexpr int U = 8, NW = ACT == 2 ? 2 : 1;
    constexpr bool UP = ACT != 0;
    __shared__ __attribute__((aligned(16))) float red[NW][4][16][20];
    int4 tl;
    int nti;
    if (!moe_work(tiles, max_tiles, ntn, tl, nti)) return;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int fr = lane & 15, kg = (lane >> 4) * 8;
    const int n0 = nti * 16 * NW;
    const bf16_t* wr = w + ((long)tl.x * N + n0 + fr) * K + kg;
    const int r = tl.y + min(fr, tl.z - 1);
    const bf16_t* xr = x + (long)(UP ? sorted[r] / top : r) * K + kg;
    f32x4 acc[NW];
#pragma unroll
    for (int t = 0; t < NW; ++t) acc[t] = (f32x4){0.f, 0.f, 0.f, 0.f};
    const int steps = K >> 5;
    for (int s0 = wid; s0 < steps; s0 += 4 * U) {
        bf16x8 a[U], b[U][NW];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int s = min(s0 + u * 4, steps - 1);
#pragma unroll
            for (int t = 0; t < NW; ++t)
                b[u][t] = __builtin_nontemporal_load(
                    (const bf16x8*)(wr + (long)t * 16 * K + s * 32));
            a[u] = *(const bf16x8*)(xr + s * 32);
        }
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (s0 + u * 4 < steps)
#pragma unroll
                for (int t = 0; t < NW; ++t)
                    acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                        b[u][t], a[u], acc[t], 0, 0, 0);
    }
#pragma unroll
    for (int t = 0; t < NW; ++t)
        *(f32x4*)&red[t][wid][fr][(lane >> 4) * 4] = acc[t];
    __syncthreads();
    const int m = threadIdx.x >> 4, c = threadIdx.x & 15;
    if (m >= tl.z) return;
    float v[NW];
#pragma unroll
    for (int t = 0; t < NW; ++t)
        v[t] = red[t][0][m][c] + red[t][1][m][c] + red[t][2][m][c] +
               red[t][3][m][c];
    const float wi = ACT == 2 && pw ? pw[sorted[tl.y + m]] : 1.f;
    out[(UP ? (long)tl.y + m : sorted[tl.y + m]) * (long)(N / NW) + nti * 16 +
        c] = f2bf(ACT == 2 ? glu_act(wi * v[0], wi * v[NW - 1], glu)
                           : ACT == 1 ? sq_relu(v[0]) : v[0]);
}

// Exact mode: 16 rows x 64 weight rows per block, f32 products.
template <int ACT>
__global__ void __launch_bounds__(256)
k_moe_gemm_f32(float* __restrict__ out, const float* __restrict__ x,
               const float* __restrict__ w, const int4* __restrict__ tiles,
               const int* __restrict__ sorted, int top, int N, int K,
               int ntn, int max_tiles, const GluParams glu,
               const float* __restrict__ pw) {
    constexpr bool UP = ACT != 0;
    __shared__ float xs[16][33], ws[64][33];
    int4 tl;
    int nti;
    if (!moe_work(tiles, max_tiles, ntn, tl, nti)) return;
    const int n0 = nti * 64;
    const int col = threadIdx.x & 63, r4 = (threadIdx.x >> 6) * 4;
    float acc[4] = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < K; k0 += 32) {
        for (int i = threadIdx.x; i < 16 * 32; i += 256) {
            const int r = tl.y + min(i >> 5, tl.z - 1);
            xs[i >> 5][i & 31] =
                x[(long)(UP ? sorted[r] / top : r) * K + k0 + (i & 31)];
        }
        for (int i = threadIdx.x; i < 64 * 32; i += 256)
            ws[i >> 5][i & 31] =
                w[((long)tl.x * N + n0 + (i >> 5)) * K + k0 + (i & 31)];
        __syncthreads();
#pragma unroll
        for (int k = 0; k < 32; ++k) {
            const float wv = ws[col][k];
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[r] += xs[r4 + r][k] * wv;
        }
        __syncthreads();
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) {
        float v = ACT == 1 ? sq_relu(acc[r]) : acc[r];
        if (ACT == 2) {
            if (pw) v *= pw[sorted[tl.y + min(r4 + r, tl.z - 1)]];
            const float u = fminf(fmaxf(__shfl_down(v, 16, WAVE), -glu.limit),
                                  glu.limit);
            v = fminf(v, glu.limit);
            const float z = glu.alpha * v * (1.f + glu.cubic * v * v);
            v = v / (1.f + expf(-z)) * (u + glu.shift);
        }
        if (r4 + r >= tl.z) continue;
        const long dst = UP ? tl.y + r4 + r : sorted[tl.y + r4 + r];
        if (ACT != 2)
            out[dst * N + n0 + col] = v;
        else if (!(col & 16))
            out[dst * (N / 2) + n0 / 2 + (col & 32) / 2 + (col & 15)] = v;
    }
}

// ===========================================================================
// Entry points. f32 != 0 selects the exact mode. 0 = success.
// ===========================================================================
template <int D, int G>
static void launch_paged_decode(hipStream_t st, void* out, const void* q,
                                const PagedKV<D>& kv, const int* pos,
                                const int* slot, float* ws, int B, int ngrp,
                                int nsplit, float scale,
                                const HeadEpilogue& epi,
                                const WindowKeys& keys) {
    const dim3 grid((unsigned)(B * kv.Hk * ngrp * nsplit));
    if (nsplit == 1 && B * kv.Hk * ngrp >= 2048)
        k_attn_decode1<D, G><<<grid, dim3(64), 0, st>>>(
            (bf16_t*)out, (const bf16_t*)q, kv, pos, 1, slot, ws, ngrp,
            nsplit, scale, epi, keys);
    else
        k_attn_decode<D, G><<<grid, dim3(256), 0, st>>>(
            (bf16_t*)out, (const bf16_t*)q, kv, pos, 1, slot, ws, ngrp,
            nsplit, scale, epi, keys);
}

template <int D>
static int paged_decode(hipStream_t st, void* out, const void* q,
                        const void* kc, const void* vc, const int* table,
                        int per_slot, const int* pos, const int* slot,
                        float* ws, int B, int Hq, int Hk, int nsplit,
                        float scale, const HeadEpilogue& epi,
                        const WindowKeys& keys) {
    const PagedKV<D> kv{(const bf16_t*)kc, (const bf16_t*)vc, table, Hk,
                        per_slot};
    const int per = Hq / Hk;
    int g = per;
    if (g > MAXG) for (g = MAXG; per % g; --g) {}
    switch (g) {
#define CASE_G(GG) case GG: launch_paged_decode<D, GG>(st, out, q, kv, pos, \
        slot, ws, B, per / GG, nsplit, scale, epi, keys); break;
        CASE_G(1) CASE_G(2) CASE_G(3) CASE_G(4)
        CASE_G(5) CASE_G(6) CASE_G(7) CASE_G(8)
#undef CASE_G
        default: return -102;
    }
    LAUNCH_CHECK();
    if (nsplit > 1) {
        k_attn_combine<<<dim3((unsigned)(B * Hq)), dim3(D), 0, st>>>(
            (bf16_t*)out, ws, Hq, D, nsplit, epi);
        LAUNCH_CHECK();
    }
    return 0;
}

extern "C" {

int gh_embed(void* stream, int f32, void* x, void* xb, const void* emb,
             const void* ptab, const void* tok, const void* pos,
             const void* w, float w_off, int N, int W, int Wtrue, float eps,
             int vocab, int max_pos) {
    if (W % 64 || N < 1) return -100;
    hipStream_t st_ = (hipStream_t)stream;
#define GO(T) k_embed<T><<<N, 256, 0, st_>>>((float*)x, (T*)xb, \
        (const T*)emb, (const T*)ptab, (const long long*)tok, \
        (const int*)pos, (const float*)w, w_off, W, Wtrue, eps, vocab, max_pos)
    if (f32) GO(float); else GO(bf16_t);
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_sum_norm(void* stream, int f32, void* xo, void* xb, const void* x,
                const void* y, const void* wt, int top, const void* ident,
                const void* w, float w_off, float alpha, void* hist,
                const void* coef, int nh, int keep, int N, int W, int Wtrue,
                float eps) {
    if (W % 64 || W > 8192 || N < 1 || (hist && nh < 1)) return -100;
    hipStream_t st_ = (hipStream_t)stream;
#define GO(T, M) k_sum_norm<T, M><<<N, 256, 0, st_>>>((float*)xo, (T*)xb, \
        (const float*)x, (const T*)y, (const float*)wt, top, \
        (const float*)ident, (const float*)w, w_off, alpha, (float*)hist, \
        (const float*)coef, nh, keep, N, W, Wtrue, eps)
    if (f32) { if (wt) GO(float, true); else GO(float, false); }
    else { if (wt) GO(bf16_t, true); else GO(bf16_t, false); }
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_post_norm(void* stream, int f32, void* x, void* xb, const void* y,
                 const void* wt, int top, const void* w, float w_off, int N,
                 int W, int Wtrue, float eps) {
    if (W % 64 || W > 8192 || N < 1) return -100;
    hipStream_t st_ = (hipStream_t)stream;
#define GO(T, M) k_post_norm<T, M><<<N, 256, 0, st_>>>((float*)x, (T*)xb, \
        (const T*)y, (const float*)wt, top, (const float*)w, w_off, W, Wtrue, \
        eps)
    if (f32) { if (wt) GO(float, true); else GO(float, false); }
    else { if (wt) GO(bf16_t, true); else GO(bf16_t, false); }
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_norm_rows(void* stream, int f32, void* out, const void* x,
                 const void* rows, const void* w, float w_off, int M, int W,
                 int Wtrue, float eps) {
    if (W % 64 || M < 1) return -100;
    hipStream_t st_ = (hipStream_t)stream;
    if (f32)
        k_norm_rows<float><<<M, 256, 0, st_>>>((float*)out, (const float*)x,
            (const int*)rows, (const float*)w, w_off, W, Wtrue, eps);
    else
        k_norm_rows<bf16_t><<<M, 256, 0, st_>>>((bf16_t*)out, (const float*)x,
            (const int*)rows, (const float*)w, w_off, W, Wtrue, eps);
    LAUNCH_CHECK();
    return 0;
}

int gh_group_norm(void* stream, int f32, void* out, void* x, const void* y,
                  const void* rows, const void* wy, const void* w, int N,
                  int W, int groups, int size, float eps) {
    if (N < 1 || W % 8 || W > 8192 || groups < 1 || size < 1 ||
        (long)groups * size > W || (!y && !out) || (y && rows)) return -100;
    const int gr = size % 8 == 0 ? 8 : size % 4 == 0 ? 4 : size % 2 ? 1 : 2;
    const int lds = (W / gr + groups) * 4;
    if (lds > 64 * 1024) return -100;
    const Groups gp{groups, size};
#define GO(T, A, B) k_group_norm<T, A, B><<<N, 256, lds, \
        (hipStream_t)stream>>>((T*)out, (float*)x, (const T*)y, \
        (const int*)rows, (const float*)wy, (const float*)w, W, gp, eps)
#define PICK(T, A) do { if (gr == 8) GO(T, A, 8); else if (gr == 4) \
        GO(T, A, 4); else if (gr == 2) GO(T, A, 2); else GO(T, A, 1); \
        } while (0)
    if (f32) { if (y) PICK(float, true); else PICK(float, false); }
    else { if (y) PICK(bf16_t, true); else PICK(bf16_t, false); }
#undef PICK
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_poly_norm(void* stream, int f32, void* out, const void* z,
                 const void* coef, int N, int F, int Ftrue, float eps) {
    if (N < 1 || F % 8 || Ftrue < 1 || Ftrue > F) return -100;
#define GO(T, NV) k_poly_norm<T, NV><<<N, 256, 0, (hipStream_t)stream>>>( \
        (T*)out, (const T*)z, (const float*)coef, F, Ftrue, eps)
#define PICK(T) do { if (F <= 4096) GO(T, 2); else if (F <= 8192) GO(T, 4); \
        else if (F <= 16384) GO(T, 8); else GO(T, 0); } while (0)
    if (f32) PICK(float); else PICK(bf16_t);
#undef PICK
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_glu_f32(void* stream, void* out, const void* gu, long n, int F,
               float alpha, float limit, float shift, float cubic) {
    if (n < 1) return -100;
    const int grid = (int)min((n * F + 255) / 256, (long)4096);
    k_glu_f32<<<grid, 256, 0, (hipStream_t)stream>>>(
        (float*)out, (const float*)gu, n, F,
        GluParams{alpha, limit, shift, cubic});
    LAUNCH_CHECK();
    return 0;
}

int gh_proj_f32(void* stream, void* out, const void* x, const void* w,
                const void* bias, int M, int N, int K) {
    if (K % 32 || M < 1 || N < 1) return -100;
    hipStream_t st_ = (hipStream_t)stream;
#define GO(NT) k_proj_f32<NT><<<dim3((M + 15) / 16, \
        (N + 16 * NT - 1) / (16 * NT)), 512, 0, st_>>>((float*)out, \
        (const bf16_t*)x, (const bf16_t*)w, (const float*)bias, M, N, K)
    // few rows: narrow blocks, so that more of them stream the weights
    if (M <= 512 || N <= 16) GO(1);
    else if (N <= 32) GO(2);
    else if ((N + 79) / 80 < (N + 63) / 64) GO(5);
    else GO(4);
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_streams_start(void* stream, int f32, void* x, void* h, const void* emb,
                     const void* tok, float scale, const void* in,
                     const void* w, int N, int ns, int W, int Wtrue, float eps,
                     int vocab) {
    if (N < 1 || ns < 1 || W % 64 || W > 8192) return -100;
#define GO(T) k_streams_start<T><<<N, 256, 0, (hipStream_t)stream>>>( \
        (float*)x, (T*)h, (const T*)emb, (const long long*)tok, scale, \
        (const float*)in, (const float*)w, ns, W, Wtrue, eps, vocab)
    if (f32) GO(float); else GO(bf16_t);
#undef GO
    LAUNCH_CHECK();
    return 0;
}

// moe: y holds `top` rows per token, and extra (nullable) one more
int gh_streams_join(void* stream, int f32, int moe, void* x, void* h,
                    const void* y, int top, const void* extra,
                    const void* extra_z, int extra_ld, const void* hc,
                    const void* in, const void* w, int N, int ns, int W,
                    int Wtrue, float eps) {
    if (N < 1 || ns < 1 || ns > 16 || W % 64 || W > 8192 ||
        (moe && top < 1) || (h && !(in && w)) || (extra && !extra_z))
        return -100;
#define GO(T, S, NV, M) k_streams_join<T, S, NV, M><<<N, 256, 0, \
        (hipStream_t)stream>>>((float*)x, (T*)h, (const T*)y, top, \
        (const T*)extra, (const float*)extra_z, extra_ld, (const float*)hc, \
        (const float*)in, (const float*)w, ns, W, Wtrue, eps)
#define PICKV(T, S, M) do { if (W <= 4096) GO(T, S, 2, M); \
        else GO(T, S, 4, M); } while (0)
#define PICK(T, M) do { if (ns == 1) PICKV(T, 1, M); \
        else if (ns == 2) PICKV(T, 2, M); else if (ns <= 4) PICKV(T, 4, M); \
        else if (ns <= 8) GO(T, 8, 4, M); else GO(T, 16, 4, M); } while (0)
    if (f32) { if (moe) PICK(float, true); else PICK(float, false); }
    else { if (moe) PICK(bf16_t, true); else PICK(bf16_t, false); }
#undef PICK
#undef PICKV
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_streams_norm(void* stream, int f32, void* out, const void* x,
                    const void* rows, const void* w, int M, int ns, int W,
                    int Wtrue, float eps) {
    if (M < 1 || ns < 1 || W % 64 || W > 8192) return -100;
#define GO(T) k_streams_norm<T><<<M, 256, 0, (hipStream_t)stream>>>((T*)out, \
        (const float*)x, (const int*)rows, (const float*)w, ns, W, Wtrue, eps)
    if (f32) GO(float); else GO(bf16_t);
#undef GO
    LAUNCH_CHECK();
    return 0;
}

// cos_ and sin_ (nullable): tables of rot_rows x rot_half; act_0, act_n:
// columns that get SiLU in place (which may be all there is: H and G 0)
int gh_qknorm_kv(void* stream, int f32, void* qkv, void* q_out,
                 void* kc, void* vc, const void* table, int per_slot,
                 const void* pos, const void* slot, int N, int H, int G,
                 int P, int ld_, int dim, float eps, float coef, int every,
                 const void* cos_, const void* sin_, int rot_half,
                 int rot_rows, int act_0, int act_n) {
    if (N < 1 || (G ? H % G : H) || every < 1 || rot_half % 4 || 2 * rot_half > P ||
        act_0 % 8 || act_n % 8 || act_0 + act_n > ld_ || ld_ % 8)
        return -100;
    hipStream_t st_ = (hipStream_t)stream;
    const Rotation rot{(const float*)cos_, (const float*)sin_,
                       cos_ ? rot_half : 0, rot_rows};
    const int hw = 512 / P;
    const long per = (H + 2 * G + hw - 1) / hw + (act_n + 511) / 512;
    const unsigned grid = (unsigned)((N * per + 3) / 4);
#define GO(T, PP) k_qknorm_kv<T, PP><<<grid, 256, 0, st_>>>((T*)qkv, \
        (T*)q_out, (T*)kc, (T*)vc, (const int*)table, per_slot, \
        (const int*)pos, (const int*)slot, N, H, G, ld_, dim, eps, coef, \
        every, rot, act_0, act_n)
    if (P == 64) { if (f32) GO(float, 64); else GO(bf16_t, 64); }
    else if (P == 128) { if (f32) GO(float, 128); else GO(bf16_t, 128); }
    else if (P == 256) { if (f32) GO(float, 256); else GO(bf16_t, 256); }
    else return -101;
#undef GO
    LAUNCH_CHECK();
    return 0;
}

// Keys seen: the last `window` (0: all) and the first `keep`. Epilogue: see
// HeadEpilogue
int gh_paged_decode(void* stream, void* out, const void* q, const void* kc,
                    const void* vc, const void* table, int per_slot,
                    const void* pos, const void* slot, void* ws, int B,
                    int Hq, int Hk, int D, int nsplit, float scale,
                    int window, int keep, const void* sink, const void* gate,
                    int gate_ld, int gate_el, float oscale, int out_ld) {
    if (B < 1 || Hq % Hk || nsplit < 1 || window < 0 || keep < 0) return -100;
    const HeadEpilogue epi{(const float*)sink, (const bf16_t*)gate, gate_ld,
                           gate && gate_el, oscale, out_ld};
    const WindowKeys keys{window ? window : 1 << 30, keep};
    hipStream_t st_ = (hipStream_t)stream;
#define GO(DD) return paged_decode<DD>(st_, out, q, kc, vc, \
        (const int*)table, per_slot, (const int*)pos, (const int*)slot, \
        (float*)ws, B, Hq, Hk, nsplit, scale, epi, keys)
    if (D == 64) GO(64);
    if (D == 128) GO(128);
    if (D == 256) GO(256);
#undef GO
    return -101;
}

int gh_paged_prefill(void* stream, void* out, const void* q, const void* kc,
                     const void* vc, const void* table, int per_slot,
                     const void* meta, int ntiles, int Hq, int Hk, int D,
                     float scale, int window, int keep, const void* sink,
                     const void* gate, int gate_ld, int gate_el, float oscale,
                     int out_ld) {
    if (ntiles < 1 || Hq % Hk || window < 0 || keep < 0 ||
        (gate && gate_el && gate_ld % 4) || out_ld % 4)
        return -100;
    const HeadEpilogue epi{(const float*)sink, (const bf16_t*)gate, gate_ld,
                           gate && gate_el, oscale, out_ld};
    hipStream_t st_ = (hipStream_t)stream;
#define GO(DD, K, ...) k_paged_prefill<DD, K><<<dim3(ntiles, Hq), 256, 0, \
        st_>>>((bf16_t*)out, (const bf16_t*)q, \
        PagedKV<DD>{(const bf16_t*)kc, (const bf16_t*)vc, (const int*)table, \
                    Hk, per_slot}, (const int*)meta, Hq, Hq / Hk, scale, epi, \
        K{__VA_ARGS__})
#define PICK(DD) do { if (window) GO(DD, WindowKeys, window, keep); \
        else GO(DD, AllKeys); } while (0)
    if (D == 64) PICK(64);
    else if (D == 128) PICK(128);
    else if (D == 256) PICK(256);
    else return -101;
#undef PICK
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_attn_rows_f32(void* stream, void* out, const void* q, const void* kc,
                     const void* vc, const void* table, int per_slot,
                     const void* pos, const void* slot, int N, int H, int G,
                     int P, float scale, int window, int keep,
                     const void* sink, const void* gate, int gate_ld,
                     int gate_el, float oscale, int out_ld) {
    if (N < 1 || H % G || window < 0 || keep < 0) return -100;
    hipStream_t st_ = (hipStream_t)stream;
    const WindowKeys keys{window ? window : 1 << 30, keep};
#define GO(PP) k_attn_rows_f32<PP><<<(unsigned)((long)N * H), 256, 0, st_>>>( \
        (float*)out, (const float*)q, (const float*)kc, (const float*)vc, \
        (const int*)table, per_slot, (const int*)pos, (const int*)slot, H, G, \
        scale, (const float*)sink, (const float*)gate, gate_ld, gate_el, \
        oscale, out_ld ? out_ld : H * P, keys)
    if (P == 64) GO(64);
    else if (P == 128) GO(128);
    else if (P == 256) GO(256);
    else return -101;
#undef GO
    LAUNCH_CHECK();
    return 0;
}

// kind: Rec
int gh_rec_step(void* stream, int f32, int kind, void* o, void* S, const void* mst,
                const void* qkv, const void* gr, const void* segs,
                const void* pos, const void* slot, int nseg, int H, int DK,
                int DV, int ld_, float qscale, float cap, int rpb) {
    if (nseg < 1 || DK % 64 || DV % 64 || DK > 1024 || rpb < 1 || kind < 0 ||
        kind > CONSTANT || (kind == MLSTM && !mst))
        return -100;
    hipStream_t st_ = (hipStream_t)stream;
    const dim3 grid((unsigned)nseg, (unsigned)H,
                    (unsigned)((DV + (kind == MLSTM) + rpb - 1) / rpb));
#define GO(T, L, J, C) k_rec_step<T, L, J, C><<<grid, 256, 0, st_>>>( \
        (float*)o, (float*)S, (const float*)mst, (const T*)qkv, \
        (const float*)gr, (const int4*)segs, (const int*)pos, \
        (const int*)slot, H, DK, DV, ld_, qscale, cap, rpb)
#define PICK(T, C) do { if (DK <= 64) GO(T, 16, 1, C); \
        else if (DK <= 128) GO(T, 32, 1, C); \
        else if (DK <= 256) GO(T, 64, 1, C); \
        else if (DK <= 512) GO(T, 64, 2, C); else GO(T, 64, 4, C); } while (0)
    if (kind == MLSTM) {
        if (f32) PICK(float, MLSTM); else PICK(bf16_t, MLSTM);
    } else if (kind == CHANNELS) {
        if (f32) PICK(float, CHANNELS); else PICK(bf16_t, CHANNELS);
    } else {
        if (f32) PICK(float, CONSTANT); else PICK(bf16_t, CONSTANT);
    }
#undef PICK
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_rec_out(void* stream, int f32, int silu, void* out, const void* o,
               void* mst, const void* qkv, const void* gr, const void* segs,
               const void* pos, const void* slot, const void* norm, int nseg,
               int plain0, int nplain, int H, int DK, int DV, int ld_,
               int dvtrue, float cap, float eps) {
    if (nseg + nplain < 1) return -100;
    hipStream_t st_ = (hipStream_t)stream;
    const unsigned grid = (unsigned)(((long)(nseg + nplain) * H + 3) / 4);
#define GO(T, G) k_rec_out<T, G><<<grid, 256, 0, st_>>>((T*)out, \
        (const float*)o, (float*)mst, (const T*)qkv, (const float*)gr, \
        (const int4*)segs, (const int*)pos, (const int*)slot, \
        (const float*)norm, nseg, plain0, nplain, H, DK, DV, ld_, dvtrue, \
        cap, eps)
    if (silu) { if (f32) GO(float, true); else GO(bf16_t, true); }
    else { if (f32) GO(float, false); else GO(bf16_t, false); }
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_rec_row_out(void* stream, int f32, void* out, const void* o,
                   const void* gate, const void* norm, int N, int H, int DV,
                   int ld_, int out_ld, int true_cols, float eps) {
    if (N < 1 || H < 1 || DV % 64 || ld_ % 4 || out_ld % 4 || true_cols < 1)
        return -100;
#define GO(T, NV) k_rec_row_out<T, NV><<<N, 256, 0, (hipStream_t)stream>>>( \
        (T*)out, (const float*)o, (const T*)gate, (const float*)norm, H, DV, \
        ld_, out_ld, true_cols, eps)
#define PICK(T) do { if (H * DV <= 4096) GO(T, 4); \
        else if (H * DV <= 8192) GO(T, 8); else GO(T, 0); } while (0)
    if (f32) PICK(float); else PICK(bf16_t);
#undef PICK
#undef GO
    LAUNCH_CHECK();
    return 0;
}

// constant: lightning attention (gr: log decay by head; mst unused)
int gh_mlstm_chunks(void* stream, int constant, void* o, void* S, void* mst,
                    void* dS, void* scal, const void* qkv, const void* gr,
                    const void* chunks, const void* segs, int nchunks,
                    int nseg, int H, int DK, int DV, int ld_, float qscale,
                    float cap) {
    if (nchunks < 1 || nseg < 1 || DK % 64 || DV % 64 || (!constant && !mst))
        return -100;
    hipStream_t st_ = (hipStream_t)stream;
    const long quads = (long)(DV + !constant) * DK / 4;
#define GO(C) do { \
    k_mlstm_chunk_state<C><<<dim3(nchunks, H, (DK / 64) * (DV / 64)), 256, 0, \
        st_>>>((float*)dS, (float*)scal, (const float*)mst, \
        (const bf16_t*)qkv, (const float*)gr, (const int4*)chunks, \
        (const int4*)segs, H, DK, DV, ld_, cap); \
    LAUNCH_CHECK(); \
    k_mlstm_chunk_scan<C><<<dim3(nseg, H, (unsigned)((quads + 255) / 256)), \
        256, 0, st_>>>((float*)dS, (float*)scal, (float*)S, (float*)mst, \
        (const int4*)segs, H, DK, DV); \
    LAUNCH_CHECK(); \
    k_mlstm_chunk_out<C><<<dim3(nchunks, H, (DV + 127) / 128), 256, 0, \
        st_>>>((float*)o, (const float*)dS, (const float*)scal, \
        (const bf16_t*)qkv, (const float*)gr, (const int4*)chunks, H, DK, DV, \
        ld_, qscale, cap); \
    LAUNCH_CHECK(); } while (0)
    if (constant) GO(true); else GO(false);
#undef GO
    return 0;
}

int gh_gla_decay(void* stream, void* b, const void* u, const void* w,
                 const void* bias, const void* chunks, int nd, int nchunks,
                 int R, int C, float inv_tau) {
    if (nd + nchunks < 1 || R < 1 || C < 1) return -100;
#define GO(U) k_gla_decay<U><<<dim3((nd + U - 1) / U + nchunks, \
        (C + 255) / 256), 256, 0, (hipStream_t)stream>>>((float*)b, \
        (const float*)u, (const float*)w, (const float*)bias, \
        (const int4*)chunks, nd, R, C, inv_tau)
    if (nchunks) GO(16); else GO(4);
#undef GO
    LAUNCH_CHECK();
    return 0;
}

int gh_gla_chunks(void* stream, void* o, void* S, void* dS, const void* qkv,
                  const void* b, const void* chunks, const void* segs,
                  int nchunks, int nseg, int H, int DK, int DV, int ld_,
                  float qscale) {
    if (nchunks < 1 || nseg < 1 || DK % 64 || DV % 64) return -100;
    hipStream_t st_ = (hipStream_t)stream;
    // few chunks: value columns in blocks of their own, though each then takes
    // the decays or scores again
    const bool many = nchunks * H >= 512;
    k_gla_chunk_state<<<dim3(nchunks, H, DK / 64 * (many ? 1 : DV / 64)), 256,
                        0, st_>>>((float*)dS, (const bf16_t*)qkv,
        (const float*)b, (const int4*)chunks, H, DK, DV, ld_);
    LAUNCH_CHECK();
    const long quads = (long)DV * DK / 4;
    k_gla_chunk_scan<<<dim3(nseg, H, (unsigned)((quads + 255) / 256)), 256, 0,
                       st_>>>((float*)dS, (float*)S, (const float*)b,
        (const int4*)chunks, (const int4*)segs, H, DK, DV);
    LAUNCH_CHECK();
    k_gla_chunk_out<<<dim3(nchunks, H, many ? 1 : (DV + 127) / 128), 256, 0,
                      st_>>>((float*)o,
        (const float*)dS, (const bf16_t*)qkv, (const float*)b,
        (const int4*)chunks, H, DK, DV, ld_, qscale);
    LAUNCH_CHECK();
    return 0;
}

// E router outputs (rows of stride ldz), of which the first `experts` have
// weights. corr (nullable): correction of the choice; ident (nullable): sum of
// a token's weights beyond the experts
int gh_moe_route(void* stream, void* idx, void* wt, void* rank, void* counts,
                 void* sorted, void* tiles, const void* z, int ldz,
                 const void* corr, void* ident, int N, int E, int experts,
                 int top, int groups, int keep, float eps, float scale, int sigmoid, int bm,
                 int max_tiles) {
    if (ldz < E || (sigmoid && (corr || ident))) return -100;
    if (N < 1 || E < 1 || E > 1024 || top < 1 || experts < 1 || experts > E ||
        groups < 1 || E % groups || keep < 1 || keep > groups ||
        top > E / groups * keep)
        return -100;
    hipStream_t st_ = (hipStream_t)stream;
#define GO(V) k_moe_route<V><<<(N + 4 * tpw - 1) / (4 * tpw), 256, 0, st_>>>((int*)idx, \
        (float*)wt, (int*)rank, (int*)counts, (const float*)z, \
        ldz, (const float*)corr, (float*)ident, N, E, experts, top, groups, \
        keep, eps, scale, sigmoid, tpw)
    const int tpw = min(max(N / 2048, 1), 16);
    if (E <= 64) GO(1);
    else if (E <= 128) GO(2);
    else if (E <= 256) GO(4);
    else GO(16);
#undef GO
    LAUNCH_CHECK();
    const long pairs = (long)N * top;
    k_moe_scatter<<<(unsigned)((pairs + 255) / 256), 256, 0, st_>>>(
        (int*)sorted, (int4*)tiles, (const int*)idx, (const int*)rank,
        (const int*)counts, (int)pairs, experts, bm, max_tiles);
    LAUNCH_CHECK();
    return 0;
}

// act: 0 down, 1 up with squared ReLU, 2 gate and up (N weight rows, in turns
// of 16 | 16) with the gated unit's constants; pw (nullable): weights of the
// pairs on its input. bm: rows per tile of the list: 16 (few pairs; the exact mode) or
// 128
int gh_moe_gemm(void* stream, int f32, int act, void* out, const void* x,
                const void* w, const void* tiles, const void* sorted,
                int top, int N, int K, int bm, int max_tiles, float alpha,
                float limit, float shift, float cubic, const void* pw) {
    if (N % (act == 2 ? 128 : 64) || K % 64 || max_tiles < 1 || act < 0 ||
        act > 2)
        return -100;
    const GluParams glu{alpha, limit, shift, cubic};
    hipStream_t st_ = (hipStream_t)stream;
    if (f32) {
        if (bm != 16) return -103;
        const int ntn = N / 64;
        const unsigned grid = (unsigned)((max_tiles * ntn + 7) / 8 * 8);
#define GO(U) k_moe_gemm_f32<U><<<grid, 256, 0, st_>>>((float*)out, \
        (const float*)x, (const float*)w, (const int4*)tiles, \
        (const int*)sorted, top, N, K, ntn, max_tiles, glu, (const float*)pw)
        if (act == 2) GO(2); else if (act) GO(1); else GO(0);
#undef GO
        LAUNCH_CHECK();
        return 0;
    }
#define ARGS (bf16_t*)out, (const bf16_t*)x, (const bf16_t*)w, \
        (const int4*)tiles, (const int*)sorted, top, N, K, ntn, max_tiles, \
        glu, (const float*)pw
    if (bm == 128) {
        const int ntn = (N + 127) / 128;
        const unsigned grid = (unsigned)((max_tiles * ntn + 7) / 8 * 8);
        if (act == 2) k_moe_gemm<2, 2><<<grid, 256, 0, st_>>>(ARGS);
        else if (act) k_moe_gemm<1, 2><<<grid, 256, 0, st_>>>(ARGS);
        else k_moe_gemm<0, 2><<<grid, 256, 0, st_>>>(ARGS);
    } else if (bm == 16) {
        const int ntn = N / (act == 2 ? 32 : 16);
        const unsigned grid = (unsigned)((max_tiles * ntn + 7) / 8 * 8);
        if (act == 2) k_moe_gemm_few<2><<<grid, 256, 0, st_>>>(ARGS);
        else if (act) k_moe_gemm_few<1><<<grid, 256, 0, st_>>>(ARGS);
        else k_moe_gemm_few<0><<<grid, 256, 0, st_>>>(ARGS);
    } else {
        return -103;
    }
#undef ARGS
    LAUNCH_CHECK();
    return 0;
}

}  // extern "C"
