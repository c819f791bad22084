// layered_blocks.hip — further building blocks of layer-list models (kernels/layered.h): RMS norm in groups with a weight (alone, added to the
// residual stream, and followed by the next sublayer's norm), the cached row of latent attention (normed latent + rotated shared key part), products
// with one small matrix per head (absorbing the key expansion into the query, expanding values), the polynomial-norm activation, a mixture of
// experts (sigmoid router, top-k, rows grouped by expert, one grouped product per projection), the per-layer token input and the weighted
// average over the depth of the stack.  wave64, gfx950.  Norms, routers, angles and the residual sum are f32 in both operand types.
#include <hip/hip_runtime.h>
#include <math.h>
#include <algorithm>
#include "../common.h"
#include "layered.h"

namespace nvr { namespace kl {

namespace {

typedef uint16_t bf16_t;
__device__ __forceinline__ float ld_f(const float *p, int64_t i) { return p[i]; }
__device__ __forceinline__ float ld_f(const bf16_t *p, int64_t i) { return __uint_as_float((uint32_t)p[i] << 16); }
__device__ __forceinline__ void st_f(float *p, int64_t i, float v) { p[i] = v; }
__device__ __forceinline__ void st_f(bf16_t *p, int64_t i, float v) {       // round to nearest even
    uint32_t u = __float_as_uint(v);
    if ((u & 0x7fffffffu) > 0x7f800000u) { p[i] = (bf16_t)((u >> 16) | 0x40); return; }
    u += 0x7fffu + ((u >> 16) & 1u);
    p[i] = (bf16_t)(u >> 16);
}
__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}
__device__ __forceinline__ float block_sum256(float v, float *red) {       // red: 4 floats of LDS
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}
__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float gelu_tanh_f(float z) { return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))); }

__device__ __forceinline__ float gelu_erf_f(float z) { return 0.5f * z * (1.0f + erff(z * 0.70710678118654752f)); }

int launched(const char *what) {
    hipError_t e = hipGetLastError();
    if (e != hipSuccess) return nvr::fail(NVR_ERR_HIP, "%s launch failed: %s", what, hipGetErrorString(e));
    return 0;
}

// ------------------------------------------------------------------------------------------------ RMS norm in groups
// One workgroup per row, a wave per group (groups beyond four in turns).  IT: type of the input rows.  ADD: the normed row is added to the f32 row xres (the
// sublayer's output joining the residual stream) instead of being stored; with w2 the new residual row is normed once more into out (the next sublayer's input).
template <class IT, class OT, bool ADD>
__global__ __launch_bounds__(256) void group_norm_kernel(const IT *__restrict__ in, int64_t ldi, const int32_t *__restrict__ rows, int W, int groups, float eps,
                                                         const float *__restrict__ w, float *__restrict__ xres, const float *__restrict__ w2, int plain,
                                                         OT *__restrict__ out, int64_t ldo) {
    const int64_t r = blockIdx.x, src = rows ? rows[r] : r;
    const IT *x = in + src * ldi;
    const int n = W / groups, lane = threadIdx.x & 63;
    for (int g = threadIdx.x >> 6; g < groups; g += 4) {
        const int c0 = g * n;
        float ss = 0.f;
        for (int c = lane; c < n; c += 64) { const float v = ld_f(x, c0 + c); ss += v * v; }
        const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)n + eps);
        if (!ADD) {
            for (int c = lane; c < n; c += 64) st_f(out, r * ldo + c0 + c, ld_f(x, c0 + c) * inv * w[c0 + c]);
        } else {
            float *xr = xres + r * (int64_t)W;
            float s2 = 0.f;
            for (int c = lane; c < n; c += 64) {
                const float v = xr[c0 + c] + ld_f(x, c0 + c) * inv * w[c0 + c];
                xr[c0 + c] = v; s2 += v * v;
                if (plain) st_f(out, r * ldo + c0 + c, v);
            }
            if (w2) {
                const float inv2 = 1.0f / sqrtf(wave_sum(s2) / (float)n + eps);
                for (int c = lane; c < n; c += 64) st_f(out, r * ldo + c0 + c, xr[c0 + c] * inv2 * w2[c0 + c]);   // (a lane re-reads what it wrote)
            }
        }
    }
}

// ------------------------------------------------------------------------------------------------ the cached row of latent attention
// Row t of proj holds, from column col, `rank` latent numbers and `rot` numbers of the shared key part.  The page row of the token's position receives the latent
// divided by its root mean square times w, and the key part with coordinate pairs (2i, 2i+1), or halves (i, i + rot / 2), turned by position * freq[i].
template <class CT>
__global__ __launch_bounds__(64) void latent_store_kernel(const CT *__restrict__ proj, int64_t ld, int64_t col, Batch b, int rank, int rot, float eps,
                                                          const float *__restrict__ w, const float *__restrict__ freq, CT *__restrict__ pages, CT *__restrict__ rows, int halves, float gain) {
    const int t = blockIdx.x, sq = b.row_seq[t], lane = threadIdx.x;
    const int p = b.start[sq] + (t - b.cu[sq]);
    const int blk = b.block_tables[(int64_t)sq * b.max_blocks + p / b.block_size];
    CT *dst = pages + ((int64_t)blk * b.block_size + p % b.block_size) * (rank + rot);
    const CT *src = proj + (int64_t)t * ld + col;
    float ss = 0.f;
    for (int c = lane; c < rank; c += 64) { const float v = ld_f(src, c); ss += v * v; }
    const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)rank + eps);
    CT *dst2 = rows ? rows + (int64_t)t * (rank + rot) : nullptr;      // the same row once more, in step order
    for (int c = lane; c < rank; c += 64) { const float v = ld_f(src, c) * inv * w[c]; st_f(dst, c, v); if (dst2) st_f(dst2, c, v); }
    for (int i = lane; i < rot / 2; i += 64) {
        const float ang = (float)p * freq[i], cs = gain * cosf(ang), sn = gain * sinf(ang);
        const int cu = rank + (halves ? i : 2 * i), cv = rank + (halves ? i + rot / 2 : 2 * i + 1);
        const float u = ld_f(src, cu), v = ld_f(src, cv);
        st_f(dst, cu, u * cs - v * sn); st_f(dst, cv, v * cs + u * sn);
        if (dst2) { st_f(dst2, cu, u * cs - v * sn); st_f(dst2, cv, v * cs + u * sn); }
    }
}

// q rows [H][D + rot]: the last rot numbers of every head, rotated like the key part, go to out rows [H][ldh] at column ocol
template <class CT>
__global__ __launch_bounds__(256) void rotate_heads_kernel(const CT *__restrict__ q, int64_t ldq, int qstride, int qcol, Batch b, int H, int rot, const float *__restrict__ freq,
                                                           CT *__restrict__ out, int64_t ldo, int ostride, int ocol, int halves, float gain) {
    const int t = blockIdx.x, sq = b.row_seq[t];
    const int p = b.start[sq] + (t - b.cu[sq]);
    const int half = rot / 2;
    for (int idx = threadIdx.x; idx < H * half; idx += 256) {
        const int h = idx / half, i = idx - h * half;
        const float ang = (float)p * freq[i], cs = gain * cosf(ang), sn = gain * sinf(ang);
        const int cu = halves ? i : 2 * i, cv = halves ? i + half : 2 * i + 1;
        const CT *src = q + (int64_t)t * ldq + (int64_t)h * qstride + qcol;
        const float u = ld_f(src, cu), v = ld_f(src, cv);
        CT *dst = out + (int64_t)t * ldo + (int64_t)h * ostride + ocol;
        st_f(dst, cu, u * cs - v * sn); st_f(dst, cv, v * cs + u * sn);
    }
}

// Both at once for 16-bit rows whose parts are multiples of 8 numbers (halves: a rotated part of a multiple of 16): 16-byte loads and stores, cosines and sines once per row.  RB rows
// per workgroup: 4, a wave each; or 1, its queries by all four waves.
template <int RB>
__global__ __launch_bounds__(256) void latent_rope8_kernel(LatentRopeArgs a, Batch b) {
    extern __shared__ float2 tab[];                     // [RB][half] (cosine, sine)
    const int half = a.rot >> 1, r0 = blockIdx.x * RB;
    for (int idx = threadIdx.x; idx < RB * half; idx += 256) {
        const int rr = RB == 1 ? 0 : idx / half, i = idx - rr * half, t = r0 + rr;
        if (t < b.T) { const int sq = b.row_seq[t]; const float ang = (float)(b.start[sq] + (t - b.cu[sq])) * a.freq[i]; tab[idx] = float2{a.gain * cosf(ang), a.gain * sinf(ang)}; }
    }
    __syncthreads();
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, rr = RB == 1 ? 0 : wave, t = r0 + rr;
    if (t >= b.T) return;
    const float2 *ct = tab + rr * half;
    const int nch = a.halves ? half >> 3 : a.rot >> 3;  // pieces of a rotated part: 8 numbers of each half, or 4 pairs
    auto turn = [&](const bf16_t *src, bf16_t *d1, bf16_t *d2, int i) {       // piece i of the part at src -> the same place behind d1 and d2 (d2 may be null)
        if (a.halves) {
            const uint4 x = *reinterpret_cast<const uint4 *>(src + i * 8), y = *reinterpret_cast<const uint4 *>(src + half + i * 8);
            const bf16_t *xe = reinterpret_cast<const bf16_t *>(&x), *ye = reinterpret_cast<const bf16_t *>(&y);
            uint4 o1, o2; bf16_t *e1 = reinterpret_cast<bf16_t *>(&o1), *e2 = reinterpret_cast<bf16_t *>(&o2);
#pragma unroll
            for (int k = 0; k < 8; ++k) {
                const float2 c = ct[i * 8 + k]; const float u = ld_f(xe, k), v = ld_f(ye, k);
                st_f(e1, k, u * c.x - v * c.y); st_f(e2, k, v * c.x + u * c.y);
            }
            *reinterpret_cast<uint4 *>(d1 + i * 8) = o1; *reinterpret_cast<uint4 *>(d1 + half + i * 8) = o2;
            if (d2) { *reinterpret_cast<uint4 *>(d2 + i * 8) = o1; *reinterpret_cast<uint4 *>(d2 + half + i * 8) = o2; }
        } else {
            const uint4 x = *reinterpret_cast<const uint4 *>(src + i * 8); const bf16_t *xe = reinterpret_cast<const bf16_t *>(&x);
            uint4 o; bf16_t *e = reinterpret_cast<bf16_t *>(&o);
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                const float2 c = ct[i * 4 + k]; const float u = ld_f(xe, 2 * k), v = ld_f(xe, 2 * k + 1);
                st_f(e, 2 * k, u * c.x - v * c.y); st_f(e, 2 * k + 1, v * c.x + u * c.y);
            }
            *reinterpret_cast<uint4 *>(d1 + i * 8) = o;
            if (d2) *reinterpret_cast<uint4 *>(d2 + i * 8) = o;
        }
    };
    if (a.pages && (RB > 1 || wave == 0)) {
        const int sq = b.row_seq[t], p = b.start[sq] + (t - b.cu[sq]), blk = b.block_tables[(int64_t)sq * b.max_blocks + p / b.block_size];
        bf16_t *d1 = (bf16_t *)a.pages + ((int64_t)blk * b.block_size + p % b.block_size) * (a.rank + a.rot), *d2 = a.rows ? (bf16_t *)a.rows + (int64_t)t * (a.rank + a.rot) : nullptr;
        const bf16_t *src = (const bf16_t *)a.proj + (int64_t)t * a.ld + a.col;
        float ss = 0.f;
        for (int c = lane * 8; c < a.rank; c += 512) {
            const uint4 x = *reinterpret_cast<const uint4 *>(src + c); const bf16_t *xe = reinterpret_cast<const bf16_t *>(&x);
#pragma unroll
            for (int k = 0; k < 8; ++k) { const float v = ld_f(xe, k); ss += v * v; }
        }
        const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)a.rank + a.eps);
        for (int c = lane * 8; c < a.rank; c += 512) {
            const uint4 x = *reinterpret_cast<const uint4 *>(src + c); const bf16_t *xe = reinterpret_cast<const bf16_t *>(&x);
            uint4 o; bf16_t *e = reinterpret_cast<bf16_t *>(&o);
#pragma unroll
            for (int k = 0; k < 8; ++k) st_f(e, k, ld_f(xe, k) * inv * a.w[c + k]);
            *reinterpret_cast<uint4 *>(d1 + c) = o;
            if (d2) *reinterpret_cast<uint4 *>(d2 + c) = o;
        }
        for (int i = lane; i < nch; i += 64) turn(src + a.rank, d1 + a.rank, d2 ? d2 + a.rank : nullptr, i);
    }
    if (a.q)
        for (int idx = RB == 1 ? threadIdx.x : lane; idx < a.H * nch; idx += RB == 1 ? 256 : 64) {
            const int h = idx / nch, i = idx - h * nch;
            turn((const bf16_t *)a.q + (int64_t)t * a.ldq + h * a.qstride + a.qcol, (bf16_t *)a.out + (int64_t)t * a.ldo + h * a.ostride + a.ocol, nullptr, i);
        }
}

// ------------------------------------------------------------------------------------------------ one small matrix per head / per group of rows
// A 64 x 64 tile of y = a . w^T per workgroup, K in steps of 16 through LDS, 4 x 4 outputs per thread, f32 accumulation.
struct TileJob {
    const void *a; int64_t lda; const void *w; int64_t ldw; void *y; int64_t ldy;
    int rows, K, N;                               // this job's extent
    const void *gate; int64_t ldg;                // y *= sigmoid(gate) (same row / column as y) when not null
    const int32_t *src; const float *rscale; int src_div;   // row r of a is row src[r] / src_div of the array, times rscale[src[r]], when src is not null
};
template <class ET>
__device__ __forceinline__ void tile_product(const TileJob &j, int row0, int col0, float (*As)[68], float (*Ws)[68]) {
    const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4;
    const ET *a = (const ET *)j.a; const ET *w = (const ET *)j.w;
    float acc[4][4] = {};
    for (int k0 = 0; k0 < j.K; k0 += 16) {
        for (int idx = threadIdx.x; idx < 64 * 16; idx += 256) {
            const int r = idx >> 4, k = idx & 15;
            float av = 0.f, wv = 0.f;
            if (row0 + r < j.rows && k0 + k < j.K) {
                if (j.src) { const int sidx = j.src[row0 + r]; av = ld_f(a, (int64_t)(sidx / j.src_div) * j.lda + k0 + k) * j.rscale[sidx]; }
                else av = ld_f(a, (int64_t)(row0 + r) * j.lda + k0 + k);
            }
            if (col0 + r < j.N && k0 + k < j.K) wv = ld_f(w, (int64_t)(col0 + r) * j.ldw + k0 + k);
            if (sizeof(ET) == 2 && j.src) { bf16_t h; st_f(&h, 0, av); av = ld_f(&h, 0); }     // (the scaled row is an operand: one rounding, as a stored copy would have)
            As[k][r] = av; Ws[k][r] = wv;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < 16; ++k) {
            float av[4], wv[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) { av[i] = As[k][ty * 4 + i]; wv[i] = Ws[k][tx * 4 + i]; }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int c = 0; c < 4; ++c) acc[i][c] = fmaf(av[i], wv[c], acc[i][c]);
        }
        __syncthreads();
    }
    ET *y = (ET *)j.y;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int c = 0; c < 4; ++c) {
            const int r = row0 + ty * 4 + i, n = col0 + tx * 4 + c;
            if (r < j.rows && n < j.N) {
                float v = acc[i][c];
                if (j.gate) v *= sigmoid_f(ld_f((const ET *)j.gate, (int64_t)r * j.ldg + n));
                st_f(y, (int64_t)r * j.ldy + n, v);
            }
        }
}

// The same on the matrix cores for bfloat16 operands (K a multiple of 8, rows 16-byte aligned): v_mfma_f32_16x16x32_bf16, fragments straight from global
// memory (a lane's 8 consecutive k of its row / column are one 16-byte load; nothing staged in LDS, no barrier).  WR = 4: the four waves take 16 rows each of
// a 64 x 64 tile; WR = 1: they take 64 columns each of a 16 x 256 tile (few rows: decode-sized steps, experts with few tokens).
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
template <int WR>
__device__ __forceinline__ void tile_product_mfma(const TileJob &j, int row0, int col0) {
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lm = lane & 15, lq = lane >> 4;
    const int rbase = row0 + (WR == 4 ? wave * 16 : 0), cbase = col0 + (WR == 4 ? 0 : wave * 64);
    if (rbase >= j.rows || cbase >= j.N) return;
    const bf16_t *w = (const bf16_t *)j.w;
    const int r = rbase + lm;
    const bool rok = r < j.rows;
    const bf16_t *ap = (const bf16_t *)j.a; float rs = 1.f;
    if (rok) {
        if (j.src) { const int sidx = j.src[r]; ap += (int64_t)(sidx / j.src_div) * j.lda; rs = j.rscale[sidx]; }
        else ap += (int64_t)r * j.lda;
    }
    const bf16_t *wp[4]; bool cok[4];
#pragma unroll
    for (int cb = 0; cb < 4; ++cb) { const int n = cbase + cb * 16 + lm; cok[cb] = n < j.N; wp[cb] = w + (int64_t)(cok[cb] ? n : 0) * j.ldw; }
    f32x4 acc[4];
#pragma unroll
    for (int cb = 0; cb < 4; ++cb) acc[cb] = f32x4{0.f, 0.f, 0.f, 0.f};
    const uint4 zero{0, 0, 0, 0};
#pragma unroll 2
    for (int k0 = 0; k0 < j.K; k0 += 32) {
        const int k = k0 + lq * 8;
        const bool kok = k < j.K;
        uint4 av = (rok && kok) ? *reinterpret_cast<const uint4 *>(ap + k) : zero;
        uint4 wv[4];
#pragma unroll
        for (int cb = 0; cb < 4; ++cb) wv[cb] = (cok[cb] && kok) ? *reinterpret_cast<const uint4 *>(wp[cb] + k) : zero;
        if (j.src) {                                        // the scaled row is an operand: one rounding, as a stored copy would have
            bf16_t *e = reinterpret_cast<bf16_t *>(&av);
#pragma unroll
            for (int y = 0; y < 8; ++y) st_f(e, y, ld_f(e, y) * rs);
        }
        const bf16x8 af = __builtin_bit_cast(bf16x8, av);
#pragma unroll
        for (int cb = 0; cb < 4; ++cb) acc[cb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af, __builtin_bit_cast(bf16x8, wv[cb]), acc[cb], 0, 0, 0);
    }
    bf16_t *y = (bf16_t *)j.y;
#pragma unroll
    for (int cb = 0; cb < 4; ++cb)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int rr = rbase + lq * 4 + i, n = cbase + cb * 16 + lm;
            if (rr < j.rows && n < j.N) {
                float v = acc[cb][i];
                if (j.gate) v *= sigmoid_f(ld_f((const bf16_t *)j.gate, (int64_t)rr * j.ldg + n));
                st_f(y, (int64_t)rr * j.ldy + n, v);
            }
        }
}

// Many rows: a 128 x 128 tile per workgroup, K in steps of 64 through LDS (the next step's 16-byte pieces are requested before the current step's
// arithmetic); the four waves own 64 x 64 quarters, 32 MFMAs per step.
__device__ __forceinline__ void tile_product_mfma128(const TileJob &j, int row0, int col0, bf16_t *As, bf16_t *Ws) {
    constexpr int KS = 64, LD = KS + 8;                     // rows stay 16-byte aligned and spread over the banks
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lm = lane & 15, lq = lane >> 4, wr = wave >> 1, wc = wave & 1;
    const int lrow = threadIdx.x >> 3, lch = threadIdx.x & 7;
    const bf16_t *ap[4], *wp[4]; bool aok[4], wok[4]; float rs[4] = {1.f, 1.f, 1.f, 1.f};
#pragma unroll
    for (int q = 0; q < 4; ++q) {
        const int r = row0 + lrow + 32 * q, n = col0 + lrow + 32 * q;
        aok[q] = r < j.rows; wok[q] = n < j.N;
        ap[q] = (const bf16_t *)j.a; wp[q] = (const bf16_t *)j.w + (int64_t)(wok[q] ? n : 0) * j.ldw;
        if (aok[q]) {
            if (j.src) { const int sidx = j.src[r]; ap[q] += (int64_t)(sidx / j.src_div) * j.lda; rs[q] = j.rscale[sidx]; }
            else ap[q] += (int64_t)r * j.lda;
        }
    }
    f32x4 acc[4][4];
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[i][c] = f32x4{0.f, 0.f, 0.f, 0.f};
    const uint4 zero{0, 0, 0, 0};
    uint4 ra[4], rw[4];
    auto fetch = [&](int k0) {
        const int k = k0 + lch * 8;
        const bool kok = k < j.K;
#pragma unroll
        for (int q = 0; q < 4; ++q) {
            ra[q] = (aok[q] && kok) ? *reinterpret_cast<const uint4 *>(ap[q] + k) : zero;
            rw[q] = (wok[q] && kok) ? *reinterpret_cast<const uint4 *>(wp[q] + k) : zero;
        }
    };
    fetch(0);
    for (int k0 = 0; k0 < j.K; k0 += KS) {
        if (j.src) {
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                bf16_t *e = reinterpret_cast<bf16_t *>(&ra[q]);
#pragma unroll
                for (int y = 0; y < 8; ++y) st_f(e, y, ld_f(e, y) * rs[q]);
            }
        }
        __syncthreads();
#pragma unroll
        for (int q = 0; q < 4; ++q) {
            *reinterpret_cast<uint4 *>(As + (lrow + 32 * q) * LD + lch * 8) = ra[q];
            *reinterpret_cast<uint4 *>(Ws + (lrow + 32 * q) * LD + lch * 8) = rw[q];
        }
        __syncthreads();
        if (k0 + KS < j.K) fetch(k0 + KS);
#pragma unroll
        for (int kk = 0; kk < KS; kk += 32) {
            bf16x8 af[4], wf[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                af[i] = *reinterpret_cast<const bf16x8 *>(As + (wr * 64 + i * 16 + lm) * LD + kk + lq * 8);
                wf[i] = *reinterpret_cast<const bf16x8 *>(Ws + (wc * 64 + i * 16 + lm) * LD + kk + lq * 8);
            }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int c = 0; c < 4; ++c) acc[i][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af[i], wf[c], acc[i][c], 0, 0, 0);
        }
    }
    bf16_t *y = (bf16_t *)j.y;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int c = 0; c < 4; ++c)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int rr = row0 + wr * 64 + i * 16 + lq * 4 + e, n = col0 + wc * 64 + c * 16 + lm;
                if (rr < j.rows && n < j.N) {
                    float v = acc[i][c][e];
                    if (j.gate) v *= sigmoid_f(ld_f((const bf16_t *)j.gate, (int64_t)rr * j.ldg + n));
                    st_f(y, (int64_t)rr * j.ldy + n, v);
                }
            }
}

__global__ __launch_bounds__(256) void head_linear_mfma128_kernel(HeadLinearArgs p) {
    __shared__ __attribute__((aligned(16))) bf16_t As[128 * 72], Ws[128 * 72];
    const int h = blockIdx.z;
    TileJob j{};
    j.a = (const bf16_t *)p.a + (int64_t)h * p.ha; j.lda = p.lda; j.w = (const bf16_t *)p.w + (int64_t)h * p.N * p.K; j.ldw = p.K;
    j.y = (bf16_t *)p.y + (int64_t)h * p.hy; j.ldy = p.ldy; j.rows = p.T; j.K = p.K; j.N = p.N;
    j.gate = p.gate ? (const void *)((const bf16_t *)p.gate + (int64_t)h * p.hg) : nullptr; j.ldg = p.ldg;
    tile_product_mfma128(j, blockIdx.y * 128, blockIdx.x * 128, As, Ws);
}

__global__ __launch_bounds__(256) void grouped_linear_mfma128_kernel(GroupedLinearArgs p) {
    __shared__ __attribute__((aligned(16))) bf16_t As[128 * 72], Ws[128 * 72];
    int tile = blockIdx.y, e = 0, lo = 0, hi = 0;
    for (; e < p.groups; ++e) {
        lo = p.off[e]; hi = p.off[e + 1];
        const int nt = (hi - lo + 127) >> 7;
        if (tile < nt) break;
        tile -= nt;
    }
    if (e == p.groups) return;                              // (every thread of the workgroup leaves: no barrier is left waiting)
    TileJob j{};
    j.lda = p.lda; j.w = (const bf16_t *)p.w + (int64_t)e * p.N * p.K; j.ldw = p.K; j.y = (bf16_t *)p.y + (int64_t)lo * p.ldy; j.ldy = p.ldy;
    j.rows = hi - lo; j.K = p.K; j.N = p.N;
    if (p.src) { j.a = p.a; j.src = p.src + lo; j.rscale = p.rscale; j.src_div = p.src_div; }
    else j.a = (const bf16_t *)p.a + (int64_t)lo * p.lda;
    tile_product_mfma128(j, tile * 128, blockIdx.x * 128, As, Ws);
}

// Few rows (decode-sized steps, experts with a handful of tokens): a 16 x 64 tile per workgroup and the four waves split K, so that a product whose cost is
// reading the matrix is spread over four times as many workgroups; the partial sums meet in LDS.
__device__ __forceinline__ void tile_product_mfma_ksplit(const TileJob &j, int row0, int col0, float *part) {      // part: [3][16 * 64] floats of LDS
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lm = lane & 15, lq = lane >> 4;
    const bf16_t *w = (const bf16_t *)j.w;
    const int r = row0 + lm;
    const bool rok = r < j.rows;
    const bf16_t *ap = (const bf16_t *)j.a; float rs = 1.f;
    if (rok) {
        if (j.src) { const int sidx = j.src[r]; ap += (int64_t)(sidx / j.src_div) * j.lda; rs = j.rscale[sidx]; }
        else ap += (int64_t)r * j.lda;
    }
    const bf16_t *wp[4]; bool cok[4];
#pragma unroll
    for (int cb = 0; cb < 4; ++cb) { const int n = col0 + cb * 16 + lm; cok[cb] = n < j.N; wp[cb] = w + (int64_t)(cok[cb] ? n : 0) * j.ldw; }
    f32x4 acc[4];
#pragma unroll
    for (int cb = 0; cb < 4; ++cb) acc[cb] = f32x4{0.f, 0.f, 0.f, 0.f};
    const uint4 zero{0, 0, 0, 0};
    const int kq = ((j.K + 3) / 4 + 31) / 32 * 32, kbeg = wave * kq, kend = min(j.K, kbeg + kq);
#pragma unroll 2
    for (int k0 = kbeg; k0 < kend; k0 += 32) {
        const int k = k0 + lq * 8;
        const bool kok = k < kend;
        uint4 av = (rok && kok) ? *reinterpret_cast<const uint4 *>(ap + k) : zero;
        uint4 wv[4];
#pragma unroll
        for (int cb = 0; cb < 4; ++cb) wv[cb] = (cok[cb] && kok) ? *reinterpret_cast<const uint4 *>(wp[cb] + k) : zero;
        if (j.src) {
            bf16_t *e = reinterpret_cast<bf16_t *>(&av);
#pragma unroll
            for (int y = 0; y < 8; ++y) st_f(e, y, ld_f(e, y) * rs);
        }
        const bf16x8 af = __builtin_bit_cast(bf16x8, av);
#pragma unroll
        for (int cb = 0; cb < 4; ++cb) acc[cb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af, __builtin_bit_cast(bf16x8, wv[cb]), acc[cb], 0, 0, 0);
    }
    if (wave > 0)
#pragma unroll
        for (int cb = 0; cb < 4; ++cb)
#pragma unroll
            for (int i = 0; i < 4; ++i) part[(wave - 1) * 1024 + (lq * 4 + i) * 64 + cb * 16 + lm] = acc[cb][i];
    __syncthreads();
    if (wave > 0) return;
    bf16_t *y = (bf16_t *)j.y;
#pragma unroll
    for (int cb = 0; cb < 4; ++cb)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int rr = row0 + lq * 4 + i, n = col0 + cb * 16 + lm, at = (lq * 4 + i) * 64 + cb * 16 + lm;
            if (rr < j.rows && n < j.N) {
                float v = (acc[cb][i] + part[at]) + (part[1024 + at] + part[2048 + at]);
                if (j.gate) v *= sigmoid_f(ld_f((const bf16_t *)j.gate, (int64_t)rr * j.ldg + n));
                st_f(y, (int64_t)rr * j.ldy + n, v);
            }
        }
}

__global__ __launch_bounds__(256) void head_linear_ksplit_kernel(HeadLinearArgs p) {
    __shared__ float part[3 * 1024];
    const int h = blockIdx.z;
    TileJob j{};
    j.a = (const bf16_t *)p.a + (int64_t)h * p.ha; j.lda = p.lda; j.w = (const bf16_t *)p.w + (int64_t)h * p.N * p.K; j.ldw = p.K;
    j.y = (bf16_t *)p.y + (int64_t)h * p.hy; j.ldy = p.ldy; j.rows = p.T; j.K = p.K; j.N = p.N;
    j.gate = p.gate ? (const void *)((const bf16_t *)p.gate + (int64_t)h * p.hg) : nullptr; j.ldg = p.ldg;
    tile_product_mfma_ksplit(j, blockIdx.y * 16, blockIdx.x * 64, part);
}

__global__ __launch_bounds__(256) void grouped_linear_ksplit_kernel(GroupedLinearArgs p) {
    __shared__ float part[3 * 1024];
    int tile = blockIdx.y, e = 0, lo = 0, hi = 0;
    for (; e < p.groups; ++e) {
        lo = p.off[e]; hi = p.off[e + 1];
        const int nt = (hi - lo + 15) >> 4;
        if (tile < nt) break;
        tile -= nt;
    }
    if (e == p.groups) return;                              // (the whole workgroup leaves)
    TileJob j{};
    j.lda = p.lda; j.w = (const bf16_t *)p.w + (int64_t)e * p.N * p.K; j.ldw = p.K; j.y = (bf16_t *)p.y + (int64_t)lo * p.ldy; j.ldy = p.ldy;
    j.rows = hi - lo; j.K = p.K; j.N = p.N;
    if (p.src) { j.a = p.a; j.src = p.src + lo; j.rscale = p.rscale; j.src_div = p.src_div; }
    else j.a = (const bf16_t *)p.a + (int64_t)lo * p.lda;
    tile_product_mfma_ksplit(j, tile * 16, blockIdx.x * 64, part);
}

template <int WR>
__global__ __launch_bounds__(256) void head_linear_mfma_kernel(HeadLinearArgs p) {
    const int h = blockIdx.z;
    TileJob j{};
    j.a = (const bf16_t *)p.a + (int64_t)h * p.ha; j.lda = p.lda; j.w = (const bf16_t *)p.w + (int64_t)h * p.N * p.K; j.ldw = p.K;
    j.y = (bf16_t *)p.y + (int64_t)h * p.hy; j.ldy = p.ldy; j.rows = p.T; j.K = p.K; j.N = p.N;
    j.gate = p.gate ? (const void *)((const bf16_t *)p.gate + (int64_t)h * p.hg) : nullptr; j.ldg = p.ldg;
    tile_product_mfma<WR>(j, blockIdx.y * (WR * 16), blockIdx.x * (WR == 4 ? 64 : 256));
}

template <int WR>
__global__ __launch_bounds__(256) void grouped_linear_mfma_kernel(GroupedLinearArgs p) {
    constexpr int TR = WR * 16;
    int tile = blockIdx.y, e = 0, lo = 0, hi = 0;
    for (; e < p.groups; ++e) {
        lo = p.off[e]; hi = p.off[e + 1];
        const int nt = (hi - lo + TR - 1) / TR;
        if (tile < nt) break;
        tile -= nt;
    }
    if (e == p.groups) return;
    TileJob j{};
    j.lda = p.lda; j.w = (const bf16_t *)p.w + (int64_t)e * p.N * p.K; j.ldw = p.K; j.y = (bf16_t *)p.y + (int64_t)lo * p.ldy; j.ldy = p.ldy;
    j.rows = hi - lo; j.K = p.K; j.N = p.N;
    if (p.src) { j.a = p.a; j.src = p.src + lo; j.rscale = p.rscale; j.src_div = p.src_div; }
    else j.a = (const bf16_t *)p.a + (int64_t)lo * p.lda;
    tile_product_mfma<WR>(j, tile * TR, blockIdx.x * (WR == 4 ? 64 : 256));
}

// y[t][h][n] = sum_k a[t][h][k] w[h][n][k]: blockIdx.z is the head
template <class ET>
__global__ __launch_bounds__(256) void head_linear_kernel(HeadLinearArgs p) {
    __shared__ float As[16][68], Ws[16][68];
    const int h = blockIdx.z;
    TileJob j{};
    j.a = (const ET *)p.a + (int64_t)h * p.ha; j.lda = p.lda; j.w = (const ET *)p.w + (int64_t)h * p.N * p.K; j.ldw = p.K;
    j.y = (ET *)p.y + (int64_t)h * p.hy; j.ldy = p.ldy; j.rows = p.T; j.K = p.K; j.N = p.N;
    j.gate = p.gate ? (const void *)((const ET *)p.gate + (int64_t)h * p.hg) : nullptr; j.ldg = p.ldg;
    tile_product<ET>(j, blockIdx.y * 64, blockIdx.x * 64, As, Ws);
}

// Rows grouped by expert: group e owns rows off[e] .. off[e+1]-1 and the matrix w[e] ([N][K]).  blockIdx.y walks the row tiles of all groups (at most
// rows / 64 + groups of them); a workgroup finds its group by walking the offsets, and leaves when it is beyond the last tile.
template <class ET>
__global__ __launch_bounds__(256) void grouped_linear_kernel(GroupedLinearArgs p) {
    __shared__ float As[16][68], Ws[16][68];
    int tile = blockIdx.y, e = 0, lo = 0, hi = 0;
    for (; e < p.groups; ++e) {
        lo = p.off[e]; hi = p.off[e + 1];
        const int nt = (hi - lo + 63) >> 6;
        if (tile < nt) break;
        tile -= nt;
    }
    if (e == p.groups) return;
    TileJob j{};
    j.lda = p.lda; j.w = (const ET *)p.w + (int64_t)e * p.N * p.K; j.ldw = p.K; j.y = (ET *)p.y + (int64_t)lo * p.ldy; j.ldy = p.ldy;
    j.rows = hi - lo; j.K = p.K; j.N = p.N;
    if (p.src) { j.a = p.a; j.src = p.src + lo; j.rscale = p.rscale; j.src_div = p.src_div; }
    else j.a = (const ET *)p.a + (int64_t)lo * p.lda;
    tile_product<ET>(j, tile * 64, blockIdx.x * 64, As, Ws);
}

// ------------------------------------------------------------------------------------------------ activations
// out = c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3 with N(v) = v / sqrt(mean(v^2) + eps) over the row
template <class OT>
__global__ __launch_bounds__(256) void poly_norm_kernel(const OT *__restrict__ z, int64_t ldz, int F, float eps, const float *__restrict__ coef, OT *__restrict__ out, int64_t ldo) {
    __shared__ float red[4];
    const int64_t t = blockIdx.x;
    float s1 = 0.f, s2 = 0.f, s3 = 0.f;
    for (int c = threadIdx.x; c < F; c += 256) { const float v = ld_f(z, t * ldz + c), v2 = v * v; s1 += v2; s2 += v2 * v2; s3 += v2 * v2 * v2; }
    s1 = block_sum256(s1, red); s2 = block_sum256(s2, red); s3 = block_sum256(s3, red);
    const float i1 = coef[0] / sqrtf(s1 / (float)F + eps), i2 = coef[1] / sqrtf(s2 / (float)F + eps), i3 = coef[2] / sqrtf(s3 / (float)F + eps), e = coef[3];
    for (int c = threadIdx.x; c < F; c += 256) { const float v = ld_f(z, t * ldz + c); st_f(out, t * ldo + c, v * i1 + v * v * i2 + v * v * v * i3 + e); }
}

// out = act(gate) * up; gu rows [2 F] (gate columns, then up columns); GELU: the tanh form, else silu
template <class OT, bool GELU>
__global__ __launch_bounds__(256) void gated_mul_kernel(const OT *__restrict__ gu, int64_t T, int64_t F, OT *__restrict__ out, int64_t ldo) {
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= T * F) return;
    const int64_t t = idx / F, c = idx - t * F;
    const float g = ld_f(gu, t * 2 * F + c);
    st_f(out, t * ldo + c, (GELU ? gelu_tanh_f(g) : g * sigmoid_f(g)) * ld_f(gu, t * 2 * F + F + c));
}

// 16-bit rows, 8 numbers per thread (F and the stride multiples of 8, 16-byte aligned rows)
template <bool GELU>
__global__ __launch_bounds__(256) void gated_mul8_kernel(const bf16_t *__restrict__ gu, int64_t T, int64_t F8, bf16_t *__restrict__ out, int64_t ldo) {
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= T * F8) return;
    const int64_t t = idx / F8, c = (idx - t * F8) * 8;
    uint4 gv = *reinterpret_cast<const uint4 *>(gu + t * 16 * F8 + c);
    const uint4 uv = *reinterpret_cast<const uint4 *>(gu + t * 16 * F8 + 8 * F8 + c);
    bf16_t *ge = reinterpret_cast<bf16_t *>(&gv); const bf16_t *ue = reinterpret_cast<const bf16_t *>(&uv);
#pragma unroll
    for (int k = 0; k < 8; ++k) { const float g = ld_f(ge, k); st_f(ge, k, (GELU ? gelu_tanh_f(g) : g * sigmoid_f(g)) * ld_f(ue, k)); }
    *reinterpret_cast<uint4 *>(out + t * ldo + c) = gv;
}

// ------------------------------------------------------------------------------------------------ mixture of experts
// Router: z = Wr h in f32; the `top` largest logits of a token (the lower index wins a tie) go to sel, their sigmoid to score ([T][top]).  The logits and not the
// scores are compared: the order is the same, and saturated scores do not tie.  softmax: the score of a chosen expert is its share e^(z - max) / sum over ALL experts,
// divided by the sum of the chosen shares (+ 1e-20).  Rows E .. E + extra - 1 of wr are further projections of h whose values leave as they are.
template <class OT>
__global__ __launch_bounds__(256) void moe_route_kernel(const OT *__restrict__ h, int64_t ldh, int W, const float *__restrict__ wr, int E, int top,
                                                        int32_t *__restrict__ sel, float *__restrict__ score, int softmax, int extra, float *__restrict__ extra_out,
                                                        const float *__restrict__ logits, int64_t ldl, const float *__restrict__ correction) {
    extern __shared__ float sc[];                       // [E + extra], with a correction also [E] choice scores
    const int64_t t = blockIdx.x; const int lane = threadIdx.x & 63;
    if (logits)                                         // the products were formed by a matrix product before this launch
        for (int e = threadIdx.x; e < E + extra; e += 256) { const float d = logits[t * ldl + e]; sc[e] = d; if (e >= E) extra_out[t * extra + (e - E)] = d; }
    else
    for (int e = threadIdx.x >> 6; e < E + extra; e += 4) {
        float d = 0.f;
        for (int c = lane; c < W; c += 64) d = fmaf(ld_f(h, t * ldh + c), wr[(int64_t)e * W + c], d);
        d = wave_sum(d);
        if (lane == 0) { sc[e] = d; if (e >= E) extra_out[t * extra + (e - E)] = d; }
    }
    __syncthreads();
    float zmax = 0.f, zsum = 1.f;
    if (softmax && threadIdx.x < 64) {                  // (the first wave keeps both for its choices below)
        zmax = -INFINITY;
        for (int e = lane; e < E; e += 64) zmax = fmaxf(zmax, sc[e]);
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) zmax = fmaxf(zmax, __shfl_xor(zmax, o, 64));
        zsum = 0.f;
        for (int e = lane; e < E; e += 64) zsum += expf(sc[e] - zmax);
        zsum = wave_sum(zsum);
    }
    float *ch = sc;                                     // what the choice compares: the logits, or share + correction
    if (correction) {
        ch = sc + E + extra;
        if (threadIdx.x < 64) for (int e = lane; e < E; e += 64) ch[e] = expf(sc[e] - zmax) / zsum + correction[e];       // (a lane reads its own entries back)
    }
    float chosen = 0.f;                                 // (lane 0: the sum of the chosen shares)
    for (int k = 0; k < top; ++k) {                     // the first wave: top times the arg-max over the experts' logits
        if (threadIdx.x < 64) {
            float best = -INFINITY; int bi = E;
            for (int e = lane; e < E; e += 64) if (ch[e] > best || (ch[e] == best && e < bi)) { best = ch[e]; bi = e; }
#pragma unroll
            for (int o = 32; o > 0; o >>= 1) {
                const float ob = __shfl_xor(best, o, 64); const int oi = __shfl_xor(bi, o, 64);
                if (ob > best || (ob == best && oi < bi)) { best = ob; bi = oi; }
            }
            if (bi >= E) bi = E - 1;                        // (logits that are not numbers compare false everywhere: the index still has to be an expert's)
            if (lane == 0) {
                const float z = correction ? sc[bi] : best;
                const float sv = softmax ? expf(z - zmax) / zsum : sigmoid_f(z);
                sel[t * top + k] = bi; score[t * top + k] = sv; chosen += sv; ch[bi] = -INFINITY;
            }
        }
        __syncthreads();
    }
    if (softmax && threadIdx.x == 0) for (int k = 0; k < top; ++k) score[t * top + k] /= chosen + 1e-20f;
}

// The same for logits formed beforehand and at most 64 experts: a wave per token, the experts across its lanes, nothing in LDS.  Lane k < top leaves with choice k and its score.
__device__ __forceinline__ void route_wave(int64_t t, int E, int top, int softmax, int extra, float *__restrict__ extra_out, const float *__restrict__ logits, int64_t ldl,
                                           const float *__restrict__ correction, int &my, float &mine) {
    const int lane = threadIdx.x & 63;
    const float *lr = logits + t * ldl;
    if (lane < extra) extra_out[t * extra + lane] = lr[E + lane];
    const float z = lane < E ? lr[lane] : -INFINITY;
    float sv = 0.f;
    if (softmax) {
        float zmax = z;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) zmax = fmaxf(zmax, __shfl_xor(zmax, o, 64));
        sv = lane < E ? expf(z - zmax) : 0.f;
        sv /= wave_sum(sv);
    } else if (lane < E) sv = sigmoid_f(z);
    const float ch = lane < E ? (correction ? sv + correction[lane] : z) : -INFINITY;      // what the choice compares
    bool open = lane < E;                               // not chosen yet
    float chosen = 0.f;
    my = -1; mine = 0.f;
    for (int k = 0; k < top; ++k) {
        float best = open ? ch : -INFINITY; int bi = open ? lane : 64;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) {
            const float ob = __shfl_xor(best, o, 64); const int oi = __shfl_xor(bi, o, 64);
            if (ob > best || (ob == best && oi < bi) || (bi == 64 && oi < 64)) { best = ob; bi = oi; }
        }
        bi = min(bi, E - 1);                            // (choices that are not numbers: the index still has to be an expert's)
        const float s = __shfl(sv, bi, 64);
        if (lane == k) { my = bi; mine = s; }
        chosen += s;
        if (lane == bi) open = false;
    }
    if (softmax) mine /= chosen + 1e-20f;
}
__global__ __launch_bounds__(256) void moe_route_wave_kernel(int T, int E, int top, int32_t *__restrict__ sel, float *__restrict__ score, int softmax, int extra,
                                                             float *__restrict__ extra_out, const float *__restrict__ logits, int64_t ldl, const float *__restrict__ correction) {
    const int64_t t = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6); const int lane = threadIdx.x & 63;
    if (t >= T) return;                                 // (a whole wave)
    int my; float mine;
    route_wave(t, E, top, softmax, extra, extra_out, logits, ldl, correction, my, mine);
    if (lane < top) { sel[t * top + lane] = my; score[t * top + lane] = mine; }
}

// Few tokens: both of the two steps above and below in one workgroup — the choices of up to 1024 (token, choice) pairs, then the experts' groups (rows not padded).
__global__ __launch_bounds__(1024) void moe_route_group_kernel(int T, int E, int El, int top, int32_t *__restrict__ sel, float *__restrict__ score, int softmax, int extra,
                                                               float *__restrict__ extra_out, const float *__restrict__ logits, int64_t ldl, const float *__restrict__ correction,
                                                               int32_t *__restrict__ off, int32_t *__restrict__ order, int32_t *__restrict__ place_of) {
    __shared__ int32_t chosen_e[1024], cnt[65];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    if (threadIdx.x < 65) cnt[threadIdx.x] = 0;
    __syncthreads();
    for (int t = wave; t < T; t += 16) {
        int my; float mine;
        route_wave(t, E, top, softmax, extra, extra_out, logits, ldl, correction, my, mine);
        if (lane < top) { sel[t * top + lane] = my; score[t * top + lane] = mine; chosen_e[t * top + lane] = my; if (my < El) atomicAdd(&cnt[my], 1); }
    }
    __syncthreads();
    if (wave == 0) {                                    // exclusive sum over the experts, one per lane
        const int c = lane < El ? cnt[lane] : 0;
        int run = c;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) { const int v = __shfl_up(run, o, 64); if (lane >= o) run += v; }
        if (lane < El) { cnt[lane] = run - c; off[lane] = run - c; }
        if (lane == El - 1) off[El] = run;
    }
    __syncthreads();
    const int i = threadIdx.x;
    if (i < T * top) {
        const int e = chosen_e[i];
        if (e >= El) place_of[i] = -1;
        else { const int place = atomicAdd(&cnt[e], 1); order[place] = i; place_of[i] = place; }
    }
}

// One workgroup: counts per expert, offsets, and a place for every (token, choice) among its expert's rows.  order[place] = token * top + choice;
// place_of[token * top + choice] = place (-1: a choice >= E has no group).  Which place inside its expert a row gets is left to the atomics: a row's result does not depend on it.
__global__ __launch_bounds__(1024) void moe_group_kernel(const int32_t *__restrict__ sel, int n, int E, int pad, int nblocks, int32_t *__restrict__ off,
                                                         int32_t *__restrict__ order, int32_t *__restrict__ place_of, int32_t *__restrict__ row_w) {
    extern __shared__ int32_t cnt[];                    // [E + 1] counts, then running offsets
    for (int e = threadIdx.x; e <= E; e += 1024) cnt[e] = 0;
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += 1024) if (sel[i] < E) atomicAdd(&cnt[sel[i]], 1);
    __syncthreads();
    if (threadIdx.x == 0) {                             // an expert's rows start at a multiple of pad; row_w names the expert of every block of pad rows
        int run = 0;
        for (int e = 0; e < E; ++e) {
            const int c = cnt[e], padded = (c + pad - 1) / pad * pad;
            cnt[e] = run; off[e] = run;
            if (row_w) for (int bk = run / pad; bk < (run + padded) / pad && bk < nblocks; ++bk) row_w[bk] = e;
            run += padded;
        }
        off[E] = run;
        if (row_w) for (int bk = run / pad; bk < nblocks; ++bk) row_w[bk] = 0;      // (blocks behind the last expert: any matrix, their rows are nobody's)
    }
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += 1024) {
        if (sel[i] >= E) { place_of[i] = -1; continue; }
        const int place = atomicAdd(&cnt[sel[i]], 1);
        place_of[i] = place;
        if (pad == 1) order[place] = i;                 // (padded places run past the choices; the padded form is read through place_of)
    }
}

// The same over many choices, in two launches of nb workgroups with a stretch of the choices each: counts[b][e] first; then every workgroup adds up the counts before its own, so that its
// places start where the stretches before it end (workgroup 0 also writes the offsets and the blocks' experts).
__global__ __launch_bounds__(256) void moe_count_kernel(const int32_t *__restrict__ sel, int n, int per, int E, int32_t *__restrict__ counts) {
    extern __shared__ int32_t cnt[];                    // [E]
    for (int e = threadIdx.x; e < E; e += 256) cnt[e] = 0;
    __syncthreads();
    const int i0 = blockIdx.x * per, i1 = min(n, i0 + per);
    for (int i = i0 + threadIdx.x; i < i1; i += 256) if (sel[i] < E) atomicAdd(&cnt[sel[i]], 1);
    __syncthreads();
    for (int e = threadIdx.x; e < E; e += 256) counts[blockIdx.x * E + e] = cnt[e];
}
__global__ __launch_bounds__(256) void moe_place_kernel(const int32_t *__restrict__ sel, int n, int per, int E, int pad, int nblocks, const int32_t *__restrict__ counts, int nb,
                                                        int32_t *__restrict__ off, int32_t *__restrict__ order, int32_t *__restrict__ place_of, int32_t *__restrict__ row_w) {
    extern __shared__ int32_t sh[];                     // [E] the next place of every expert, [E + 1] offsets
    int32_t *next = sh, *start = sh + E;
    for (int e = threadIdx.x; e < E; e += 256) {
        int before = 0, total = 0;
        for (int b = 0; b < nb; ++b) { const int c = counts[b * E + e]; if (b < (int)blockIdx.x) before += c; total += c; }
        next[e] = before; start[e] = total;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        int run = 0;
        for (int e = 0; e < E; ++e) { const int padded = (start[e] + pad - 1) / pad * pad; start[e] = run; next[e] += run; run += padded; }
        start[E] = run;
    }
    __syncthreads();
    if (blockIdx.x == 0) {
        for (int e = threadIdx.x; e <= E; e += 256) off[e] = start[e];
        for (int bk = threadIdx.x; bk < nblocks; bk += 256) {         // (behind the last expert: any matrix, their rows are nobody's)
            int w = 0;
            if (bk * pad < start[E]) for (int e = 1; e < E; ++e) if (start[e] <= bk * pad) w = e;
            row_w[bk] = w;
        }
    }
    const int i0 = blockIdx.x * per, i1 = min(n, i0 + per);
    for (int i = i0 + threadIdx.x; i < i1; i += 256) {
        if (sel[i] >= E) { place_of[i] = -1; continue; }
        const int place = atomicAdd(&next[sel[i]], 1);
        place_of[i] = place;
        if (pad == 1) order[place] = i;                 // (padded places run past the choices; the padded form is read through place_of)
    }
}

// xs[place_of[i]] = h[i / top] * score[i] (the expert's input, in the order of the grouped rows)
template <class OT>
__global__ __launch_bounds__(256) void moe_gather_kernel(const OT *__restrict__ h, int64_t ldh, int W, int top, const int32_t *__restrict__ place_of, const float *__restrict__ score,
                                                         OT *__restrict__ xs) {
    const int64_t i = blockIdx.x, t = i / top;
    if (place_of[i] < 0) return;                        // (an expert without a matrix)
    const float sc = score[i];
    OT *dst = xs + (int64_t)place_of[i] * W;
    for (int c = threadIdx.x; c < W; c += 256) st_f(dst, c, ld_f(h, t * ldh + c) * sc);
}

// 16-bit rows, 8 numbers per thread (W and the stride multiples of 8, 16-byte aligned rows)
__global__ __launch_bounds__(256) void moe_gather8_kernel(const bf16_t *__restrict__ h, int64_t ldh, int W8, int top, int64_t n, const int32_t *__restrict__ place_of,
                                                          const float *__restrict__ score, bf16_t *__restrict__ xs) {
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x, t = idx / W8;        // (token, piece): the piece is read once for all of the token's choices
    if (t >= n) return;
    const int64_t c = (idx - t * W8) * 8;
    const uint4 v = *reinterpret_cast<const uint4 *>(h + t * ldh + c); const bf16_t *ve = reinterpret_cast<const bf16_t *>(&v);
    for (int k = 0; k < top; ++k) {
        const int64_t place = place_of[t * top + k];
        if (place < 0) continue;
        const float sc = score[t * top + k];
        uint4 o; bf16_t *oe = reinterpret_cast<bf16_t *>(&o);
#pragma unroll
        for (int y = 0; y < 8; ++y) st_f(oe, y, ld_f(ve, y) * sc);
        *reinterpret_cast<uint4 *>(xs + place * W8 * 8 + c) = o;
    }
}

// out[t] = sum_k y[place_of[t * top + k]] (+ shared[t]) in the operand type
template <class OT>
__global__ __launch_bounds__(256) void moe_combine_kernel(const OT *__restrict__ y, const int32_t *__restrict__ place_of, int top, const OT *__restrict__ shared, int W,
                                                          OT *__restrict__ out, const float *__restrict__ score, const float *__restrict__ shared_gate, int64_t gate_ld,
                                                          const OT *__restrict__ ident, int64_t ldi) {
    const int64_t t = blockIdx.x;
    const float sg = (shared && shared_gate) ? sigmoid_f(shared_gate[t * gate_ld]) : 1.f;
    for (int c = threadIdx.x; c < W; c += 256) {
        float v = shared ? ld_f(shared, t * W + c) * sg : 0.f;
        for (int k = 0; k < top; ++k) {
            const int64_t place = place_of[t * top + k];
            v += (place < 0 ? ld_f(ident, t * ldi + c) : ld_f(y, place * W + c)) * (score ? score[t * top + k] : 1.f);
        }
        st_f(out, t * W + c, v);
    }
}

// 16-bit rows, 8 numbers per thread (W and the strides multiples of 8, 16-byte aligned rows); the choices' rows are requested four at a time
__global__ __launch_bounds__(256) void moe_combine8_kernel(const bf16_t *__restrict__ y, const int32_t *__restrict__ place_of, int top, const bf16_t *__restrict__ shared, int W8, int64_t T,
                                                           bf16_t *__restrict__ out, const float *__restrict__ score, const float *__restrict__ shared_gate, int64_t gate_ld,
                                                           const bf16_t *__restrict__ ident, int64_t ldi) {
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x, t = idx / W8;
    if (t >= T) return;
    const int64_t c = (idx - t * W8) * 8, W = (int64_t)W8 * 8;
    float acc[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[e] = 0.f;
    if (shared) {
        const float sg = shared_gate ? sigmoid_f(shared_gate[t * gate_ld]) : 1.f;
        const uint4 v = *reinterpret_cast<const uint4 *>(shared + t * W + c); const bf16_t *ve = reinterpret_cast<const bf16_t *>(&v);
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] = ld_f(ve, e) * sg;
    }
    for (int k0 = 0; k0 < top; k0 += 4) {
        uint4 v[4]; float sc[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const bool on = k0 + k < top;
            const int64_t i = t * top + (on ? k0 + k : 0), place = place_of[i];
            sc[k] = on ? (score ? score[i] : 1.f) : 0.f;
            v[k] = *reinterpret_cast<const uint4 *>(place < 0 ? ident + t * ldi + c : y + place * W + c);
        }
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            if (k0 + k >= top) break;
            const bf16_t *ve = reinterpret_cast<const bf16_t *>(&v[k]);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[e] += ld_f(ve, e) * sc[k];
        }
    }
    uint4 o; bf16_t *oe = reinterpret_cast<bf16_t *>(&o);
#pragma unroll
    for (int e = 0; e < 8; ++e) st_f(oe, e, acc[e]);
    *reinterpret_cast<uint4 *>(out + t * W + c) = o;
}

// out = z Phi(z) (rows of F numbers)
template <class CT>
__global__ __launch_bounds__(256) void gelu_erf_kernel(const CT *z, int64_t ldz, int64_t T, int64_t F, CT *out, int64_t ldo) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= T * F) return;
    const int64_t t = i / F, c = i - t * F;
    st_f(out, t * ldo + c, gelu_erf_f(ld_f(z, t * ldz + c)));
}

// the same for 16-bit rows, 8 numbers per thread (F and both strides multiples of 8, 16-byte aligned rows)
__global__ __launch_bounds__(256) void gelu_erf8_kernel(const bf16_t *z, int64_t ldz, int64_t T, int64_t F8, bf16_t *out, int64_t ldo) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= T * F8) return;
    const int64_t t = i / F8, c = (i - t * F8) * 8;
    uint4 v = *reinterpret_cast<const uint4 *>(z + t * ldz + c);
    bf16_t *e = reinterpret_cast<bf16_t *>(&v);
#pragma unroll
    for (int k = 0; k < 8; ++k) st_f(e, k, gelu_erf_f(ld_f(e, k)));
    *reinterpret_cast<uint4 *>(out + t * ldo + c) = v;
}

// ------------------------------------------------------------------------------------------------ rows of the stream in registers
// NJ_JOIN: x += y / rms(y) * wb; then, where asked for, out = x / rms(x) * wn, or (plain) x itself in the operand type.  NJ_NORM: out = x / rms(x) * wn alone, of the rows rows[r] (null: r).
// NJ_START: x = E[id] scale + P[position] (P null: without), then out = x / rms(x) * wn.  16-bit operands, widths that are multiples of 4, one norm group: NT threads per row (64: a wave,
// four rows per workgroup, no barrier; 256: the workgroup).
enum { NJ_JOIN = 0, NJ_NORM = 1, NJ_START = 2 };
struct NormJoin { float *x; const bf16_t *y; int64_t ldy, T; int W; float eps; const float *wb, *wn; int plain; bf16_t *out; int64_t ldo; const int32_t *rows; int64_t ldx; const bf16_t *E, *P; float scale; };
__device__ __forceinline__ float4 unpack4(uint2 v) { return float4{__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16), __uint_as_float(v.y & 0xffff0000u)}; }
__device__ __forceinline__ uint2 pack4(float4 v) {
    bf16_t h[4];
    st_f(h, 0, v.x); st_f(h, 1, v.y); st_f(h, 2, v.z); st_f(h, 3, v.w);
    return uint2{(uint32_t)h[0] | ((uint32_t)h[1] << 16), (uint32_t)h[2] | ((uint32_t)h[3] << 16)};
}
__device__ __forceinline__ float square4(float4 v) { return (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w); }
template <int NT, int NV, int KIND>
__global__ __launch_bounds__(256) void norm_join4_kernel(NormJoin a, Batch b) {
    __shared__ float red[4];
    const int W4 = a.W >> 2, l = threadIdx.x & (NT - 1);
    const int64_t t = (int64_t)blockIdx.x * (256 / NT) + threadIdx.x / NT;
    if (NT == 64 && t >= a.T) return;                   // (a whole wave: nobody waits for it)
    float *xr = a.x + (KIND == NJ_NORM && a.rows ? (int64_t)a.rows[t] : t) * a.ldx;
    const bf16_t *er = nullptr, *pr = nullptr;
    if (KIND == NJ_START) {
        er = a.E + b.ids[t] * (int64_t)a.W;
        const int sq = b.row_seq[t];
        if (a.P) pr = a.P + (int64_t)(b.start[sq] + ((int)t - b.cu[sq])) * a.W;
    }
    float4 xs[NV], ys[NV];
    float ss = 0.f, s2 = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c4 = l + k * NT;
        xs[k] = ys[k] = float4{0.f, 0.f, 0.f, 0.f};
        if (c4 < W4) {
            if (KIND == NJ_START) {
                const float4 e = unpack4(*reinterpret_cast<const uint2 *>(er + c4 * 4));
                xs[k] = float4{e.x * a.scale, e.y * a.scale, e.z * a.scale, e.w * a.scale};
                if (pr) { const float4 q = unpack4(*reinterpret_cast<const uint2 *>(pr + c4 * 4)); xs[k].x += q.x; xs[k].y += q.y; xs[k].z += q.z; xs[k].w += q.w; }
                *reinterpret_cast<float4 *>(xr + c4 * 4) = xs[k];
            } else xs[k] = *reinterpret_cast<const float4 *>(xr + c4 * 4);
            if (KIND == NJ_JOIN) ys[k] = unpack4(*reinterpret_cast<const uint2 *>(a.y + t * a.ldy + c4 * 4));
        }
        if (KIND == NJ_JOIN) ss += square4(ys[k]); else s2 += square4(xs[k]);
    }
    if (KIND == NJ_JOIN) {
        const float f = 1.0f / sqrtf((NT == 64 ? wave_sum(ss) : block_sum256(ss, red)) / (float)a.W + a.eps);
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int c4 = l + k * NT;
            if (c4 < W4) {
                const float4 w = *reinterpret_cast<const float4 *>(a.wb + c4 * 4);
                xs[k].x += ys[k].x * f * w.x; xs[k].y += ys[k].y * f * w.y; xs[k].z += ys[k].z * f * w.z; xs[k].w += ys[k].w * f * w.w;
                *reinterpret_cast<float4 *>(xr + c4 * 4) = xs[k];
                s2 += square4(xs[k]);
            }
        }
        if (!a.wn && !a.plain) return;
    }
    const float f2 = a.wn ? 1.0f / sqrtf((NT == 64 ? wave_sum(s2) : block_sum256(s2, red)) / (float)a.W + a.eps) : 1.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c4 = l + k * NT;
        if (c4 < W4) {
            const float4 w = a.wn ? *reinterpret_cast<const float4 *>(a.wn + c4 * 4) : float4{1.f, 1.f, 1.f, 1.f};
            *reinterpret_cast<uint2 *>(a.out + t * a.ldo + c4 * 4) = pack4(float4{xs[k].x * f2 * w.x, xs[k].y * f2 * w.y, xs[k].z * f2 * w.z, xs[k].w * f2 * w.w});
        }
    }
}

// The end of a layer with a token input for few rows, a workgroup of 1024 per row: a sublayer's result joins (x += y / rms(y) * wb), z = Wg x, g = gelu_tanh(z) * E[id], u = Wp g,
// x += u / rms(u) * ws, and the next norm.  The roundings are those of the launches it stands for (x, z, g and u as 16-bit operands).
template <int NV>
__global__ __launch_bounds__(1024) void side_step_kernel(SideStepArgs a) {
    extern __shared__ __attribute__((aligned(16))) char sm_[];
    bf16_t *xb = (bf16_t *)sm_; bf16_t *gs = xb + a.W;   // [W] x, [dim] g, operand type
    __shared__ float red[16];
    const int64_t t = blockIdx.x;
    const int W = a.W, W4 = W >> 2, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, dim = a.dim;
    auto sum_all = [&](float v) {
        v = wave_sum(v);
        __syncthreads();
        if (lane == 0) red[wave] = v;
        __syncthreads();
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < 16; ++i) s += red[i];
        return s;
    };
    float *xr = a.x + t * W;
    float4 xs[NV], ys[NV];
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c4 = tid + k * 1024;
        xs[k] = ys[k] = float4{0.f, 0.f, 0.f, 0.f};
        if (c4 < W4) { xs[k] = *reinterpret_cast<const float4 *>(xr + c4 * 4); ys[k] = unpack4(*reinterpret_cast<const uint2 *>((const bf16_t *)a.y + t * a.ldy + c4 * 4)); }
        ss += square4(ys[k]);
    }
    const float f = 1.0f / sqrtf(sum_all(ss) / (float)W + a.eps);
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c4 = tid + k * 1024;
        if (c4 < W4) {
            const float4 w = *reinterpret_cast<const float4 *>(a.wb + c4 * 4);
            xs[k].x += ys[k].x * f * w.x; xs[k].y += ys[k].y * f * w.y; xs[k].z += ys[k].z * f * w.z; xs[k].w += ys[k].w * f * w.w;
            *reinterpret_cast<uint2 *>(xb + c4 * 4) = pack4(xs[k]);
        }
    }
    __syncthreads();
    const bf16_t *Wg = (const bf16_t *)a.gate, *er = (const bf16_t *)a.E + a.ids[t] * a.lde + a.ecol;
    auto dot8 = [](uint4 u, uint4 v, float acc) {
        const bf16_t *ue = reinterpret_cast<const bf16_t *>(&u), *ve = reinterpret_cast<const bf16_t *>(&v);
#pragma unroll
        for (int k = 0; k < 8; ++k) acc = fmaf(ld_f(ue, k), ld_f(ve, k), acc);
        return acc;
    };
    for (int d0 = wave * 4; d0 < dim; d0 += 64) {       // four numbers of z per wave at a time
        float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
        for (int c = lane * 8; c < W; c += 512) {
            const uint4 xv = *reinterpret_cast<const uint4 *>(xb + c);
            uint4 wv[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) wv[i] = *reinterpret_cast<const uint4 *>(Wg + (int64_t)min(d0 + i, dim - 1) * W + c);
#pragma unroll
            for (int i = 0; i < 4; ++i) acc[i] = dot8(wv[i], xv, acc[i]);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float z = wave_sum(acc[i]);
            if (lane == 0 && d0 + i < dim) { bf16_t h; st_f(&h, 0, z); st_f(gs, d0 + i, gelu_tanh_f(ld_f(&h, 0)) * ld_f(er, d0 + i)); }
        }
    }
    __syncthreads();
    const bf16_t *Wp = (const bf16_t *)a.proj;
    float s1 = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c4 = tid + k * 1024;
        ys[k] = float4{0.f, 0.f, 0.f, 0.f};
        if (c4 < W4) {
            float acc[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
            for (int d = 0; d < dim; d += 8) {
                const uint4 gv = *reinterpret_cast<const uint4 *>(gs + d);
#pragma unroll
                for (int i = 0; i < 4; ++i) acc[i] = dot8(*reinterpret_cast<const uint4 *>(Wp + (int64_t)(c4 * 4 + i) * dim + d), gv, acc[i]);
            }
            ys[k] = unpack4(pack4(float4{acc[0], acc[1], acc[2], acc[3]}));
        }
        s1 += square4(ys[k]);
    }
    const float f1 = 1.0f / sqrtf(sum_all(s1) / (float)W + a.eps);
    float s2 = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c4 = tid + k * 1024;
        if (c4 < W4) {
            const float4 w = *reinterpret_cast<const float4 *>(a.ws + c4 * 4);
            xs[k].x += ys[k].x * f1 * w.x; xs[k].y += ys[k].y * f1 * w.y; xs[k].z += ys[k].z * f1 * w.z; xs[k].w += ys[k].w * f1 * w.w;
            *reinterpret_cast<float4 *>(xr + c4 * 4) = xs[k];
            s2 += square4(xs[k]);
        }
    }
    if (!a.wn) return;
    const float f2 = 1.0f / sqrtf(sum_all(s2) / (float)W + a.eps);
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c4 = tid + k * 1024;
        if (c4 < W4) {
            const float4 w = *reinterpret_cast<const float4 *>(a.wn + c4 * 4);
            *reinterpret_cast<uint2 *>((bf16_t *)a.out + t * a.ldo + c4 * 4) = pack4(float4{xs[k].x * f2 * w.x, xs[k].y * f2 * w.y, xs[k].z * f2 * w.z, xs[k].w * f2 * w.w});
        }
    }
}

// ------------------------------------------------------------------------------------------------ end of a layer
// Per row: (1) the token input's last step: x += y / rms(y) * wn for the projected rows y (side_y); (2) X_(i+1) = x goes to its
// place among the kept streams and x becomes sum_j mix[j] X_j over the nx kept streams (X_0 the embedding output ... X_(nx-1) this layer's); (3) with wnext the next layer's
// first norm (in groups) of the new x goes to out.  Each part is optional (null pointers).  The row lives in LDS.
template <class OT>
__global__ __launch_bounds__(256) void layer_tail_kernel(LayerTailArgs p) {
    extern __shared__ float sm[];                       // [W] x, [W] y
    __shared__ float red[4];
    const int64_t t = blockIdx.x; const int W = p.W, lane = threadIdx.x & 63;
    float *xs = sm, *ys = sm + W;
    float *xr = p.x + t * W;
    for (int c = threadIdx.x; c < W; c += 256) xs[c] = xr[c];
    __syncthreads();
    if (p.side_y) {
        const OT *sy = (const OT *)p.side_y + t * W;
        float ss = 0.f;
        for (int c = threadIdx.x; c < W; c += 256) { const float y = ld_f(sy, c); ys[c] = y; ss += y * y; }
        ss = block_sum256(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)W + p.eps);
        for (int c = threadIdx.x; c < W; c += 256) xs[c] += ys[c] * inv * p.side_norm[c];
        __syncthreads();
    }
    if (p.kept) {
        float *mine = p.kept + ((int64_t)(p.nx - 1) * p.kept_rows + t) * W;
        const float wl = p.mix[p.nx - 1];
        for (int c = threadIdx.x; c < W; c += 256) {
            const float v = xs[c];
            mine[c] = v;
            float acc = 0.f;
            for (int jx = 0; jx < p.nx - 1; ++jx) acc = fmaf(p.mix[jx], p.kept[((int64_t)jx * p.kept_rows + t) * W + c], acc);
            xs[c] = fmaf(wl, v, acc);
        }
        __syncthreads();
    }
    for (int c = threadIdx.x; c < W; c += 256) xr[c] = xs[c];
    if (p.wnext) {
        const int n = W / p.groups;
        OT *o = (OT *)p.out + t * W;
        for (int g = threadIdx.x >> 6; g < p.groups; g += 4) {
            float ss = 0.f;
            for (int c = lane; c < n; c += 64) { const float v = xs[g * n + c]; ss += v * v; }
            const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)n + p.eps);
            for (int c = lane; c < n; c += 64) st_f(o, g * n + c, xs[g * n + c] * inv * p.wnext[g * n + c]);
        }
    }
}

// g[t][d] = gelu_tanh(z[t][d]) * E[ids[t]][ecol + d] (the token input between its two projections)
template <class OT>
__global__ __launch_bounds__(256) void side_gate_kernel(const OT *__restrict__ z, const int64_t *__restrict__ ids, const OT *__restrict__ E, int64_t lde, int ecol, int dim,
                                                        int64_t n, OT *__restrict__ g) {
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= n) return;
    const int64_t t = idx / dim; const int d = (int)(idx - t * dim);
    st_f(g, idx, gelu_tanh_f(ld_f(z, idx)) * ld_f(E, ids[t] * lde + ecol + d));
}

// y[t][c] *= sigmoid(g[t][c])
template <class OT>
__global__ __launch_bounds__(256) void sigmoid_gate_kernel(OT *__restrict__ y, int64_t ldy, const OT *__restrict__ g, int64_t ldg, int64_t T, int64_t N) {
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= T * N) return;
    const int64_t t = idx / N, c = idx - t * N;
    st_f(y, t * ldy + c, ld_f(y, t * ldy + c) * sigmoid_f(ld_f(g, t * ldg + c)));
}

// the same for 16-bit rows, 8 numbers per thread (N and both strides multiples of 8, 16-byte aligned rows)
__global__ __launch_bounds__(256) void sigmoid_gate8_kernel(bf16_t *__restrict__ y, int64_t ldy, const bf16_t *__restrict__ g, int64_t ldg, int64_t T, int64_t N8) {
    const int64_t idx = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= T * N8) return;
    const int64_t t = idx / N8, c = (idx - t * N8) * 8;
    uint4 yv = *reinterpret_cast<const uint4 *>(y + t * ldy + c);
    const uint4 gv = *reinterpret_cast<const uint4 *>(g + t * ldg + c);
    bf16_t *ye = reinterpret_cast<bf16_t *>(&yv); const bf16_t *ge = reinterpret_cast<const bf16_t *>(&gv);
#pragma unroll
    for (int k = 0; k < 8; ++k) st_f(ye, k, ld_f(ye, k) * sigmoid_f(ld_f(ge, k)));
    *reinterpret_cast<uint4 *>(y + t * ldy + c) = yv;
}

template <class ET>
__global__ __launch_bounds__(256) void embed_keep_kernel(const ET *__restrict__ E, const int64_t *__restrict__ ids, int W, float *__restrict__ x, float *__restrict__ kept) {
    const int64_t t = blockIdx.x, id = ids[t];
    for (int c = threadIdx.x; c < W; c += 256) { const float v = ld_f(E, id * W + c); x[t * W + c] = v; if (kept) kept[t * W + c] = v; }
}

}  // namespace

static const size_t kMaxLds = 160 * 1024 - 2048;

int prepare_blocks() {
    NVR_HIP_CHECK(hipFuncSetAttribute((const void *)layer_tail_kernel<float>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds));
    NVR_HIP_CHECK(hipFuncSetAttribute((const void *)layer_tail_kernel<bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds));
    return 0;
}

int embed_keep(const void *E, bool bf16, const int64_t *ids, int64_t T, int64_t W, float *x, float *kept, hipStream_t s) {
    if (T == 0) return 0;
    if (bf16) embed_keep_kernel<bf16_t><<<dim3((unsigned)T), dim3(256), 0, s>>>((const bf16_t *)E, ids, (int)W, x, kept);
    else embed_keep_kernel<float><<<dim3((unsigned)T), dim3(256), 0, s>>>((const float *)E, ids, (int)W, x, kept);
    return launched("embed_keep");
}

static bool aligned16(const void *p) { return ((uintptr_t)p & 15) == 0; }

static bool norm_join4_ok(int64_t W, const float *x, const void *y, int64_t ldy, const float *wb, const float *wn, const void *out, int64_t ldo) {
    return W % 4 == 0 && W <= 8192 && ldy % 4 == 0 && ldo % 4 == 0 && aligned16(x) && aligned16(y) && aligned16(wb) && aligned16(wn) && aligned16(out);
}
template <int KIND>
static int norm_join4(const NormJoin &a, const Batch &b, hipStream_t s) {
    const int64_t W4 = a.W / 4;
    const bool wave = a.T >= 1024 && W4 <= 256;         // many rows: a wave per row up to 1024 numbers; few rows: a workgroup per row
    const dim3 grid((unsigned)(wave ? (a.T + 3) / 4 : a.T)), blk(256);
#define NVR_NJ(NT_, NV_) norm_join4_kernel<NT_, NV_, KIND><<<grid, blk, 0, s>>>(a, b)
    if (wave) { if (W4 <= 64) NVR_NJ(64, 1); else if (W4 <= 128) NVR_NJ(64, 2); else NVR_NJ(64, 4); }
    else if (W4 <= 256) NVR_NJ(256, 1); else if (W4 <= 512) NVR_NJ(256, 2); else if (W4 <= 1024) NVR_NJ(256, 4); else NVR_NJ(256, 8);
#undef NVR_NJ
    return launched("norm_join4");
}

int embed_norm(const void *E, const void *P, bool bf16, const Batch &b, int64_t W, float scale, float *x, float eps, const float *wn, void *out, hipStream_t s) {
    if (b.T == 0) return 0;
    if (bf16 && norm_join4_ok(W, x, E, W, wn, wn, out, W) && aligned16(P)) {
        NormJoin j{}; j.x = x; j.ldx = W; j.T = b.T; j.W = (int)W; j.eps = eps; j.wn = wn; j.out = (bf16_t *)out; j.ldo = W; j.E = (const bf16_t *)E; j.P = (const bf16_t *)P; j.scale = scale;
        return norm_join4<NJ_START>(j, b, s);
    }
    if (int rc = embed_pos(E, P, bf16, b, W, scale, x, s)) return rc;
    GroupNormArgs n{}; n.in = x; n.ldi = W; n.in_f32 = true; n.rows_n = b.T; n.W = W; n.groups = 1; n.eps = eps; n.w = wn; n.out = out; n.ldo = W;
    return group_norm(n, bf16, s);
}

bool side_step_ok(const SideStepArgs &a, bool bf16) {
    return bf16 && a.T <= 64 && a.W % 8 == 0 && a.W <= 8192 && a.dim % 8 == 0 && a.dim <= 4096 && a.ldy % 4 == 0 && a.ldo % 4 == 0 && aligned16(a.x) && aligned16(a.y) && aligned16(a.wb) && aligned16(a.ws) && aligned16(a.wn) &&
           aligned16(a.out) && aligned16(a.gate) && aligned16(a.proj);
}
int side_step(const SideStepArgs &a, hipStream_t s) {
    if (a.T == 0) return 0;
    if (!side_step_ok(a, true)) return nvr::fail(NVR_ERR_UNSUPPORTED, "side_step: %d rows of %d numbers, token input of %d", a.T, a.W, a.dim);
    const size_t lds = (size_t)(a.W + a.dim) * 2;
    if (a.W <= 4096) side_step_kernel<1><<<dim3((unsigned)a.T), dim3(1024), lds, s>>>(a);
    else side_step_kernel<2><<<dim3((unsigned)a.T), dim3(1024), lds, s>>>(a);
    return launched("side_step");
}

int group_norm(const GroupNormArgs &a, bool bf16, hipStream_t s) {
    if (a.rows_n == 0) return 0;
    if (a.groups < 1 || a.W % a.groups) return nvr::fail(NVR_ERR_INVALID_ARG, "group_norm: %ld columns in %d groups", (long)a.W, a.groups);
    if (bf16 && a.xres && a.groups == 1 && !a.in_f32 && !a.rows && !(a.w2 && a.out_plain) && norm_join4_ok(a.W, a.xres, a.in, a.ldi, a.w, a.w2, a.out, a.ldo))
    {
        NormJoin j{}; j.x = a.xres; j.ldx = a.W; j.y = (const bf16_t *)a.in; j.ldy = a.ldi; j.T = a.rows_n; j.W = (int)a.W; j.eps = a.eps; j.wb = a.w; j.wn = a.w2; j.plain = a.out_plain ? 1 : 0; j.out = (bf16_t *)a.out; j.ldo = a.ldo;
        return norm_join4<NJ_JOIN>(j, Batch{}, s);
    }
    if (bf16 && !a.xres && a.groups == 1 && a.in_f32 && norm_join4_ok(a.W, (const float *)a.in, nullptr, a.ldi, nullptr, a.w, a.out, a.ldo)) {
        NormJoin j{}; j.x = (float *)a.in; j.ldx = a.ldi; j.rows = a.rows; j.T = a.rows_n; j.W = (int)a.W; j.eps = a.eps; j.wn = a.w; j.out = (bf16_t *)a.out; j.ldo = a.ldo;
        return norm_join4<NJ_NORM>(j, Batch{}, s);
    }
    if (a.out_plain && (a.w2 || !a.xres)) return nvr::fail(NVR_ERR_INVALID_ARG, "group_norm: a plain copy leaves only with the residual sum, instead of the next norm");
    const dim3 grid((unsigned)a.rows_n), blk(256);
    const int W = (int)a.W;
    if (a.xres) {                                        // operand-type rows joining the f32 stream
        if (bf16) group_norm_kernel<bf16_t, bf16_t, true><<<grid, blk, 0, s>>>((const bf16_t *)a.in, a.ldi, nullptr, W, a.groups, a.eps, a.w, a.xres, a.w2, a.out_plain ? 1 : 0, (bf16_t *)a.out, a.ldo);
        else group_norm_kernel<float, float, true><<<grid, blk, 0, s>>>((const float *)a.in, a.ldi, nullptr, W, a.groups, a.eps, a.w, a.xres, a.w2, a.out_plain ? 1 : 0, (float *)a.out, a.ldo);
    } else if (a.in_f32) {
        if (bf16) group_norm_kernel<float, bf16_t, false><<<grid, blk, 0, s>>>((const float *)a.in, a.ldi, a.rows, W, a.groups, a.eps, a.w, nullptr, nullptr, 0, (bf16_t *)a.out, a.ldo);
        else group_norm_kernel<float, float, false><<<grid, blk, 0, s>>>((const float *)a.in, a.ldi, a.rows, W, a.groups, a.eps, a.w, nullptr, nullptr, 0, (float *)a.out, a.ldo);
    } else {
        if (bf16) group_norm_kernel<bf16_t, bf16_t, false><<<grid, blk, 0, s>>>((const bf16_t *)a.in, a.ldi, a.rows, W, a.groups, a.eps, a.w, nullptr, nullptr, 0, (bf16_t *)a.out, a.ldo);
        else group_norm_kernel<float, float, false><<<grid, blk, 0, s>>>((const float *)a.in, a.ldi, a.rows, W, a.groups, a.eps, a.w, nullptr, nullptr, 0, (float *)a.out, a.ldo);
    }
    return launched("group_norm");
}

int latent_rope(const LatentRopeArgs &a, const Batch &b, bool bf16, hipStream_t s) {
    if (b.T == 0) return 0;
    if (a.rot % 2) return nvr::fail(NVR_ERR_INVALID_ARG, "latent_rope: %d rotated coordinates", a.rot);
    const bool turns = a.q && a.rot > 0;
    if (!a.pages && !turns) return 0;
    const bool vec = bf16 && a.rot % (a.halves ? 16 : 8) == 0 && a.rot <= 4096 && (!a.pages || (a.rank % 8 == 0 && a.ld % 8 == 0 && a.col % 8 == 0 && aligned16(a.proj) && aligned16(a.pages) && aligned16(a.rows))) &&
                     (!turns || (((a.ldq | a.qstride | a.qcol | a.ldo | a.ostride | a.ocol) & 7) == 0 && aligned16(a.q) && aligned16(a.out)));
    if (vec) {
        LatentRopeArgs v = a;
        if (!turns) v.q = nullptr;
        const size_t lds = (size_t)std::max(a.rot / 2, 1) * sizeof(float2);
        if (b.T >= 1024 && 4 * lds <= 60000) latent_rope8_kernel<4><<<dim3((unsigned)((b.T + 3) / 4)), dim3(256), 4 * lds, s>>>(v, b);
        else latent_rope8_kernel<1><<<dim3((unsigned)b.T), dim3(256), lds, s>>>(v, b);
        return launched("latent_rope");
    }
    const int hv = a.halves ? 1 : 0;
    if (a.pages) {
        if (bf16) latent_store_kernel<bf16_t><<<dim3((unsigned)b.T), dim3(64), 0, s>>>((const bf16_t *)a.proj, a.ld, a.col, b, a.rank, a.rot, a.eps, a.w, a.freq, (bf16_t *)a.pages, (bf16_t *)a.rows, hv, a.gain);
        else latent_store_kernel<float><<<dim3((unsigned)b.T), dim3(64), 0, s>>>((const float *)a.proj, a.ld, a.col, b, a.rank, a.rot, a.eps, a.w, a.freq, (float *)a.pages, (float *)a.rows, hv, a.gain);
    }
    if (turns) {
        if (bf16) rotate_heads_kernel<bf16_t><<<dim3((unsigned)b.T), dim3(256), 0, s>>>((const bf16_t *)a.q, a.ldq, (int)a.qstride, (int)a.qcol, b, a.H, a.rot, a.freq, (bf16_t *)a.out, a.ldo, (int)a.ostride, (int)a.ocol, hv, a.gain);
        else rotate_heads_kernel<float><<<dim3((unsigned)b.T), dim3(256), 0, s>>>((const float *)a.q, a.ldq, (int)a.qstride, (int)a.qcol, b, a.H, a.rot, a.freq, (float *)a.out, a.ldo, (int)a.ostride, (int)a.ocol, hv, a.gain);
    }
    return launched("latent_rope");
}

int head_linear(const HeadLinearArgs &a, bool bf16, hipStream_t s) {
    if (a.T == 0 || a.N == 0 || a.H == 0) return 0;
    if (bf16 && a.K % 8 == 0 && a.lda % 8 == 0 && a.ha % 8 == 0 && aligned16(a.a) && aligned16(a.w)) {
        if (a.T >= 128) head_linear_mfma128_kernel<<<dim3((unsigned)((a.N + 127) / 128), (unsigned)((a.T + 127) / 128), (unsigned)a.H), dim3(256), 0, s>>>(a);
        else if (a.T <= 16) head_linear_ksplit_kernel<<<dim3((unsigned)((a.N + 63) / 64), (unsigned)((a.T + 15) / 16), (unsigned)a.H), dim3(256), 0, s>>>(a);
        else head_linear_mfma_kernel<4><<<dim3((unsigned)((a.N + 63) / 64), (unsigned)((a.T + 63) / 64), (unsigned)a.H), dim3(256), 0, s>>>(a);
        return launched("head_linear");
    }
    const dim3 grid((unsigned)((a.N + 63) / 64), (unsigned)((a.T + 63) / 64), (unsigned)a.H);
    if (bf16) head_linear_kernel<bf16_t><<<grid, dim3(256), 0, s>>>(a);
    else head_linear_kernel<float><<<grid, dim3(256), 0, s>>>(a);
    return launched("head_linear");
}

int grouped_linear(const GroupedLinearArgs &a, bool bf16, hipStream_t s) {
    if (a.max_rows == 0 || a.N == 0 || a.groups == 0) return 0;
    if (bf16 && a.K % 8 == 0 && a.lda % 8 == 0 && aligned16(a.a) && aligned16(a.w)) {
        if (a.max_rows >= 96 * a.groups) grouped_linear_mfma128_kernel<<<dim3((unsigned)((a.N + 127) / 128), (unsigned)(a.max_rows / 128 + a.groups)), dim3(256), 0, s>>>(a);
        else if (a.max_rows <= 16 * a.groups) grouped_linear_ksplit_kernel<<<dim3((unsigned)((a.N + 63) / 64), (unsigned)(a.max_rows / 16 + a.groups)), dim3(256), 0, s>>>(a);
        else grouped_linear_mfma_kernel<4><<<dim3((unsigned)((a.N + 63) / 64), (unsigned)(a.max_rows / 64 + a.groups)), dim3(256), 0, s>>>(a);
        return launched("grouped_linear");
    }
    const dim3 grid((unsigned)((a.N + 63) / 64), (unsigned)(a.max_rows / 64 + a.groups));
    if (bf16) grouped_linear_kernel<bf16_t><<<grid, dim3(256), 0, s>>>(a);
    else grouped_linear_kernel<float><<<grid, dim3(256), 0, s>>>(a);
    return launched("grouped_linear");
}

int poly_norm(const void *z, int64_t ldz, int64_t T, int64_t F, float eps, const float *coef, void *out, int64_t ldo, bool bf16, hipStream_t s) {
    if (T == 0) return 0;
    if (bf16) poly_norm_kernel<bf16_t><<<dim3((unsigned)T), dim3(256), 0, s>>>((const bf16_t *)z, ldz, (int)F, eps, coef, (bf16_t *)out, ldo);
    else poly_norm_kernel<float><<<dim3((unsigned)T), dim3(256), 0, s>>>((const float *)z, ldz, (int)F, eps, coef, (float *)out, ldo);
    return launched("poly_norm");
}

template <bool GELU>
static int gated_mul(const void *gu, int64_t T, int64_t F, void *out, int64_t ldo, bool bf16, hipStream_t s) {
    if (T * F == 0) return 0;
    if (bf16 && F % 8 == 0 && ldo % 8 == 0 && aligned16(gu) && aligned16(out)) {
        gated_mul8_kernel<GELU><<<dim3((unsigned)((T * (F / 8) + 255) / 256)), dim3(256), 0, s>>>((const bf16_t *)gu, T, F / 8, (bf16_t *)out, ldo);
        return launched("gated_mul");
    }
    const dim3 grid((unsigned)((T * F + 255) / 256));
    if (bf16) gated_mul_kernel<bf16_t, GELU><<<grid, dim3(256), 0, s>>>((const bf16_t *)gu, T, F, (bf16_t *)out, ldo);
    else gated_mul_kernel<float, GELU><<<grid, dim3(256), 0, s>>>((const float *)gu, T, F, (float *)out, ldo);
    return launched("gated_mul");
}
int silu_mul(const void *gu, int64_t T, int64_t F, void *out, int64_t ldo, bool bf16, hipStream_t s) { return gated_mul<false>(gu, T, F, out, ldo, bf16, s); }
int gelu_mul(const void *gu, int64_t T, int64_t F, void *out, int64_t ldo, bool bf16, hipStream_t s) { return gated_mul<true>(gu, T, F, out, ldo, bf16, s); }

int gelu_erf(const void *z, int64_t ldz, int64_t T, int64_t F, void *out, int64_t ldo, bool bf16, hipStream_t s) {
    if (T * F == 0) return 0;
    if (bf16 && F % 8 == 0 && ldz % 8 == 0 && ldo % 8 == 0 && aligned16(z) && aligned16(out)) {
        gelu_erf8_kernel<<<dim3((unsigned)((T * (F / 8) + 255) / 256)), dim3(256), 0, s>>>((const bf16_t *)z, ldz, T, F / 8, (bf16_t *)out, ldo);
        return launched("gelu_erf");
    }
    const dim3 grid((unsigned)((T * F + 255) / 256));
    if (bf16) gelu_erf_kernel<bf16_t><<<grid, dim3(256), 0, s>>>((const bf16_t *)z, ldz, T, F, (bf16_t *)out, ldo);
    else gelu_erf_kernel<float><<<grid, dim3(256), 0, s>>>((const float *)z, ldz, T, F, (float *)out, ldo);
    return launched("gelu_erf");
}

int moe_route(const void *h, int64_t ldh, int64_t T, int64_t W, const float *wr, int64_t E, int64_t top, int32_t *sel, float *score, int32_t *off, int32_t *order,
              int32_t *place_of, int64_t pad, int32_t *row_w, int64_t nblocks, bool bf16, hipStream_t s, bool softmax, int64_t extra, float *extra_out,
              const float *logits, int64_t ldl, const float *correction, int64_t identity) {
    if (T == 0) return 0;
    if (correction && !softmax) return nvr::fail(NVR_ERR_INVALID_ARG, "moe_route: a correction belongs to softmax scores");
    if (identity < 0 || identity >= E) return nvr::fail(NVR_ERR_INVALID_ARG, "moe_route: %ld of %ld experts without a matrix", (long)identity, (long)E);
    if (extra < 0 || (extra > 0 && !extra_out)) return nvr::fail(NVR_ERR_INVALID_ARG, "moe_route: %ld further rows without a place for them", (long)extra);
    if (top < 1 || top > E) return nvr::fail(NVR_ERR_INVALID_ARG, "moe_route: %ld of %ld experts", (long)top, (long)E);
    if ((size_t)(2 * E + extra + 1) * 4 > 60000) return nvr::fail(NVR_ERR_UNSUPPORTED, "moe_route: %ld experts", (long)E);
    if (logits && E <= 64 && extra <= 64 && T * top <= 1024 && pad == 1 && !row_w) {
        moe_route_group_kernel<<<dim3(1), dim3(1024), 0, s>>>((int)T, (int)E, (int)(E - identity), (int)top, sel, score, softmax ? 1 : 0, (int)extra, extra_out, logits, ldl, correction, off, order, place_of);
        return launched("moe_route");
    }
    if (logits && E <= 64 && extra <= 64)
        moe_route_wave_kernel<<<dim3((unsigned)((T + 3) / 4)), dim3(256), 0, s>>>((int)T, (int)E, (int)top, sel, score, softmax ? 1 : 0, (int)extra, extra_out, logits, ldl, correction);
    else if (bf16) moe_route_kernel<bf16_t><<<dim3((unsigned)T), dim3(256), (size_t)(E + extra + (correction ? E : 0)) * 4, s>>>((const bf16_t *)h, ldh, (int)W, wr, (int)E, (int)top, sel, score, softmax ? 1 : 0, (int)extra, extra_out, logits, ldl, correction);
    else moe_route_kernel<float><<<dim3((unsigned)T), dim3(256), (size_t)(E + extra + (correction ? E : 0)) * 4, s>>>((const float *)h, ldh, (int)W, wr, (int)E, (int)top, sel, score, softmax ? 1 : 0, (int)extra, extra_out, logits, ldl, correction);
    if (int rc = launched("moe_route")) return rc;
    if (pad < 1) return nvr::fail(NVR_ERR_INVALID_ARG, "moe_route: rows padded to %ld", (long)pad);
    if (row_w && T * top >= 4096 && E - identity <= 256) {            // many choices: the counts of the workgroups go behind row_w
        const int64_t n = T * top, El = E - identity, nb = std::min<int64_t>((n + 1023) / 1024, std::max<int64_t>(1, 1024 / El)), per = (n + nb - 1) / nb;
        int32_t *counts = row_w + nblocks;
        moe_count_kernel<<<dim3((unsigned)nb), dim3(256), (size_t)El * 4, s>>>(sel, (int)n, (int)per, (int)El, counts);
        moe_place_kernel<<<dim3((unsigned)nb), dim3(256), (size_t)(2 * El + 1) * 4, s>>>(sel, (int)n, (int)per, (int)El, (int)pad, (int)nblocks, counts, (int)nb, off, order, place_of, row_w);
        return launched("moe_place");
    }
    moe_group_kernel<<<dim3(1), dim3(1024), (size_t)(E - identity + 1) * 4, s>>>(sel, (int)(T * top), (int)(E - identity), (int)pad, (int)nblocks, off, order, place_of, row_w);
    return launched("moe_group");
}

int moe_gather(const void *h, int64_t ldh, int64_t T, int64_t W, int64_t top, const int32_t *place_of, const float *score, void *xs, bool bf16, hipStream_t s) {
    if (T * top == 0) return 0;
    if (bf16 && W % 8 == 0 && ldh % 8 == 0 && aligned16(h) && aligned16(xs)) {
        moe_gather8_kernel<<<dim3((unsigned)((T * (W / 8) + 255) / 256)), dim3(256), 0, s>>>((const bf16_t *)h, ldh, (int)(W / 8), (int)top, T, place_of, score, (bf16_t *)xs);
        return launched("moe_gather");
    }
    if (bf16) moe_gather_kernel<bf16_t><<<dim3((unsigned)(T * top)), dim3(256), 0, s>>>((const bf16_t *)h, ldh, (int)W, (int)top, place_of, score, (bf16_t *)xs);
    else moe_gather_kernel<float><<<dim3((unsigned)(T * top)), dim3(256), 0, s>>>((const float *)h, ldh, (int)W, (int)top, place_of, score, (float *)xs);
    return launched("moe_gather");
}

int moe_combine(const void *y, const int32_t *place_of, int64_t T, int64_t top, const void *shared, int64_t W, void *out, bool bf16, hipStream_t s,
                const float *score, const float *shared_gate, int64_t gate_ld, const void *ident, int64_t ldi) {
    if (T == 0) return 0;
    if (bf16 && W % 8 == 0 && ldi % 8 == 0 && aligned16(y) && aligned16(shared) && aligned16(out) && aligned16(ident)) {
        moe_combine8_kernel<<<dim3((unsigned)((T * (W / 8) + 255) / 256)), dim3(256), 0, s>>>((const bf16_t *)y, place_of, (int)top, (const bf16_t *)shared, (int)(W / 8), T, (bf16_t *)out, score, shared_gate,
                                                                                             gate_ld, (const bf16_t *)ident, ldi);
        return launched("moe_combine");
    }
    if (bf16) moe_combine_kernel<bf16_t><<<dim3((unsigned)T), dim3(256), 0, s>>>((const bf16_t *)y, place_of, (int)top, (const bf16_t *)shared, (int)W, (bf16_t *)out, score, shared_gate, gate_ld, (const bf16_t *)ident, ldi);
    else moe_combine_kernel<float><<<dim3((unsigned)T), dim3(256), 0, s>>>((const float *)y, place_of, (int)top, (const float *)shared, (int)W, (float *)out, score, shared_gate, gate_ld, (const float *)ident, ldi);
    return launched("moe_combine");
}

int sigmoid_gate(void *y, int64_t ldy, const void *g, int64_t ldg, int64_t T, int64_t N, bool bf16, hipStream_t s) {
    if (T * N == 0) return 0;
    if (bf16 && N % 8 == 0 && ldy % 8 == 0 && ldg % 8 == 0 && (((uintptr_t)y | (uintptr_t)g) & 15) == 0) {
        sigmoid_gate8_kernel<<<dim3((unsigned)((T * (N / 8) + 255) / 256)), dim3(256), 0, s>>>((bf16_t *)y, ldy, (const bf16_t *)g, ldg, T, N / 8);
        return launched("sigmoid_gate");
    }
    const dim3 grid((unsigned)((T * N + 255) / 256));
    if (bf16) sigmoid_gate_kernel<bf16_t><<<grid, dim3(256), 0, s>>>((bf16_t *)y, ldy, (const bf16_t *)g, ldg, T, N);
    else sigmoid_gate_kernel<float><<<grid, dim3(256), 0, s>>>((float *)y, ldy, (const float *)g, ldg, T, N);
    return launched("sigmoid_gate");
}

int side_gate(const void *z, const int64_t *ids, const void *E, int64_t lde, int64_t ecol, int64_t dim, int64_t T, void *g, bool bf16, hipStream_t s) {
    if (T * dim == 0) return 0;
    const dim3 grid((unsigned)((T * dim + 255) / 256));
    if (bf16) side_gate_kernel<bf16_t><<<grid, dim3(256), 0, s>>>((const bf16_t *)z, ids, (const bf16_t *)E, lde, (int)ecol, (int)dim, T * dim, (bf16_t *)g);
    else side_gate_kernel<float><<<grid, dim3(256), 0, s>>>((const float *)z, ids, (const float *)E, lde, (int)ecol, (int)dim, T * dim, (float *)g);
    return launched("side_gate");
}

int layer_tail(const LayerTailArgs &a, bool bf16, hipStream_t s) {
    if (a.T == 0) return 0;
    if (bf16 && a.side_y && !a.kept && (!a.wnext || a.groups == 1) && norm_join4_ok(a.W, a.x, a.side_y, a.W, a.side_norm, a.wnext, a.out, a.W))
    {
        NormJoin j{}; j.x = a.x; j.ldx = a.W; j.y = (const bf16_t *)a.side_y; j.ldy = a.W; j.T = a.T; j.W = a.W; j.eps = a.eps; j.wb = a.side_norm; j.wn = a.wnext; j.out = (bf16_t *)a.out; j.ldo = a.W;
        return norm_join4<NJ_JOIN>(j, Batch{}, s);
    }
    const size_t lds = (size_t)2 * a.W * 4;
    if (lds > kMaxLds) return nvr::fail(NVR_ERR_UNSUPPORTED, "layer_tail: rows of %d numbers do not fit LDS", a.W);
    if (a.wnext && (a.groups < 1 || a.W % a.groups)) return nvr::fail(NVR_ERR_INVALID_ARG, "layer_tail: %d columns in %d groups", a.W, a.groups);
    if (bf16) layer_tail_kernel<bf16_t><<<dim3((unsigned)a.T), dim3(256), lds, s>>>(a);
    else layer_tail_kernel<float><<<dim3((unsigned)a.T), dim3(256), lds, s>>>(a);
    return launched("layer_tail");
}

}}  // namespace nvr::kl
