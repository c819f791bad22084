// layered_streams.hip — blocks of layers whose residual is a set of parallel streams (kernels/layered.h): a sublayer's result written into the streams with the next
// sublayer's input read out of them and layer-normed in the same pass, and the queries / keys / values of an attention with projection biases, a rotation of number
// pairs, unit norms per head behind it and values mixed with an earlier layer's.  The streams, their sums, norms and angles are f32 in both operand types.  wave64, gfx950.
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
__device__ __forceinline__ uint32_t pack2(float a, float b) { bf16_t h[2]; st_f(h, 0, a); st_f(h, 1, b); return (uint32_t)h[0] | ((uint32_t)h[1] << 16); }
__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}
__device__ __forceinline__ float block_sum(float v, float *red) {           // 256 threads; red: 4 floats of LDS; every thread gets the sum
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    return (red[0] + red[1]) + (red[2] + red[3]);
}

int launched(const char *what) {
    hipError_t e = hipGetLastError();
    if (e != hipSuccess) return nvr::fail(NVR_ERR_HIP, "%s launch failed: %s", what, hipGetErrorString(e));
    return 0;
}

// ------------------------------------------------------------------------------------------------ parallel residual streams
// General form (any width, any number of streams that fits LDS): one workgroup per row.  A thread keeps the old streams of its column in LDS (its own slots, no
// barrier), forms the new ones, and leaves u = sum_s win[s] x_s in LDS for the norm.
enum { ST_START = 0, ST_STEP = 1, ST_SUM = 2 };
template <class OT, int MODE>
__global__ __launch_bounds__(256) void stream_step_kernel(StreamArgs a) {
    extern __shared__ float sm[];                       // [W] u, [S][256] old streams
    __shared__ float red[4];
    const int W = a.W, S = a.S, tid = threadIdx.x;
    const int64_t r = blockIdx.x, t = a.rows ? a.rows[r] : r;
    float *us = sm, *old = sm + W, *xr = a.x + t * S * W;
    const OT *er = MODE == ST_START ? (const OT *)a.E + a.ids[t] * (int64_t)W : nullptr;
    const OT *yr = MODE == ST_START ? nullptr : (const OT *)a.y + t * a.ldy;
    float sum = 0.f;
    for (int c = tid; c < W; c += 256) {
        float u = 0.f;
        if (MODE == ST_START) {
            const float v = ld_f(er, c);
            for (int s = 0; s < S; ++s) { xr[(int64_t)s * W + c] = v; u += a.win[s] * v; }
        } else {
            float y;
            if (a.place) {
                y = 0.f;
                for (int k = 0; k < a.top; ++k) {
                    const int64_t pl = a.place[t * a.top + k];
                    y += a.score[t * a.top + k] * (pl < 0 ? ld_f((const OT *)a.ident, t * a.ldi + c) : ld_f((const OT *)a.y, pl * a.ldy + c));
                }
            } else y = ld_f(yr, c);
            for (int s = 0; s < S; ++s) old[s * 256 + tid] = xr[(int64_t)s * W + c];
            for (int q = 0; q < S; ++q) {
                float v = a.wout[q] * y;
                for (int s = 0; s < S; ++s) v += a.mix[s * S + q] * old[s * 256 + tid];
                if (MODE == ST_STEP) { xr[(int64_t)q * W + c] = v; u += a.win[q] * v; } else u += v;
            }
        }
        us[c] = u; sum += u;
    }
    const float mean = block_sum(sum, red) / (float)W;
    float var = 0.f;
    for (int c = tid; c < W; c += 256) { const float d = us[c] - mean; var += d * d; }      // (a thread re-reads what it wrote)
    const float f = 1.0f / sqrtf(block_sum(var, red) / (float)W + a.eps);
    OT *o = (OT *)a.out + r * a.ldo;
    for (int c = tid; c < W; c += 256) st_f(o, c, (us[c] - mean) * f * a.w[c]);
}

// The step for 16-bit operands and widths that are multiples of 4: NT threads per row (64: a wave, four rows per workgroup, no barrier; 256: the workgroup), a row's
// streams, result and u in registers, 16-byte loads and stores of the streams.
// KIND: the start, a step, or a step whose y is the weighted sum of a token's chosen experts' rows.
enum { K_START = 0, K_STEP = 1, K_EXPERTS = 2 };
template <int S, int NT, int NV, int KIND>
__global__ __launch_bounds__(256) void stream_step4_kernel(StreamArgs a) {
    constexpr bool START = KIND == K_START;
    __shared__ float red[4];
    const int W = a.W, W4 = W >> 2, l = threadIdx.x & (NT - 1);
    const int64_t r = (int64_t)blockIdx.x * (256 / NT) + threadIdx.x / NT;
    if (NT == 64 && r >= a.T) return;                   // (a whole wave: nobody waits for it)
    const int64_t t = a.rows ? a.rows[r] : r;
    const bool fin = !START && a.sum;                   // (the end: u is the sum of the new streams, which stay where they were)
    float *xr = a.x + t * S * W;
    const bf16_t *yr = START ? (const bf16_t *)a.E + a.ids[t] * (int64_t)W : (const bf16_t *)a.y + t * a.ldy;      // (the start: every stream is this row)
    float4 xs[NV][START ? 1 : S], yf[NV]; uint2 ys[NV];
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c4 = l + k * NT;
        if (c4 < W4) {
#pragma unroll
            for (int s = 0; s < (START ? 0 : S); ++s) xs[k][s] = *reinterpret_cast<const float4 *>(xr + (int64_t)s * W + c4 * 4);
            if (KIND != K_EXPERTS) ys[k] = *reinterpret_cast<const uint2 *>(yr + c4 * 4);
        }
    }
    auto unpack = [](uint2 v) { return float4{__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16), __uint_as_float(v.y & 0xffff0000u)}; };
    if (KIND == K_EXPERTS) {                            // the choices' rows are requested four at a time
#pragma unroll
        for (int k = 0; k < NV; ++k) yf[k] = float4{0.f, 0.f, 0.f, 0.f};
        for (int j0 = 0; j0 < a.top; j0 += 4) {
            uint2 v[4][NV]; float sc[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int64_t i = t * a.top + min(j0 + j, a.top - 1), pl = a.place[i];
                sc[j] = a.score[i];
                const bf16_t *row = pl < 0 ? (const bf16_t *)a.ident + t * a.ldi : (const bf16_t *)a.y + pl * a.ldy;
#pragma unroll
                for (int k = 0; k < NV; ++k) if (l + k * NT < W4) v[j][k] = *reinterpret_cast<const uint2 *>(row + (l + k * NT) * 4);
            }
#pragma unroll
            for (int j = 0; j < 4; ++j)
                if (j0 + j < a.top)
#pragma unroll
                    for (int k = 0; k < NV; ++k) if (l + k * NT < W4) { const float4 e = unpack(v[j][k]); yf[k].x += sc[j] * e.x; yf[k].y += sc[j] * e.y; yf[k].z += sc[j] * e.z; yf[k].w += sc[j] * e.w; }
        }
    }
    float mix[S][S], wo[S], wi[S];
#pragma unroll
    for (int s = 0; s < S; ++s) {
        wo[s] = START ? 1.f : a.wout[s]; wi[s] = fin ? 1.f : a.win[s];
#pragma unroll
        for (int q = 0; q < S; ++q) mix[s][q] = START ? 0.f : a.mix[s * S + q];
    }
    float4 u[NV]; float sum = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c4 = l + k * NT;
        u[k] = float4{0.f, 0.f, 0.f, 0.f};
        if (c4 < W4) {
            if (KIND != K_EXPERTS) yf[k] = unpack(ys[k]);
#pragma unroll
            for (int q = 0; q < S; ++q) {
                float4 v{wo[q] * yf[k].x, wo[q] * yf[k].y, wo[q] * yf[k].z, wo[q] * yf[k].w};
#pragma unroll
                for (int s = 0; s < (START ? 0 : S); ++s) { v.x += mix[s][q] * xs[k][s].x; v.y += mix[s][q] * xs[k][s].y; v.z += mix[s][q] * xs[k][s].z; v.w += mix[s][q] * xs[k][s].w; }
                if (!fin) *reinterpret_cast<float4 *>(xr + (int64_t)q * W + c4 * 4) = v;
                u[k].x += wi[q] * v.x; u[k].y += wi[q] * v.y; u[k].z += wi[q] * v.z; u[k].w += wi[q] * v.w;
            }
            sum += (u[k].x + u[k].y) + (u[k].z + u[k].w);
        }
    }
    const float mean = (NT == 64 ? wave_sum(sum) : block_sum(sum, red)) / (float)W;
    float var = 0.f;
#pragma unroll
    for (int k = 0; k < NV; ++k)
        if (l + k * NT < W4) { const float a0 = u[k].x - mean, a1 = u[k].y - mean, a2 = u[k].z - mean, a3 = u[k].w - mean; var += (a0 * a0 + a1 * a1) + (a2 * a2 + a3 * a3); }
    const float f = 1.0f / sqrtf((NT == 64 ? wave_sum(var) : block_sum(var, red)) / (float)W + a.eps);
    bf16_t *o = (bf16_t *)a.out + r * a.ldo;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int c4 = l + k * NT;
        if (c4 < W4) {
            const float4 w = *reinterpret_cast<const float4 *>(a.w + c4 * 4);
            *reinterpret_cast<uint2 *>(o + c4 * 4) = uint2{pack2((u[k].x - mean) * f * w.x, (u[k].y - mean) * f * w.y), pack2((u[k].z - mean) * f * w.z, (u[k].w - mean) * f * w.w)};
        }
    }
}

// ------------------------------------------------------------------------------------------------ queries, keys and values on their way to the attention
// The numbers (a, b) of piece i of a head: a rotated pair while i < half, then what the rotation leaves, two at a time (b == D: absent, D odd).
__device__ __forceinline__ void piece_of(int i, int half, bool pairs, int &a, int &b) {
    if (i < half && !pairs) { a = i; b = i + half; } else { a = 2 * i; b = 2 * i + 1; }
}

// General form: one workgroup per row, a wave per head at a time.
template <class CT>
__global__ __launch_bounds__(256) void qkv_rope_kernel(QkvRopeArgs a, Batch b) {
    extern __shared__ float sm[];                       // [half] cosines, [half] sines
    const int t = blockIdx.x, sq = b.row_seq[t], lane = threadIdx.x & 63;
    const int p = b.start[sq] + (t - b.cu[sq]);
    const int blk = b.block_tables[(int64_t)sq * b.max_blocks + p / b.block_size], jj = p % b.block_size;
    const int64_t row = (int64_t)blk * b.block_size + jj;
    CT *pr = (CT *)a.proj + (int64_t)t * a.ld;
    const int D = a.D, half = a.rot / 2, np = (D + 1) / 2;
    float *cs = sm, *sn = sm + half;
    const float gain = a.gain == 0.f ? 1.f : a.gain;
    for (int i = threadIdx.x; i < half; i += 256) { const float ang = (float)p * a.freq[i]; cs[i] = gain * cosf(ang); sn[i] = gain * sinf(ang); }
    __syncthreads();
    for (int hd = threadIdx.x >> 6; hd < a.H + a.G; hd += 4) {
        const bool isq = hd < a.H;
        const int h = isq ? hd : hd - a.H;
        CT *src = pr + (isq ? a.qcol : a.kcol) + (int64_t)h * D;
        const float *bias = isq ? a.bq : a.bk, *wn = isq ? a.wq : a.wk;
        CT *dst = isq ? src : (CT *)a.kc + (row * a.G + h) * D;
        auto raw = [&](int c) { return c < D ? ld_f(src, c) + (bias ? bias[(int64_t)h * D + c] : 0.f) : 0.f; };
        float pre = 1.f;
        if (wn) {
            float ss = 0.f;
            for (int c = lane; c < D; c += 64) { const float v = raw(c); ss += v * v; }
            pre = 1.0f / sqrtf(wave_sum(ss) / (float)D + a.eps);
        }
        auto turned = [&](int i, int ca, int cb, float &u, float &v) {
            u = raw(ca); v = raw(cb);
            if (wn) { u *= pre * wn[ca]; v *= cb < D ? pre * wn[cb] : 0.f; }
            if (i < half) { const float c = cs[i], s = sn[i], u0 = u; u = u0 * c - v * s; v = v * c + u0 * s; }
        };
        float f = 1.f;
        if (a.unit) {
            float ss = 0.f;
            for (int i = lane; i < np; i += 64) { int ca, cb; piece_of(i, half, a.pairs, ca, cb); float u, v; turned(i, ca, cb, u, v); ss += u * u + v * v; }
            f = 1.0f / sqrtf(wave_sum(ss) / (float)D + a.eps);
        }
        for (int i = lane; i < np; i += 64) {           // (a lane reads its piece, then writes it)
            int ca, cb; piece_of(i, half, a.pairs, ca, cb);
            float u, v; turned(i, ca, cb, u, v);
            st_f(dst, ca, u * f); if (cb < D) st_f(dst, cb, v * f);
        }
    }
    const int GV = (a.Gv > 0 ? a.Gv : a.G) * a.Dv;
    CT *vc = (CT *)a.vc;
    const int64_t grp = ((int64_t)blk * (b.block_size >> 3) + (jj >> 3)) * GV;        // grouped value pages: [block][block_size / 8][G][Dv][8 keys]
    const float lam = a.v_first ? *a.lambda : 0.f;
    for (int c = threadIdx.x; c < GV; c += 256) {
        float v = ld_f(pr, a.vcol + c) + (a.bv ? a.bv[c] : 0.f);
        if (a.v_keep) st_f((CT *)a.v_keep, (int64_t)t * GV + c, v);
        if (a.v_first) v = (1.0f - lam) * v + lam * ld_f((const CT *)a.v_first, (int64_t)t * GV + c);
        if (a.v_grouped) st_f(vc, (grp + c) * 8 + (jj & 7), v); else st_f(vc, row * GV + c, v);
    }
}

// 16-bit rows, all parts multiples of 8 numbers: LP lanes with 8 numbers each per head (16-byte loads and stores, pairs inside a lane — with HALVES the partner's 8 numbers come
// from the lane half / 8 further —, the sums of squares by shuffles), 64 / LP heads per wave at a time; RB rows per workgroup (1: the four waves share a row's heads; 4: a wave per row), cosines and sines once per row.
template <int LP, int RB, bool HALVES>
__global__ __launch_bounds__(256) void qkv_rope8_kernel(QkvRopeArgs a, Batch b) {
    extern __shared__ float2 tab[];                     // [RB][half] (cosine, sine)
    constexpr int WR = 4 / RB, HW = 64 / LP;            // waves per row, heads per wave and pass
    const int half = a.rot / 2, r0 = blockIdx.x * RB;
    for (int idx = threadIdx.x; idx < RB * half; idx += 256) {
        const int rr = RB == 1 ? 0 : idx / half, i = idx - rr * half, t = r0 + rr;
        if (t < b.T) { const int sq = b.row_seq[t]; const float ang = (float)(b.start[sq] + (t - b.cu[sq])) * a.freq[i], gain = a.gain == 0.f ? 1.f : a.gain; tab[idx] = float2{gain * cosf(ang), gain * sinf(ang)}; }
    }
    __syncthreads();
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, rr = wave / WR, wv = wave % WR, t = r0 + rr;
    if (t >= b.T) return;
    const int sq = b.row_seq[t], p = b.start[sq] + (t - b.cu[sq]);
    const int blk = b.block_tables[(int64_t)sq * b.max_blocks + p / b.block_size], jj = p % b.block_size;
    const int64_t row = (int64_t)blk * b.block_size + jj;
    bf16_t *pr = (bf16_t *)a.proj + (int64_t)t * a.ld;
    const int D = a.D, l = lane & (LP - 1), sub = lane / LP;
    const float2 *ct = tab + rr * half;
    for (int hd0 = wv * HW; hd0 < a.H + a.G; hd0 += WR * HW) {          // (the bound is the wave's: every lane takes part in the shuffles)
        const int hd = hd0 + sub;
        const bool on = hd < a.H + a.G && l * 8 < D, isq = hd < a.H;
        const int h = isq ? hd : hd - a.H;
        float e[8] = {};
        float ss = 0.f;
        bf16_t *src = pr + (isq ? a.qcol : a.kcol) + (int64_t)h * D + l * 8;
        if (on) {
            const uint4 v = *reinterpret_cast<const uint4 *>(src); const bf16_t *ve = reinterpret_cast<const bf16_t *>(&v);
#pragma unroll
            for (int k = 0; k < 8; ++k) e[k] = ld_f(ve, k);
            const float *bias = isq ? a.bq : a.bk;
            if (bias) {
                const float4 b0 = *reinterpret_cast<const float4 *>(bias + (int64_t)h * D + l * 8), b1 = *reinterpret_cast<const float4 *>(bias + (int64_t)h * D + l * 8 + 4);
                e[0] += b0.x; e[1] += b0.y; e[2] += b0.z; e[3] += b0.w; e[4] += b1.x; e[5] += b1.y; e[6] += b1.z; e[7] += b1.w;
            }
        }
        const float *wn = isq ? a.wq : a.wk;
        if (a.wq || a.wk) {                                 // (every lane of the wave: q and k heads may share a pass)
            float sw = 0.f;
            if (on)
#pragma unroll
                for (int k = 0; k < 8; ++k) sw += e[k] * e[k];
#pragma unroll
            for (int o = LP / 2; o > 0; o >>= 1) sw += __shfl_xor(sw, o, 64);
            if (on && wn) {
                const float pre = 1.0f / sqrtf(sw / (float)D + a.eps);
                const float4 w0 = *reinterpret_cast<const float4 *>(wn + l * 8), w1 = *reinterpret_cast<const float4 *>(wn + l * 8 + 4);
                e[0] *= pre * w0.x; e[1] *= pre * w0.y; e[2] *= pre * w0.z; e[3] *= pre * w0.w; e[4] *= pre * w1.x; e[5] *= pre * w1.y; e[6] *= pre * w1.z; e[7] *= pre * w1.w;
            }
        }
        if (HALVES) {
            const int hl = half >> 3, i0 = l < hl ? l : l - hl;
            const bool turn = on && l < 2 * hl;
            const int other = (lane & ~(LP - 1)) + (l < 2 * hl ? (l < hl ? l + hl : l - hl) : l);
#pragma unroll
            for (int k = 0; k < 8; ++k) {
                const float v2 = __shfl(e[k], other, 64);
                if (turn) { const float2 q = ct[i0 * 8 + k]; e[k] = l < hl ? e[k] * q.x - v2 * q.y : e[k] * q.x + v2 * q.y; }
            }
            if (on)
#pragma unroll
                for (int k = 0; k < 8; ++k) ss += e[k] * e[k];
        } else if (on) {
#pragma unroll
            for (int k = 0; k < 4; ++k) {
                const int i = l * 4 + k;
                if (i < half) { const float2 q = ct[i]; const float u = e[2 * k], v2 = e[2 * k + 1]; e[2 * k] = u * q.x - v2 * q.y; e[2 * k + 1] = v2 * q.x + u * q.y; }
                ss += e[2 * k] * e[2 * k] + e[2 * k + 1] * e[2 * k + 1];
            }
        }
        float f = 1.f;
        if (a.unit) {
#pragma unroll
            for (int o = LP / 2; o > 0; o >>= 1) ss += __shfl_xor(ss, o, 64);
            f = 1.0f / sqrtf(ss / (float)D + a.eps);
        }
        if (on) {
            const uint4 o{pack2(e[0] * f, e[1] * f), pack2(e[2] * f, e[3] * f), pack2(e[4] * f, e[5] * f), pack2(e[6] * f, e[7] * f)};
            *reinterpret_cast<uint4 *>(isq ? src : (bf16_t *)a.kc + (row * a.G + h) * D + l * 8) = o;
        }
    }
    const int GV = (a.Gv > 0 ? a.Gv : a.G) * a.Dv;
    bf16_t *vc = (bf16_t *)a.vc;
    const int64_t grp = ((int64_t)blk * (b.block_size >> 3) + (jj >> 3)) * GV;
    const float lam = a.v_first ? *a.lambda : 0.f;
    for (int c = (wv * 64 + lane) * 8; c < GV; c += WR * 512) {
        uint4 v = *reinterpret_cast<const uint4 *>(pr + a.vcol + c); bf16_t *ve = reinterpret_cast<bf16_t *>(&v);
        float e[8];
#pragma unroll
        for (int k = 0; k < 8; ++k) e[k] = ld_f(ve, k);
        if (a.bv) {
            const float4 b0 = *reinterpret_cast<const float4 *>(a.bv + c), b1 = *reinterpret_cast<const float4 *>(a.bv + c + 4);
            e[0] += b0.x; e[1] += b0.y; e[2] += b0.z; e[3] += b0.w; e[4] += b1.x; e[5] += b1.y; e[6] += b1.z; e[7] += b1.w;
        }
        if (a.v_keep) *reinterpret_cast<uint4 *>((bf16_t *)a.v_keep + (int64_t)t * GV + c) = uint4{pack2(e[0], e[1]), pack2(e[2], e[3]), pack2(e[4], e[5]), pack2(e[6], e[7])};
        if (a.v_first) {
            const uint4 w = *reinterpret_cast<const uint4 *>((const bf16_t *)a.v_first + (int64_t)t * GV + c); const bf16_t *we = reinterpret_cast<const bf16_t *>(&w);
#pragma unroll
            for (int k = 0; k < 8; ++k) e[k] = (1.0f - lam) * e[k] + lam * ld_f(we, k);
        }
        v = uint4{pack2(e[0], e[1]), pack2(e[2], e[3]), pack2(e[4], e[5]), pack2(e[6], e[7])};
        if (!a.v_grouped) *reinterpret_cast<uint4 *>(vc + row * GV + c) = v;
        else
#pragma unroll
            for (int k = 0; k < 8; ++k) vc[(grp + c + k) * 8 + (jj & 7)] = ve[k];
    }
}

const size_t kMaxLds = 160 * 1024 - 2048;
bool aligned16(const void *p) { return ((uintptr_t)p & 15) == 0; }

template <int S, int KIND>
void step4(const StreamArgs &a, hipStream_t s) {
    const int W4 = a.W / 4;
    // many rows: a wave per row up to 1024 numbers; few rows: a workgroup per row
    if (a.T >= 1024 && W4 <= 256) {
        const dim3 grid((unsigned)((a.T + 3) / 4));
        if (W4 <= 64) stream_step4_kernel<S, 64, 1, KIND><<<grid, dim3(256), 0, s>>>(a);
        else if (W4 <= 128) stream_step4_kernel<S, 64, 2, KIND><<<grid, dim3(256), 0, s>>>(a);
        else stream_step4_kernel<S, 64, 4, KIND><<<grid, dim3(256), 0, s>>>(a);
        return;
    }
    const dim3 grid((unsigned)a.T);
    if (W4 <= 256) stream_step4_kernel<S, 256, 1, KIND><<<grid, dim3(256), 0, s>>>(a);
    else if (W4 <= 512) stream_step4_kernel<S, 256, 2, KIND><<<grid, dim3(256), 0, s>>>(a);
    else if (W4 <= 1024) stream_step4_kernel<S, 256, 4, KIND><<<grid, dim3(256), 0, s>>>(a);
    else stream_step4_kernel<S, 256, 8, KIND><<<grid, dim3(256), 0, s>>>(a);
}

template <int LP, bool HALVES>
void rope8(const QkvRopeArgs &a, const Batch &b, hipStream_t s) {
    const size_t lds = (size_t)std::max(a.rot / 2, 1) * sizeof(float2);
    if (b.T >= 1024) qkv_rope8_kernel<LP, 4, HALVES><<<dim3((unsigned)((b.T + 3) / 4)), dim3(256), 4 * lds, s>>>(a, b);
    else qkv_rope8_kernel<LP, 1, HALVES><<<dim3((unsigned)b.T), dim3(256), lds, s>>>(a, b);
}

}  // namespace

int prepare_streams() {
    const void *fns[] = {(const void *)stream_step_kernel<float, ST_START>, (const void *)stream_step_kernel<float, ST_STEP>, (const void *)stream_step_kernel<float, ST_SUM>,
                         (const void *)stream_step_kernel<bf16_t, ST_START>, (const void *)stream_step_kernel<bf16_t, ST_STEP>, (const void *)stream_step_kernel<bf16_t, ST_SUM>};
    for (const void *f : fns) NVR_HIP_CHECK(hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds));
    return 0;
}

int stream_step(const StreamArgs &a, bool bf16, hipStream_t s) {
    if (a.T == 0) return 0;
    const bool start = a.E != nullptr, sum = !start && a.sum;
    if (a.S < 1 || !a.out || !a.w || (start ? !a.ids || !a.win : !a.y || !a.mix || !a.wout || (!sum && !a.win)) || (a.rows && !sum) || (a.place && (start || a.top < 1 || !a.score || !a.ident)))
        return nvr::fail(NVR_ERR_INVALID_ARG, "stream_step: incomplete arguments (%d streams)", a.S);
    if (bf16 && a.S <= 4 && a.W % 4 == 0 && a.W <= 8192 && a.ldo % 4 == 0 && aligned16(a.x) && aligned16(a.out) && aligned16(a.w) && (start ? aligned16(a.E) : a.ldy % 4 == 0 && aligned16(a.y)) && (!a.place || (a.ldi % 4 == 0 && aligned16(a.ident)))) {
#define NVR_ST(S_) do { if (start) step4<S_, K_START>(a, s); else if (a.place) step4<S_, K_EXPERTS>(a, s); else step4<S_, K_STEP>(a, s); } while (0)
        if (a.S == 1) NVR_ST(1); else if (a.S == 2) NVR_ST(2); else if (a.S == 3) NVR_ST(3); else NVR_ST(4);
#undef NVR_ST
        return launched("stream_step");
    }
    const size_t lds = ((size_t)a.W + (start ? 0 : (size_t)a.S * 256)) * 4;
    if (lds > kMaxLds) return nvr::fail(NVR_ERR_UNSUPPORTED, "stream_step: %d streams of %d numbers do not fit LDS", a.S, a.W);
    const dim3 grid((unsigned)a.T), blk(256);
#define NVR_ST(M_) do { if (bf16) stream_step_kernel<bf16_t, M_><<<grid, blk, lds, s>>>(a); else stream_step_kernel<float, M_><<<grid, blk, lds, s>>>(a); } while (0)
    if (start) NVR_ST(ST_START); else if (sum) NVR_ST(ST_SUM); else NVR_ST(ST_STEP);
#undef NVR_ST
    return launched("stream_step");
}

int qkv_rope_store(const QkvRopeArgs &a, const Batch &b, bool bf16, hipStream_t s) {
    if (b.T == 0) return 0;
    if (a.rot % 2 || a.rot > a.D || a.rot < 0) return nvr::fail(NVR_ERR_INVALID_ARG, "qkv_rope_store: %d rotated coordinates of %d", a.rot, a.D);
    if (a.v_grouped && b.block_size % 8) return nvr::fail(NVR_ERR_INVALID_ARG, "qkv_rope_store: grouped value pages need pages of a multiple of 8 tokens");
    if (a.v_first && !a.lambda) return nvr::fail(NVR_ERR_INVALID_ARG, "qkv_rope_store: values to mix without their share");
    if ((size_t)a.rot * 4 > 60000) return nvr::fail(NVR_ERR_UNSUPPORTED, "qkv_rope_store: %d rotated coordinates", a.rot);
    const bool vec = bf16 && (a.pairs || a.rot % 16 == 0) && a.D % 8 == 0 && a.Dv % 8 == 0 && a.D <= 512 && a.ld % 8 == 0 && ((a.qcol | a.kcol | a.vcol) & 7) == 0 && a.rot <= 1024 &&
                     aligned16(a.proj) && aligned16(a.kc) && aligned16(a.vc) && aligned16(a.bq) && aligned16(a.bk) && aligned16(a.bv) && aligned16(a.v_first) && aligned16(a.v_keep) && aligned16(a.wq) && aligned16(a.wk);
    if (vec) {
#define NVR_ROPE8(LP_) do { if (a.pairs) rope8<LP_, false>(a, b, s); else rope8<LP_, true>(a, b, s); } while (0)
        if (a.D <= 32) NVR_ROPE8(4); else if (a.D <= 64) NVR_ROPE8(8); else if (a.D <= 128) NVR_ROPE8(16); else if (a.D <= 256) NVR_ROPE8(32); else NVR_ROPE8(64);
#undef NVR_ROPE8
        return launched("qkv_rope_store");
    }
    const size_t lds = (size_t)std::max(a.rot, 2) * 4;
    if (bf16) qkv_rope_kernel<bf16_t><<<dim3((unsigned)b.T), dim3(256), lds, s>>>(a, b);
    else qkv_rope_kernel<float><<<dim3((unsigned)b.T), dim3(256), lds, s>>>(a, b);
    return launched("qkv_rope_store");
}

}}  // namespace nvr::kl
