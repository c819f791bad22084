// layered_decode.hip — attention of decode-sized steps (one query position per sequence) of layer-list models (kernels/layered.h): few query rows per cached row, many keys.  A workgroup
// owns up to 16 query rows that meet the same key/value head (the heads of a group, the maps of differential attention, the heads on one latent row) and a share of the keys; its four waves
// walk the share in chunks of 32 keys each on their own, without a barrier: key fragments straight from the pages into registers, S^T = K Q^T with the query on the lane, online softmax with
// two cross-lane steps, the weights in registers as the B operand of O^T += V^T P^T, the values through a wave's own LDS image (row-major, read with the transposing ds_read_b64_tr_b16; where
// the values are the first numbers of the key rows, the key fragments are that image).  The four waves are merged in LDS, the shares by the workgroup that arrives last at the counter of its
// rows (write-through partials, nobody polls); the output of differential attention is formed there from both maps' rows.  wave64, gfx950, bfloat16 operands, f32 scores and sums.
#include <hip/hip_runtime.h>
#include <math.h>
#include <algorithm>
#include "../common.h"
#include "layered.h"

namespace nvr { namespace kl {

namespace {

typedef uint16_t bf16_t;
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x2 __attribute__((ext_vector_type(2)));
typedef unsigned int u32x4 __attribute__((ext_vector_type(4)));
typedef unsigned int u32x2 __attribute__((ext_vector_type(2)));
constexpr float kLog2e = 1.4426950408889634f;
constexpr float kNothing = -1e30f;                      // running maximum of a row that has seen no key (finite: differences stay finite)
constexpr int CH = 32;                                  // keys per chunk

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
    return v;
}
__device__ __forceinline__ bf16x4 read_tr(const char *p) { return __builtin_amdgcn_ds_read_tr16_b64_v4bf16((__attribute__((address_space(3))) bf16x4 *)p); }
// One build per size class C >= D, Dv, with no bound inside: a piece of a row past its end is read again from its last 16 bytes (the query's numbers there are zero, the output's are not stored).
constexpr int image_stride(int C) { return C * 2 + 32; }             // bytes; an odd multiple of 32: the 8 rows 32 lanes read together sit on different banks

// SHARED: the values are the first Dv numbers of the key rows.  bs_shift: log2 of the page size, or -1.  g: query rows per key/value head, in nrb groups of up to 16.  Grid: shares, groups, sequences.
template <int C, bool DIFF, bool SHARED>
__global__ __launch_bounds__(256, 1) void attn_decode_kernel(SinkAttnArgs a, Batch b, int bs_shift, int g, int nsplit, int nrb, float *__restrict__ part_o,
                                                             float *__restrict__ part_ml, unsigned int *__restrict__ tickets) {
    constexpr int NKS = C / 32, NDT = C / 16, VS = image_stride(C), OS = C + 4;
    extern __shared__ __attribute__((aligned(16))) char smem[];      // the waves' value images; behind the last chunk their outputs [4][16][OS] f32
    __shared__ float mls[4][16][2];
    __shared__ unsigned int ticket_s;
    const int z = blockIdx.x, grp = blockIdx.y, sq = blockIdx.z, pair = sq * gridDim.y + grp;
    const int kvh = nrb == 1 ? grp : grp / nrb, r0 = (grp - kvh * nrb) * 16, nr = min(16, g - r0);
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63, lm = lane & 15, lq = lane >> 4;
    const int pos = b.start[sq], ctx = pos + 1, D = a.D, Dv = a.Dv, bs = b.block_size;
    const int32_t *bt = b.block_tables + (int64_t)sq * b.max_blocks;
    const bf16_t *kc = (const bf16_t *)a.kc, *vc = (const bf16_t *)a.vc;
    char *img = smem + wave * CH * VS;
    const float scale2 = a.scale * kLog2e;

    bf16x8 qf[NKS];
    {
        const int r = r0 + min(lm, nr - 1), Dq = DIFF ? D >> 1 : D, d0 = DIFF ? (r & 1) * Dq : 0;
        const bf16_t *q = (const bf16_t *)a.q + (int64_t)sq * a.ldq + (int64_t)(kvh * g + r) * Dq + lq * 8 - d0;
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks) {
            const int d = ks * 32 + lq * 8;
            qf[ks] = bf16x8{};
            if (d >= d0 && d < d0 + Dq) qf[ks] = *reinterpret_cast<const bf16x8 *>(q + ks * 32);
        }
    }
    float m = kNothing, l = 0.f;
    if (a.sink && z == 0 && wave == 0) { m = a.sink[kvh * g + r0 + min(lm, nr - 1)] * kLog2e; l = lq == 0 ? 1.f : 0.f; }
    f32x4 o[NDT];
#pragma unroll
    for (int t = 0; t < NDT; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};

    // chunks: over the kept first keys, then from the window's first key (rounded down) on
    const int j0 = a.window > 0 ? max(0, ctx - a.window) / CH * CH : 0;
    const int kept = (a.window > 0 && a.keep_first > 0) ? min((a.keep_first + CH - 1) / CH, j0 / CH) : 0;
    const int nch = kept + (ctx - j0 + CH - 1) / CH;
    for (int x = z * 4 + wave; x < nch; x += nsplit * 4) {
        const int base = x < kept ? x * CH : j0 + (x - kept) * CH;
        bf16x8 kf[2][NKS], vf[2][NKS];
        int64_t row[2];
#pragma unroll
        for (int mt = 0; mt < 2; ++mt) {
            const int j = min(base + mt * 16 + lm, ctx - 1), pg = bs_shift >= 0 ? j >> bs_shift : j / bs;
            row[mt] = ((int64_t)bt[pg] * bs + (j - pg * bs)) * a.G + kvh;
        }
#pragma unroll
        for (int mt = 0; mt < 2; ++mt) {
            const bf16_t *kp = kc + row[mt] * D, *vp = vc + row[mt] * Dv;
#pragma unroll
            for (int ks = 0; ks < NKS; ++ks) kf[mt][ks] = *reinterpret_cast<const bf16x8 *>(kp + min(ks * 32 + lq * 8, D - 8));
            if constexpr (!SHARED)
#pragma unroll
                for (int ks = 0; ks < NKS; ++ks) vf[mt][ks] = *reinterpret_cast<const bf16x8 *>(vp + min(ks * 32 + lq * 8, Dv - 8));
        }
        f32x4 s[2];
#pragma unroll
        for (int mt = 0; mt < 2; ++mt) {
            s[mt] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int ks = 0; ks < NKS; ++ks) s[mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[mt][ks], qf[ks], s[mt], 0, 0, 0);
        }
#pragma unroll
        for (int mt = 0; mt < 2; ++mt)
#pragma unroll
            for (int ks = 0; ks < NKS; ++ks) {
                bf16x8 v;
                if constexpr (SHARED) v = kf[mt][ks]; else v = vf[mt][ks];
                *reinterpret_cast<bf16x8 *>(img + (mt * 16 + lm) * VS + (ks * 32 + lq * 8) * 2) = v;
            }
        // scores of query lm: keys base + mt * 16 + lq * 4 + e
        float mx = -INFINITY;
#pragma unroll
        for (int mt = 0; mt < 2; ++mt)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int j = base + mt * 16 + lq * 4 + e;
                const bool out = j > pos || (a.window > 0 && pos - j >= a.window && j >= a.keep_first);
                s[mt][e] = out ? -INFINITY : s[mt][e] * scale2;
                mx = fmaxf(mx, s[mt][e]);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16, 64)); mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
        const float mn = fmaxf(m, mx), alpha = __builtin_amdgcn_exp2f(m - mn);
        const bool moved = mn != m;
        m = mn;
        bf16x8 pf;
        float rs = 0.f;
#pragma unroll
        for (int mt = 0; mt < 2; ++mt)
#pragma unroll
            for (int e = 0; e < 4; ++e) { const float p = __builtin_amdgcn_exp2f(s[mt][e] - mn); rs += p; pf[mt * 4 + e] = (__bf16)p; }
        l = l * alpha + rs;
        if (__any(moved)) {
#pragma unroll
            for (int t = 0; t < NDT; ++t) o[t] *= alpha;
        }
        asm volatile("" ::: "memory");                  // (a wave's LDS requests are served in order: its image is written before it is read, and read before it is written again)
#pragma unroll
        for (int t = 0; t < NDT; ++t) {
            const char *p = img + (lq * 4 + (lm >> 2)) * VS + t * 32 + (lm & 3) * 8;
            const bf16x4 a0 = read_tr(p), a1 = read_tr(p + 16 * VS);
            bf16x8 v;
#pragma unroll
            for (int e = 0; e < 4; ++e) { v[e] = a0[e]; v[4 + e] = a1[e]; }
            o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v, pf, o[t], 0, 0, 0);
        }
        asm volatile("" ::: "memory");
    }
    l += __shfl_xor(l, 16, 64); l += __shfl_xor(l, 32, 64);
    if (lq == 0) { mls[wave][lm][0] = m; mls[wave][lm][1] = l; }
    __syncthreads();
    // the waves' outputs in one unit per row, then their sums
    float *om = (float *)smem;
    {
        const float mx = fmaxf(fmaxf(mls[0][lm][0], mls[1][lm][0]), fmaxf(mls[2][lm][0], mls[3][lm][0]));
        const float f = __builtin_amdgcn_exp2f(m - mx);
        if (lm < nr)
#pragma unroll
            for (int t = 0; t < NDT; ++t)
                *reinterpret_cast<f32x4 *>(om + (wave * 16 + lm) * OS + t * 16 + lq * 4) = o[t] * f;
    }
    __syncthreads();
    const int c4 = lane * 4;
    const bool on = c4 < Dv;
    auto own_ml = [&](int r) {                          // this workgroup's maximum and sum of row r
        const float mx = fmaxf(fmaxf(mls[0][r][0], mls[1][r][0]), fmaxf(mls[2][r][0], mls[3][r][0]));
        float s = 0.f;
#pragma unroll
        for (int w = 0; w < 4; ++w) s += mls[w][r][1] * __builtin_amdgcn_exp2f(mls[w][r][0] - mx);
        return f32x2{mx, s};
    };
    auto own_o = [&](int r) {
        f32x4 v{0.f, 0.f, 0.f, 0.f};
        if (on)
#pragma unroll
            for (int w = 0; w < 4; ++w) v += *reinterpret_cast<const f32x4 *>(om + (w * 16 + r) * OS + c4);
        return v;
    };
    // row r of the finished attention, four columns per lane
    const int64_t region = (int64_t)pair * nsplit * 16;
    auto rs_o = __builtin_amdgcn_make_buffer_rsrc((void *)(part_o + region * Dv), (short)0, nsplit * 16 * Dv * 4, 0x00020000);
    auto rs_ml = __builtin_amdgcn_make_buffer_rsrc((void *)(part_ml + region * 2), (short)0, nsplit * 16 * 2 * 4, 0x00020000);
    auto finished = [&](int r) {
        if (nsplit == 1) { const f32x2 ml = own_ml(r); return own_o(r) * (1.0f / ml[1]); }
        f32x2 ml{kNothing, 0.f};
        if (lane < nsplit) ml = __builtin_bit_cast(f32x2, __builtin_amdgcn_raw_buffer_load_b64(rs_ml, (lane * 16 + r) * 8, 0, 16));
        const float mx = wave_max(ml[0]);
        float wz = __builtin_amdgcn_exp2f(ml[0] - mx);
        wz /= wave_sum(ml[1] * wz);
        f32x4 v{0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
        for (int y = 0; y < nsplit; ++y) {
            const f32x4 p = __builtin_bit_cast(f32x4, __builtin_amdgcn_raw_buffer_load_b128(rs_o, ((y * 16 + r) * Dv + min(c4, Dv - 4)) * 4, 0, 16));
            v += p * __shfl(wz, y, 64);
        }
        return v;
    };
    if (nsplit > 1) {
        for (int r = wave; r < nr; r += 4) {
            const f32x4 v = own_o(r);
            if (on) __builtin_amdgcn_raw_buffer_store_b128(__builtin_bit_cast(u32x4, v), rs_o, ((z * 16 + r) * Dv + c4) * 4, 0, 16);
            const f32x2 ml = own_ml(r);
            if (lane == 0) __builtin_amdgcn_raw_buffer_store_b64(__builtin_bit_cast(u32x2, ml), rs_ml, (z * 16 + r) * 8, 0, 16);
        }
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");                      // every wave's partials have left ...
        __syncthreads();
        if (threadIdx.x == 0) ticket_s = __hip_atomic_fetch_add(tickets + pair, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);      // ... one ticket
        __syncthreads();
        if (ticket_s != (unsigned)(nsplit - 1)) return;                       // not the last share of these rows
        __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
        if (threadIdx.x == 0) __hip_atomic_store(tickets + pair, 0u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);                     // for the next launch
    }
    auto store4 = [&](int h, f32x4 v) {
        if (!on) return;
        const bf16x4 w{(__bf16)v[0], (__bf16)v[1], (__bf16)v[2], (__bf16)v[3]};
        *reinterpret_cast<bf16x4 *>((bf16_t *)a.out + (int64_t)sq * a.ldo + (int64_t)h * Dv + c4) = w;
    };
    if (DIFF) {
        const float lam = *a.lambda;
        for (int hh = wave; hh < nr / 2; hh += 4) {
            f32x4 d = finished(2 * hh) - lam * finished(2 * hh + 1);
            if (!on) d = f32x4{0.f, 0.f, 0.f, 0.f};
            const float ss = wave_sum((d[0] * d[0] + d[1] * d[1]) + (d[2] * d[2] + d[3] * d[3]));
            const int h = ((kvh * g + r0) >> 1) + hh;
            float f = a.out_scale / sqrtf(ss / (float)Dv + a.eps);
            if (a.head_gate) f /= 1.0f + expf(-__uint_as_float((uint32_t)((const bf16_t *)a.head_gate)[(int64_t)sq * a.ldhg + h] << 16));
            store4(h, d * f);
        }
    } else
        for (int r = wave; r < nr; r += 4) store4(kvh * g + r0 + r, finished(r));
}

const size_t kMaxLds = 160 * 1024 - 4096;

template <int C>
int launch(const SinkAttnArgs &a, const Batch &b, int nsplit, int nrb, float *po, float *pml, unsigned int *tickets, hipStream_t s) {
    const dim3 grid((unsigned)nsplit, (unsigned)(a.G * nrb), (unsigned)b.B), blk(256);
    const int g = a.H * (a.lambda ? 2 : 1) / a.G;
    const size_t lds = std::max((size_t)4 * CH * image_stride(C), (size_t)4 * 16 * (C + 4) * 4);
    const bool shared = a.vld != 0;
    const int bs_shift = (b.block_size & (b.block_size - 1)) == 0 ? __builtin_ctz((unsigned)b.block_size) : -1;
    if (a.lambda) attn_decode_kernel<C, true, false><<<grid, blk, lds, s>>>(a, b, bs_shift, g, nsplit, nrb, po, pml, tickets);
    else if (shared) attn_decode_kernel<C, false, true><<<grid, blk, lds, s>>>(a, b, bs_shift, g, nsplit, nrb, po, pml, tickets);
    else attn_decode_kernel<C, false, false><<<grid, blk, lds, s>>>(a, b, bs_shift, g, nsplit, nrb, po, pml, tickets);
    hipError_t e = hipGetLastError();
    if (e != hipSuccess) return nvr::fail(NVR_ERR_HIP, "attention_decode launch failed: %s", hipGetErrorString(e));
    return 0;
}

int row_blocks(const SinkAttnArgs &a) { return (a.H * (a.lambda ? 2 : 1) / a.G + 15) / 16; }

}  // namespace

int prepare_decode() {
    const void *fns[] = {(const void *)attn_decode_kernel<64, true, false>, (const void *)attn_decode_kernel<64, false, true>, (const void *)attn_decode_kernel<64, false, false>,
                         (const void *)attn_decode_kernel<128, true, false>, (const void *)attn_decode_kernel<128, false, true>, (const void *)attn_decode_kernel<128, false, false>,
                         (const void *)attn_decode_kernel<256, true, false>, (const void *)attn_decode_kernel<256, false, true>, (const void *)attn_decode_kernel<256, false, false>};
    for (const void *f : fns) NVR_HIP_CHECK(hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)kMaxLds));
    return 0;
}

bool attention_decode_ok(const SinkAttnArgs &a, bool bf16) {
    const bool shared = a.vld != 0;
    return bf16 && !a.r1 && !a.r2 && !a.slope && !a.pen && !a.gate_bias && a.softcap == 0.f && a.chunk == 0 && !(a.lambda && a.sink) && a.G >= 1 && a.H % a.G == 0 && a.D % 32 == 0 && a.Dv % 16 == 0 &&
           a.D <= 256 && a.Dv <= 256 && !(a.v_grouped && !shared) && (!shared || (a.vc == a.kc && a.vld == a.D && a.Dv <= a.D && a.G == 1 && !a.lambda)) && a.ldq % 8 == 0 && a.ldo % 4 == 0 &&
           (((uintptr_t)a.q | (uintptr_t)a.kc | (uintptr_t)a.vc) & 15) == 0 && ((uintptr_t)a.out & 7) == 0;
}

int attention_decode_groups(const SinkAttnArgs &a) { return a.G * row_blocks(a); }

int attention_decode(const SinkAttnArgs &a, const Batch &b, int max_splits, void *workspace, size_t workspace_bytes, unsigned int *tickets, int num_tickets, hipStream_t s) {
    if (b.B == 0) return 0;
    if (b.T != b.B || b.max_rows != 1) return nvr::fail(NVR_ERR_INVALID_ARG, "attention_decode: %d rows of %d sequences (one each)", b.T, b.B);
    if (!attention_decode_ok(a, true)) return nvr::fail(NVR_ERR_UNSUPPORTED, "attention_decode: shape outside the kernel");
    const int nrb = row_blocks(a);
    const int64_t pairs = (int64_t)b.B * a.G * nrb;
    if (b.B > 65535 || a.G * nrb > 65535) return nvr::fail(NVR_ERR_INVALID_ARG, "attention_decode: %d sequences of %d groups", b.B, a.G * nrb);
    const int keys = a.window > 0 ? std::min<int64_t>(b.max_ctx, (int64_t)a.window + std::max(a.keep_first, 0) + 2 * CH) : b.max_ctx;
    // shares of the keys: two chunks per wave (one, or three and more, measured slower), at most what the workspace and a wave's lanes hold
    const size_t per = 16 * (size_t)(a.Dv + 2) * 4;
    int64_t nsplit = std::min<int64_t>({(int64_t)max_splits, ((int64_t)keys + 8 * CH - 1) / (8 * CH), 64, (int64_t)(workspace_bytes / per / (size_t)pairs)});
    if (nsplit < 1) nsplit = 1;
    if (nsplit > 1 && pairs > num_tickets) return nvr::fail(NVR_ERR_INVALID_ARG, "attention_decode: %ld groups of rows, %d counters", (long)pairs, num_tickets);
    float *po = (float *)workspace, *pml = po + pairs * nsplit * 16 * a.Dv;
    const int C = std::max(a.D, a.Dv) <= 64 ? 64 : std::max(a.D, a.Dv) <= 128 ? 128 : 256;
    return C == 64 ? launch<64>(a, b, (int)nsplit, nrb, po, pml, tickets, s) : C == 128 ? launch<128>(a, b, (int)nsplit, nrb, po, pml, tickets, s) : launch<256>(a, b, (int)nsplit, nrb, po, pml, tickets, s);
}

}}  // namespace nvr::kl
