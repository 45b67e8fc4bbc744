// Skinny-M GEMM ("GEMV") for decode projections on MI355X:
//   out[M, N] = x[M, K] @ W[N, K]^T      (torch F.linear layout, bf16)
//
// Decode at small batch is weight-streaming-bound: each step reads every
// weight byte once. hipBLASLt's skinny kernels measure ~2.5x off the HBM
// roofline at M=1 (19.9us for a 50 MB qkv read, ~8us at 6.3 TB/s); this
// kernel follows the CDNA guide's GEMV row ("M <= 16 decode weights: operand
// streamed once per block, not shared across waves -> load straight to
// VGPRs, deep unroll, late vmcnt"): W rows stream through 16-B vector loads
// per lane, fp32 accumulate, one wave-reduction per (row, m). The activation
// x is tiny (8-56 KB) and L1-resident after the first pass — each lane
// re-reads only its own 16-B slices, so no LDS staging is needed.
//
// Requires K % 512 == 0 (64 lanes x 8 bf16); callers fall back to hipBLASLt
// otherwise (and for M > 8, where the MFMA path wins).

#include "common.h"
#include <algorithm>
#include <cstdlib>

typedef __attribute__((ext_vector_type(4))) unsigned int u32x4;

__device__ __forceinline__ u32x4 nt_load4(const uint32_t* p) {
    return __builtin_nontemporal_load(reinterpret_cast<const u32x4*>(p));
}


// fp32 rstd of x row m: one extra pass over the (L1-resident) activation
__device__ __forceinline__ float row_rstd(const uint32_t* xrow, int k2, int lane,
                                          float eps) {
    float ss = 0.0f;
    for (int i = lane * 4; i < k2; i += WAVE * 4) {
        uint4 xv = *reinterpret_cast<const uint4*>(xrow + i);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const float lo = bf16_lo((&xv.x)[j]), hi = bf16_hi((&xv.x)[j]);
            ss = fmaf(lo, lo, ss);
            ss = fmaf(hi, hi, ss);
        }
    }
    ss = wave_reduce_sum(ss);
    return rsqrtf(ss / (float)(k2 * 2) + eps);
}

// NORM: x is normalized on the fly (rstd prologue + norm-weight multiply) —
// the separate rmsnorm kernel and its output round-trip disappear.
// ADDRES: the epilogue adds a residual row — out = x @ W^T + residual, i.e.
// the new residual stream is produced directly by the projection.
template <int M, bool NORM, bool ADDRES, int RW = 2>
__global__ __launch_bounds__(256) void gemv_kernel(
    const uint32_t* __restrict__ x,  // [M, K/2]
    const uint32_t* __restrict__ w,  // [N, K/2]
    uint32_t* __restrict__ out,      // [M, N] bf16 (u16 scalar writes)
    const uint32_t* __restrict__ wn, // [K/2] rmsnorm weight (NORM only)
    const uint32_t* __restrict__ res,// [M, N] residual (ADDRES only)
    int N, int k2 /* K/2 */, float eps) {
    const int lane = threadIdx.x & (WAVE - 1);
    const int wid = threadIdx.x / WAVE;

    float rstd[M];
    if (NORM) {
#pragma unroll
        for (int m = 0; m < M; ++m) rstd[m] = row_rstd(x + (size_t)m * k2, k2, lane, eps);
    }

    // RW adjacent W rows per wave: multiplies the outstanding 16-B streams
    // per wave (the 1-row form measured 5.1 TB/s vs the 2-row gateup's 6.4)
    for (int row0 = (blockIdx.x * 4 + wid) * RW; row0 < N;
         row0 += gridDim.x * 4 * RW) {
        const uint32_t* wr[RW];
        bool live[RW];
#pragma unroll
        for (int rr_ = 0; rr_ < RW; ++rr_) {
            live[rr_] = row0 + rr_ < N;
            wr[rr_] = w + (size_t)(live[rr_] ? row0 + rr_ : row0) * k2;
        }
        float acc[RW][M];
#pragma unroll
        for (int rr_ = 0; rr_ < RW; ++rr_)
#pragma unroll
            for (int m = 0; m < M; ++m) acc[rr_][m] = 0.0f;
        for (int i = lane * 4; i < k2; i += WAVE * 4) {
            // stream W non-temporally: each byte is read exactly once per
            // step; keep L2 for the KV cache and activations
            u32x4 wv[RW];
#pragma unroll
            for (int rr_ = 0; rr_ < RW; ++rr_) wv[rr_] = nt_load4(wr[rr_] + i);
#pragma unroll
            for (int m = 0; m < M; ++m) {
                uint4 xv = *reinterpret_cast<const uint4*>(x + (size_t)m * k2 + i);
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    float xl = bf16_lo((&xv.x)[j]), xh = bf16_hi((&xv.x)[j]);
                    if (NORM) {
                        const uint32_t wnw = wn[i + j];
                        xl *= rstd[m] * bf16_lo(wnw);
                        xh *= rstd[m] * bf16_hi(wnw);
                    }
#pragma unroll
                    for (int rr_ = 0; rr_ < RW; ++rr_) {
                        acc[rr_][m] = fmaf(xl, bf16_lo(wv[rr_][j]), acc[rr_][m]);
                        acc[rr_][m] = fmaf(xh, bf16_hi(wv[rr_][j]), acc[rr_][m]);
                    }
                }
            }
        }
#pragma unroll
        for (int m = 0; m < M; ++m) {
#pragma unroll
            for (int rr_ = 0; rr_ < RW; ++rr_) {
                float v = wave_reduce_sum(acc[rr_][m]);
                if (lane == 0 && live[rr_]) {
                    if (ADDRES) {
                        v += bf16_to_f32(reinterpret_cast<const uint16_t*>(
                            res)[(size_t)m * N + row0 + rr_]);
                    }
                    reinterpret_cast<uint16_t*>(out)[(size_t)m * N + row0 + rr_] =
                        f32_to_bf16(v);
                }
            }
        }
    }
}

// gate activation of the fused gate-up kernels: 0 = silu, 1 = gelu in its tanh
// approximation, g/2 * (1 + tanh(k (g + 0.044715 g^3))), k = sqrt(2/pi)
__device__ __forceinline__ float gate_act(float g, int act) {
    if (act == 1) {
        const float t = tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g));
        return 0.5f * g * (1.0f + t);
    }
    return g / (1.0f + __expf(-g));
}

// Fused gate-up + SiLU GEMV for the MLP up-projection: the fused weight
// holds gate rows [0, I) and up rows [I, 2I); each wave computes BOTH rows
// r and I + r and writes act[m][r] = silu(gate) * up directly — the separate
// [1, 2I] intermediate and the silu_mul pass never materialize.
template <int M, bool NORM>
__global__ __launch_bounds__(256) void gemv_gateup_kernel(
    const uint32_t* __restrict__ x,  // [M, K/2]
    const uint32_t* __restrict__ w,  // [2I, K/2] (gate; up)
    uint32_t* __restrict__ out,      // [M, I] bf16
    const uint32_t* __restrict__ wn, // [K/2] rmsnorm weight (NORM only)
    int I, int k2, float eps, int act) {
    const int lane = threadIdx.x & (WAVE - 1);
    const int wid = threadIdx.x / WAVE;

    float rstd[M];
    if (NORM) {
#pragma unroll
        for (int m = 0; m < M; ++m) rstd[m] = row_rstd(x + (size_t)m * k2, k2, lane, eps);
    }

    for (int row = blockIdx.x * 4 + wid; row < I; row += gridDim.x * 4) {
        const uint32_t* grow = w + (size_t)row * k2;
        const uint32_t* urow = w + (size_t)(I + row) * k2;
        float accg[M], accu[M];
#pragma unroll
        for (int m = 0; m < M; ++m) accg[m] = accu[m] = 0.0f;
        for (int i = lane * 4; i < k2; i += WAVE * 4) {
            u32x4 gv = nt_load4(grow + i);
            u32x4 uv = nt_load4(urow + i);
#pragma unroll
            for (int m = 0; m < M; ++m) {
                uint4 xv = *reinterpret_cast<const uint4*>(x + (size_t)m * k2 + i);
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    float xl = bf16_lo((&xv.x)[j]), xh = bf16_hi((&xv.x)[j]);
                    if (NORM) {
                        const uint32_t wnw = wn[i + j];
                        xl *= rstd[m] * bf16_lo(wnw);
                        xh *= rstd[m] * bf16_hi(wnw);
                    }
                    accg[m] = fmaf(xl, bf16_lo(gv[j]), accg[m]);
                    accg[m] = fmaf(xh, bf16_hi(gv[j]), accg[m]);
                    accu[m] = fmaf(xl, bf16_lo(uv[j]), accu[m]);
                    accu[m] = fmaf(xh, bf16_hi(uv[j]), accu[m]);
                }
            }
        }
#pragma unroll
        for (int m = 0; m < M; ++m) {
            const float g = wave_reduce_sum(accg[m]);
            const float u = wave_reduce_sum(accu[m]);
            if (lane == 0) {
                const float a = gate_act(g, act) * u;
                reinterpret_cast<uint16_t*>(out)[(size_t)m * I + row] = f32_to_bf16(a);
            }
        }
    }
}

static bool gemv_bf16_use_mfma(int M, int K, int gateup);
extern "C" int oa_gemv_bf16_mfma(void* stream, const void* x, const void* w,
                                 void* out, const void* wn, const void* res,
                                 int M, int N, int K, float eps, int mode,
                                 int gateup);

static int gemv_gateup_impl(void* stream, const void* x, const void* w,
                            void* out, const void* wn, int M, int I, int K,
                            float eps, int norm, int act) {
    if (K % 8 != 0) return -100;
    if (gemv_bf16_use_mfma(M, K, 1))
        return oa_gemv_bf16_mfma(stream, x, w, out, wn, nullptr, M, 2 * I, K,
                                 eps, norm ? 1 : 0, 1 + act);
    const int k2 = K / 2;
    const int grid = min(2048, CEIL_DIV(I, 4));
#define LAUNCH_GU(MV)                                                          \
    do {                                                                       \
        if (norm)                                                              \
            hipLaunchKernelGGL((gemv_gateup_kernel<MV, true>), dim3(grid),     \
                               dim3(256), 0, (hipStream_t)stream,              \
                               (const uint32_t*)x, (const uint32_t*)w,         \
                               (uint32_t*)out, (const uint32_t*)wn, I, k2, eps, act);\
        else                                                                   \
            hipLaunchKernelGGL((gemv_gateup_kernel<MV, false>), dim3(grid),    \
                               dim3(256), 0, (hipStream_t)stream,              \
                               (const uint32_t*)x, (const uint32_t*)w,         \
                               (uint32_t*)out, (const uint32_t*)wn, I, k2, eps, act);\
    } while (0)
    switch (M) {
        case 1: LAUNCH_GU(1); break;
        case 2: LAUNCH_GU(2); break;
        case 3: LAUNCH_GU(3); break;
        case 4: LAUNCH_GU(4); break;
        case 5: LAUNCH_GU(5); break;
        case 6: LAUNCH_GU(6); break;
        case 7: LAUNCH_GU(7); break;
        case 8: LAUNCH_GU(8); break;
        case 12: LAUNCH_GU(12); break;
        case 16: LAUNCH_GU(16); break;
        default: return -101;
    }
#undef LAUNCH_GU
    HIP_CHECK_LAUNCH();
    return 0;
}

extern "C" int oa_gemv_gateup_ex(void* stream, const void* x, const void* w,
                                 void* out, const void* wn, int M, int I, int K,
                                 float eps, int norm) {
    return gemv_gateup_impl(stream, x, w, out, wn, M, I, K, eps, norm, 0);
}

extern "C" int oa_gemv_gateup(void* stream, const void* x, const void* w,
                              void* out, int M, int I, int K) {
    return gemv_gateup_impl(stream, x, w, out, nullptr, M, I, K, 0.0f, 0, 0);
}

// act: 0 silu, 1 gelu (tanh form)
extern "C" int oa_gemv_gateup_act(void* stream, const void* x, const void* w,
                                  void* out, int M, int I, int K, int act) {
    if (act < 0 || act > 1) return -105;
    return gemv_gateup_impl(stream, x, w, out, nullptr, M, I, K, 0.0f, 0, act);
}

// mode: 0 plain, 1 norm-prologue, 2 residual-add epilogue, 3 both
extern "C" int oa_gemv_ex(void* stream, const void* x, const void* w, void* out,
                          const void* wn, const void* res, int M, int N, int K,
                          float eps, int mode) {
    if (K % 8 != 0) return -100;
    if (gemv_bf16_use_mfma(M, K, 0))
        return oa_gemv_bf16_mfma(stream, x, w, out, wn, res, M, N, K, eps,
                                 mode, 0);
    const int k2 = K / 2;
    // 4 rows/wave won +3-6% in the ISOLATED probe on wide outputs
    // (scripts/gemv_ab.py) but lost 3% in-model (decode step 3.63 -> 3.75 ms,
    // within-box A/B) — real decode interleaves the W stream with KV/L2
    // traffic the probe does not. Default OFF; OPSAGENT_GEMV_RW4_MIN_N
    // re-enables for experiments.
    static int rw4_min_n = -1;
    static int rw1_max_n = -1;
    if (rw4_min_n < 0) {
        const char* e = getenv("OPSAGENT_GEMV_RW4_MIN_N");
        rw4_min_n = e ? atoi(e) : (1 << 30);
        // RW=1 for small-N outputs: at N=4096 the RW=2 grid is only 512
        // workgroups (2 per CU — half the SIMD slots idle); one row per wave
        // doubles the wave count and the streams in flight. In-model A/B
        // (8B turn, same box): off 438.1 ms, N<=6144 431.0 ms, N<=4096
        // 431.9 ms — default N<=6144 (covers o_proj and the fused-norm qkv).
        const char* e1 = getenv("OPSAGENT_GEMV_RW1_MAX_N");
        rw1_max_n = e1 ? atoi(e1) : 6144;
    }
    const bool rw4 = N >= rw4_min_n;
    const bool rw1 = !rw4 && N <= rw1_max_n;
    const int grid = min(2048, CEIL_DIV(N, rw4 ? 16 : (rw1 ? 4 : 8)));
#define LAUNCH_NM(MV, NORMV, RESV)                                            \
    do {                                                                       \
        if (rw4)                                                               \
            hipLaunchKernelGGL((gemv_kernel<MV, NORMV, RESV, 4>), dim3(grid),  \
                               dim3(256), 0, (hipStream_t)stream,              \
                               (const uint32_t*)x, (const uint32_t*)w,         \
                               (uint32_t*)out, (const uint32_t*)wn,            \
                               (const uint32_t*)res, N, k2, eps);              \
        else if (rw1)                                                          \
            hipLaunchKernelGGL((gemv_kernel<MV, NORMV, RESV, 1>), dim3(grid),  \
                               dim3(256), 0, (hipStream_t)stream,              \
                               (const uint32_t*)x, (const uint32_t*)w,         \
                               (uint32_t*)out, (const uint32_t*)wn,            \
                               (const uint32_t*)res, N, k2, eps);              \
        else                                                                   \
            hipLaunchKernelGGL((gemv_kernel<MV, NORMV, RESV, 2>), dim3(grid),  \
                               dim3(256), 0, (hipStream_t)stream,              \
                               (const uint32_t*)x, (const uint32_t*)w,         \
                               (uint32_t*)out, (const uint32_t*)wn,            \
                               (const uint32_t*)res, N, k2, eps);              \
    } while (0)
#define LAUNCH_MODE(MV)                                                        \
    do {                                                                       \
        switch (mode) {                                                        \
            case 0: LAUNCH_NM(MV, false, false); break;                        \
            case 1: LAUNCH_NM(MV, true, false); break;                         \
            case 2: LAUNCH_NM(MV, false, true); break;                         \
            case 3: LAUNCH_NM(MV, true, true); break;                          \
            default: return -102;                                              \
        }                                                                      \
    } while (0)
    switch (M) {
        case 1: LAUNCH_MODE(1); break;
        case 2: LAUNCH_MODE(2); break;
        case 3: LAUNCH_MODE(3); break;
        case 4: LAUNCH_MODE(4); break;
        case 5: LAUNCH_MODE(5); break;
        case 6: LAUNCH_MODE(6); break;
        case 7: LAUNCH_MODE(7); break;
        case 8: LAUNCH_MODE(8); break;
        case 12: LAUNCH_MODE(12); break;
        case 16: LAUNCH_MODE(16); break;
        default: return -101;
    }
#undef LAUNCH_MODE
#undef LAUNCH_NM
    HIP_CHECK_LAUNCH();
    return 0;
}

extern "C" int oa_gemv(void* stream, const void* x, const void* w, void* out,
                       int M, int N, int K) {
    return oa_gemv_ex(stream, x, w, out, nullptr, nullptr, M, N, K, 0.0f, 0);
}

// RW=4 probe variant (within-probe A/B only — guide rule 24)
extern "C" int oa_gemv_rw4(void* stream, const void* x, const void* w, void* out,
                           int M, int N, int K) {
    if (K % 8 != 0) return -100;
    const int k2 = K / 2;
    const int grid = min(2048, CEIL_DIV(N, 16));
    switch (M) {
        case 1:
            hipLaunchKernelGGL((gemv_kernel<1, false, false, 4>), dim3(grid),
                               dim3(256), 0, (hipStream_t)stream,
                               (const uint32_t*)x, (const uint32_t*)w,
                               (uint32_t*)out, nullptr, nullptr, N, k2, 0.0f);
            break;
        default:
            return -101;
    }
    HIP_CHECK_LAUNCH();
    return 0;
}

// ---- MFMA bf16 GEMV (batched decode, M 2..16) ------------------------------
// The VALU kernels win at M <= 2 but their per-element M-loop turns
// compute-bound as the batch grows, and hipBLASLt's skinny kernels (the old
// M > 2 fallback) run ~2.5x off the stream roofline — concurrent decode
// (c=8/16) measured ~2 TB/s effective. Same architecture as the fp8 MFMA
// GEMV (fp8_moe.hip): x staged ONCE into LDS (norm applied in fp32 at stage
// time), each of the block's four waves streams 16 W rows over a quarter of
// K straight into v_mfma_f32_16x16x32_bf16 A-fragments with a PF-deep
// register prefetch ring, partial D tiles meet in LDS. The 16 B columns
// carry the batch — M up to 16 rides one weight stream.
typedef __attribute__((ext_vector_type(8))) short bf16x8g;
typedef __attribute__((ext_vector_type(4))) float f32x4g;

template <bool NORM, bool ADDRES, bool GATEUP>
__global__ __launch_bounds__(256, 1) void gemv_bf16_mfma_kernel(
    const uint32_t* __restrict__ x,   // [M, K/2] bf16x2
    const uint32_t* __restrict__ w,   // [N, K/2] (gateup: [2I, K/2])
    uint32_t* __restrict__ out,       // [M, N] bf16 (gateup: [M, I])
    const uint32_t* __restrict__ wn,  // [K/2] rmsnorm weight (NORM)
    const uint32_t* __restrict__ res, // [M, N] residual (ADDRES)
    int M, int N, int K, float eps, int act) {
    constexpr int PF = GATEUP ? 4 : 8;
    const int tid = threadIdx.x;
    const int lane = tid & (WAVE - 1);
    const int wid = tid / WAVE;
    const int fr = lane & 15;   // A row / B,D col
    const int fs = lane >> 4;   // 8-element k-slice; D rows fs*4..+3
    const int rows = GATEUP ? N / 2 : N;
    const int I = rows;
    const int row0 = blockIdx.x * 16;
    const int wrow = min(row0 + fr, rows - 1);
    const int k2 = K / 2;

    extern __shared__ __attribute__((aligned(16))) char xls[];
    const int pitch = K * 2 + 16;  // bytes; pad de-banks the batch rows

    // stage x (wave w handles batch rows m ≡ w mod 4), norm folded in fp32
    for (int m = wid; m < M; m += 4) {
        const uint32_t* xr = x + (size_t)m * k2;
        uint32_t* dst = reinterpret_cast<uint32_t*>(xls + (size_t)m * pitch);
        float rstd = 1.0f;
        if (NORM) rstd = row_rstd(xr, k2, lane, eps);
        for (int i = lane * 4; i < k2; i += WAVE * 4) {
            uint4 v = *reinterpret_cast<const uint4*>(xr + i);
            if (NORM) {
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const uint32_t g = wn[i + j];
                    const float lo = bf16_lo((&v.x)[j]) * rstd * bf16_lo(g);
                    const float hi = bf16_hi((&v.x)[j]) * rstd * bf16_hi(g);
                    (&v.x)[j] = (uint32_t)f32_to_bf16(lo) |
                                ((uint32_t)f32_to_bf16(hi) << 16);
                }
            }
            *reinterpret_cast<uint4*>(dst + i) = v;
        }
    }
    __syncthreads();

    const int ke = K / 4;               // elements per wave
    const int k0b = wid * ke * 2;       // byte offset of this wave's range
    const int nk = ke / 32;             // 32-element MFMA steps
    const char* wp = reinterpret_cast<const char*>(w);
    const uint32_t* wr0 = reinterpret_cast<const uint32_t*>(
        wp + (size_t)wrow * K * 2 + k0b) + fs * 4;
    const uint32_t* wr1 = reinterpret_cast<const uint32_t*>(
        wp + (size_t)(wrow + (GATEUP ? I : 0)) * K * 2 + k0b) + fs * 4;
    const int mrow = fr < M ? fr : 0;
    const char* xrw = xls + (size_t)mrow * pitch + k0b + fs * 16;

    f32x4g acc0 = {}, acc1 = {};
    uint4 abuf[PF], ubuf[GATEUP ? PF : 1];
    auto load_a = [&](int p, int kb) {
        u32x4 t = nt_load4(wr0 + kb * 16);
        abuf[p] = *reinterpret_cast<uint4*>(&t);
        if (GATEUP) {
            u32x4 t2 = nt_load4(wr1 + kb * 16);
            ubuf[p] = *reinterpret_cast<uint4*>(&t2);
        }
    };
#pragma unroll
    for (int p = 0; p < PF; ++p) load_a(p, p);
    // x fragment double-buffered ONE step ahead: an inline ds_read feeding
    // its own MFMA serializes on lgkmcnt(0) every step (measured in the .s)
    uint4 bcur = *reinterpret_cast<const uint4*>(xrw);
    for (int kb0 = 0; kb0 < nk; kb0 += PF) {
        const bool more = kb0 + PF < nk;
#pragma unroll
        for (int p = 0; p < PF; ++p) {
            const int kb = kb0 + p;
            uint4 bnext;
            if (kb + 1 < nk)
                bnext = *reinterpret_cast<const uint4*>(xrw + (kb + 1) * 64);
            acc0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                *reinterpret_cast<bf16x8g*>(&abuf[p]),
                *reinterpret_cast<bf16x8g*>(&bcur), acc0, 0, 0, 0);
            if (GATEUP)
                acc1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                    *reinterpret_cast<bf16x8g*>(&ubuf[p]),
                    *reinterpret_cast<bf16x8g*>(&bcur), acc1, 0, 0, 0);
            if (more) load_a(p, kb0 + PF + p);
            if (kb + 1 < nk) bcur = bnext;
        }
    }

    // intra-block reduction: [wave][plane][col fr][row fs*4+i] f32 in LDS
    __syncthreads();  // x reads done before the tiles overwrite the image
    float* red = reinterpret_cast<float*>(xls);
    const int planes = GATEUP ? 2 : 1;
    {
        float* t = red + ((wid * planes) * 16 + fr) * 16 + fs * 4;
        *reinterpret_cast<f32x4g*>(t) = acc0;
        if (GATEUP) *reinterpret_cast<f32x4g*>(t + 16 * 16) = acc1;
    }
    __syncthreads();
    if (wid != 0 || fr >= M) return;
    const int m = fr;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int row = row0 + fs * 4 + i;
        if (row >= rows) continue;
        float sg = 0.0f, su = 0.0f;
#pragma unroll
        for (int wv = 0; wv < 4; ++wv) {
            sg += red[((wv * planes) * 16 + m) * 16 + fs * 4 + i];
            if (GATEUP)
                su += red[((wv * planes + 1) * 16 + m) * 16 + fs * 4 + i];
        }
        float v;
        if (GATEUP) {
            v = gate_act(sg, act) * su;
        } else {
            v = sg;
            if (ADDRES)
                v += bf16_to_f32(reinterpret_cast<const uint16_t*>(
                    res)[(size_t)m * rows + row]);
        }
        reinterpret_cast<uint16_t*>(out)[(size_t)m * rows + row] =
            f32_to_bf16(v);
    }
}

// eligibility shared by the C dispatch and its callers; must mirror the
// kernel's constraints so ineligible shapes FALL BACK, never error
static bool gemv_bf16_use_mfma(int M, int K, int gateup) {
    const char* e = getenv("OPSAGENT_BF16_GEMV_MFMA");
    if (e && e[0] == '0') return false;
    int min_m = 3;  // VALU kernels keep the measured M<=2 regime
    if (e && e[0] == 'm') min_m = atoi(e + 1);
    if (M < min_m || M > 16) return false;
    if (K % (gateup ? 512 : 1024) != 0) return false;
    // A/B-measured win region (scripts/gemv_bf16_mfma_ab.py): +29..+83%
    // at the 8B-class K<=6144 shapes; hipBLASLt keeps deep-K (70B qkv
    // K=8192 5.56 TB/s vs 3.21; 8B down K=14336 a wash) and the M=16
    // gateup (131 KiB x-image halves block occupancy). Env 'm<N>' widens
    // for experiments.
    if (!(e && e[0] == 'm')) {
        // engine A/B at c16 (same box): the M 9..16 forms LOSE ~7% end to
        // end even though the M16 microbench won — cap at the regime both
        // agree on (M <= 8, K <= 6144)
        if (K > 6144 || M > 8) return false;
    }
    const size_t img = (size_t)M * (K * 2 + 16);
    return img <= 147456;
}

extern "C" int oa_gemv_bf16_mfma(void* stream, const void* x, const void* w,
                                 void* out, const void* wn, const void* res,
                                 int M, int N, int K, float eps, int mode,
                                 int gateup) {
    const int rows = gateup ? N / 2 : N;
    const size_t img = (size_t)M * (K * 2 + 16);
    const size_t red = (size_t)(gateup ? 2 : 1) * 4 * 16 * 16 * 4;
    const size_t shmem = img > red ? img : red;
    dim3 grid(CEIL_DIV(rows, 16)), block(256);
#define LAUNCH_BMF(NORMV, RESV, GUV)                                           \
    hipLaunchKernelGGL((gemv_bf16_mfma_kernel<NORMV, RESV, GUV>), grid, block, \
                       shmem, (hipStream_t)stream, (const uint32_t*)x,         \
                       (const uint32_t*)w, (uint32_t*)out,                     \
                       (const uint32_t*)wn, (const uint32_t*)res, M, N, K, eps, \
                       gateup > 1 ? gateup - 1 : 0)
    if (gateup) {
        if (mode & 1) LAUNCH_BMF(true, false, true);
        else LAUNCH_BMF(false, false, true);
    } else {
        switch (mode) {
            case 0: LAUNCH_BMF(false, false, false); break;
            case 1: LAUNCH_BMF(true, false, false); break;
            case 2: LAUNCH_BMF(false, true, false); break;
            case 3: LAUNCH_BMF(true, true, false); break;
            default: return -102;
        }
    }
#undef LAUNCH_BMF
    HIP_CHECK_LAUNCH();
    return 0;
}

// ---- grouped rows -----------------------------------------------------------
// One launch for all projections of a layer that read the same normed input or
// per-projection variants of it: the weight's rows [N, K] are cut into groups,
// group g = rows [begin, end), reads activation plane `plane` of x [P, M, K]
// and writes act(row . x) to column row - begin of its own output rows.
// begin and end are multiples of 16, so neither the two adjacent rows of a
// wave nor the 16 rows of a matrix-core tile straddle a group. In a paired group
// gate and up rows alternate and (row - begin) / 2 takes act(gate) * up.
#define GEMV_MAX_GROUPS 8
struct GemvGroups {
    int n;
    int end[GEMV_MAX_GROUPS];
    int plane[GEMV_MAX_GROUPS];
    int act[GEMV_MAX_GROUPS];         // 0 none, 1 silu, 2 gelu (tanh form); + 4: paired
    uint16_t* out[GEMV_MAX_GROUPS];
    int64_t os[GEMV_MAX_GROUPS];      // elements between the output rows
};

__device__ __forceinline__ int gemv_group_of(const GemvGroups& g, int row) {
    int k = 0;
    while (k + 1 < g.n && row >= g.end[k]) ++k;
    return k;
}
__device__ __forceinline__ float gemv_group_act(float v, int act) {
    return act ? gate_act(v, act - 1) : v;
}
#define GEMV_PAIRED 4

template <int M, int RW>
__global__ __launch_bounds__(256) void gemv_grouped_kernel(const uint32_t* __restrict__ x,
                                                           const uint32_t* __restrict__ w,
                                                           GemvGroups gr, int N, int k2) {
    const int lane = threadIdx.x & (WAVE - 1);
    const int wid = __builtin_amdgcn_readfirstlane(threadIdx.x / WAVE);
    for (int row0 = (blockIdx.x * 4 + wid) * RW; row0 < N; row0 += gridDim.x * 4 * RW) {
        const int gi = gemv_group_of(gr, row0);
        const uint32_t* xg = x + (size_t)gr.plane[gi] * M * k2;
        const uint32_t* wr = w + (size_t)row0 * k2;
        float acc[RW][M];
#pragma unroll
        for (int r = 0; r < RW; ++r)
#pragma unroll
            for (int m = 0; m < M; ++m) acc[r][m] = 0.0f;
        for (int i = lane * 4; i < k2; i += WAVE * 4) {
            u32x4 wv[RW];
#pragma unroll
            for (int r = 0; r < RW; ++r) wv[r] = nt_load4(wr + (size_t)r * k2 + i);
#pragma unroll
            for (int m = 0; m < M; ++m) {
                const uint4 xv = *reinterpret_cast<const uint4*>(xg + (size_t)m * k2 + i);
                const uint32_t xs[4] = {xv.x, xv.y, xv.z, xv.w};
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const float xl = bf16_lo(xs[j]), xh = bf16_hi(xs[j]);
#pragma unroll
                    for (int r = 0; r < RW; ++r) {
                        acc[r][m] = fmaf(xl, bf16_lo(wv[r][j]), acc[r][m]);
                        acc[r][m] = fmaf(xh, bf16_hi(wv[r][j]), acc[r][m]);
                    }
                }
            }
        }
        const int c0 = row0 - (gi ? gr.end[gi - 1] : 0);
        uint16_t* out = gr.out[gi];
        if (RW == 2 && (gr.act[gi] & GEMV_PAIRED)) {
#pragma unroll
            for (int m = 0; m < M; ++m) {
                const float g = wave_reduce_sum(acc[0][m]), u = wave_reduce_sum(acc[RW - 1][m]);
                if (lane == 0)
                    out[(size_t)m * gr.os[gi] + c0 / 2] =
                        f32_to_bf16(gemv_group_act(g, gr.act[gi] - GEMV_PAIRED) * u);
            }
            continue;
        }
#pragma unroll
        for (int m = 0; m < M; ++m)
#pragma unroll
            for (int r = 0; r < RW; ++r) {
                const float v = wave_reduce_sum(acc[r][m]);
                if (lane == 0)
                    out[(size_t)m * gr.os[gi] + c0 + r] = f32_to_bf16(gemv_group_act(v, gr.act[gi]));
            }
    }
}

// The matrix-core form: see gemv_bf16_mfma_kernel for the tiling. SPLIT: one
// group, K cut into pieces of `unit` columns over gridDim.y blocks; a block
// writes its float32 partial sums to part [gridDim.y, M, N], and the kernel
// that reads the product adds the pieces up. A deep K thereby fits the LDS
// image of the activations and fills the chip.
template <bool SPLIT>
__global__ __launch_bounds__(256, 1) void gemv_grouped_mfma_kernel(
    const uint32_t* __restrict__ x, const uint32_t* __restrict__ w, GemvGroups gr, int M, int K,
    int unit, float* __restrict__ part) {
    constexpr int PF = 8;
    const int tid = threadIdx.x;
    const int lane = tid & (WAVE - 1);
    const int wid = tid / WAVE;
    const int fr = lane & 15, fs = lane >> 4;
    const int row0 = blockIdx.x * 16;
    const int gi = SPLIT ? 0 : gemv_group_of(gr, row0);
    const int k2 = K / 2;
    const int kb_ = SPLIT ? blockIdx.y * unit : 0;       // first column of this block
    const int kl = SPLIT ? min(unit, K - kb_) : K;       // its columns, a multiple of 1024
    extern __shared__ __attribute__((aligned(16))) char xls[];
    const int pitch = kl * 2 + 16;
    const uint32_t* xg = x + (size_t)(SPLIT ? 0 : gr.plane[gi]) * M * k2 + kb_ / 2;
    const int ke = kl / 4;
    const int k0b = wid * ke * 2;
    const int nk = ke / 32;             // a multiple of PF
    const uint32_t* wr = reinterpret_cast<const uint32_t*>(
        reinterpret_cast<const char*>(w) + ((size_t)(row0 + fr) * K + kb_) * 2 + k0b) + fs * 4;
    u32x4 abuf[PF];
#pragma unroll
    for (int p = 0; p < PF; ++p) abuf[p] = nt_load4(wr + p * 16);
    for (int m = wid; m < M; m += 4) {
        const uint32_t* xr = xg + (size_t)m * k2;
        uint32_t* dst = reinterpret_cast<uint32_t*>(xls + (size_t)m * pitch);
        for (int i = lane * 4; i < kl / 2; i += WAVE * 4)
            *reinterpret_cast<uint4*>(dst + i) = *reinterpret_cast<const uint4*>(xr + i);
    }
    __syncthreads();
    const char* xrw = xls + (size_t)(fr < M ? fr : 0) * pitch + k0b + fs * 16;
    f32x4g acc = {};
    uint4 bcur = *reinterpret_cast<const uint4*>(xrw);
    for (int kb0 = 0; kb0 < nk; kb0 += PF) {
        const bool more = kb0 + PF < nk;
#pragma unroll
        for (int p = 0; p < PF; ++p) {
            const int kb = kb0 + p;
            uint4 bnext = bcur;
            if (kb + 1 < nk) bnext = *reinterpret_cast<const uint4*>(xrw + (kb + 1) * 64);
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<bf16x8g*>(&abuf[p]),
                                                          *reinterpret_cast<bf16x8g*>(&bcur), acc, 0, 0, 0);
            if (more) abuf[p] = nt_load4(wr + (kb0 + PF + p) * 16);
            bcur = bnext;
        }
    }
    __syncthreads();   // x reads done before the partial tiles overwrite the image
    float* red = reinterpret_cast<float*>(xls);
    *reinterpret_cast<f32x4g*>(red + (wid * 16 + fr) * 16 + fs * 4) = acc;
    __syncthreads();
    if (wid != 0 || fr >= M) return;
    float v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        v[i] = 0.0f;
#pragma unroll
        for (int wv = 0; wv < 4; ++wv) v[i] += red[(wv * 16 + fr) * 16 + fs * 4 + i];
    }
    if (SPLIT) {
        const int N = gridDim.x * 16;
        *reinterpret_cast<float4*>(part + ((size_t)blockIdx.y * M + fr) * N + row0 + fs * 4) =
            make_float4(v[0], v[1], v[2], v[3]);
        return;
    }
    const int c0 = row0 - (gi ? gr.end[gi - 1] : 0);
    if (gr.act[gi] & GEMV_PAIRED) {
        uint16_t* po = gr.out[gi] + (size_t)fr * gr.os[gi] + c0 / 2 + fs * 2;
        const int act = gr.act[gi] - GEMV_PAIRED;
#pragma unroll
        for (int i = 0; i < 2; ++i) po[i] = f32_to_bf16(gemv_group_act(v[2 * i], act) * v[2 * i + 1]);
        return;
    }
    uint16_t* out = gr.out[gi] + (size_t)fr * gr.os[gi] + c0 + fs * 4;
#pragma unroll
    for (int i = 0; i < 4; ++i) out[i] = f32_to_bf16(gemv_group_act(v[i], gr.act[gi]));
}

// Partial sums of x [M, K] @ w [N, K]^T: part [ceil(K / unit), M, N] float32.
// K and unit multiples of 1024, N of 16, M <= 16.
extern "C" int oa_gemv_split(void* stream, const void* x, const void* w, void* part, int M, int N, int K,
                             int unit) {
    if (M < 1 || M > 16 || N % 16 != 0 || K % 1024 != 0 || unit < 1024 || unit % 1024 != 0) return -100;
    const size_t img = (size_t)M * (std::min(unit, K) * 2 + 16), red = 4 * 16 * 16 * 4;
    if (img > 147456) return -104;
    GemvGroups none = {};
    hipLaunchKernelGGL(gemv_grouped_mfma_kernel<true>, dim3(N / 16, CEIL_DIV(K, unit)), dim3(256),
                       img > red ? img : red, (hipStream_t)stream, (const uint32_t*)x,
                       (const uint32_t*)w, none, M, K, unit, (float*)part);
    HIP_CHECK_LAUNCH();
    return 0;
}

// x [P, M, K] contiguous (every group's plane < P, checked by the caller);
// w [N, K]; end/plane/act/out/os: host arrays of n entries, end[n-1] = N.
// mfma: the matrix-core form (K % 1024 == 0, M <= 16), else M 1..4.
extern "C" int oa_gemv_grouped(void* stream, const void* x, const void* w, int M, int N, int K, int n,
                               const int* end, const int* plane, const int* act, void* const* out,
                               const int64_t* os, int mfma) {
    if (M < 1 || n < 1 || n > GEMV_MAX_GROUPS || K % 8 != 0) return -100;
    GemvGroups gr;
    gr.n = n;
    int prev = 0;
    bool paired = false;
    for (int i = 0; i < n; ++i) {
        const int kind = act[i] & ~GEMV_PAIRED, pair = act[i] & GEMV_PAIRED ? 1 : 0;
        if (end[i] <= prev || end[i] % 16 != 0 || plane[i] < 0 || kind < 0 || kind > 2 || !out[i] ||
            os[i] < (end[i] - prev) >> pair)
            return -101;
        paired |= pair;
        gr.end[i] = prev = end[i];
        gr.plane[i] = plane[i];
        gr.act[i] = act[i];
        gr.out[i] = (uint16_t*)out[i];
        gr.os[i] = os[i];
    }
    if (prev != N) return -102;
    hipStream_t s = (hipStream_t)stream;
    if (mfma) {
        if (M > 16 || K % 1024 != 0) return -103;
        const size_t img = (size_t)M * (K * 2 + 16), red = 4 * 16 * 16 * 4;
        if (img > 147456) return -104;
        hipLaunchKernelGGL(gemv_grouped_mfma_kernel<false>, dim3(N / 16), dim3(256), img > red ? img : red,
                           s, (const uint32_t*)x, (const uint32_t*)w, gr, M, K, K, (float*)nullptr);
        HIP_CHECK_LAUNCH();
        return 0;
    }
    const bool rw1 = N <= 6144 && !paired;
    const int grid = std::min(2048, CEIL_DIV(N, rw1 ? 4 : 8));
#define GG(MV)                                                                                     \
    do {                                                                                           \
        if (rw1) hipLaunchKernelGGL((gemv_grouped_kernel<MV, 1>), dim3(grid), dim3(256), 0, s,     \
                                    (const uint32_t*)x, (const uint32_t*)w, gr, N, K / 2);         \
        else hipLaunchKernelGGL((gemv_grouped_kernel<MV, 2>), dim3(grid), dim3(256), 0, s,         \
                                (const uint32_t*)x, (const uint32_t*)w, gr, N, K / 2);             \
    } while (0)
    switch (M) {
        case 1: GG(1); break;
        case 2: GG(2); break;
        case 3: GG(3); break;
        case 4: GG(4); break;
        default: return -105;
    }
#undef GG
    HIP_CHECK_LAUNCH();
    return 0;
}
