// dense.hip -- products with dense weight matrices (bfloat16 or float32, row-major [out][in]) for the layer-list model families.
//
// One entry point for a product (ntk_dense) with three kernel forms behind it:
//   * dense_mfma_kernel   bf16 weights, more than kGemvRows rows: 128 x 128 / 64 x 128 / 64 x 64 output tiles on v_mfma_f32_16x16x32_bf16; the F32 activations are rounded
//                         to bfloat16 (nearest even) on their way into LDS, sums stay F32 in the accumulators;
//   * dense_fma_kernel    float32 weights, more than kGemvRows rows: the same tiling with plain F32 FMAs, k ascending (true 32-bit);
//   * dense_gemv_kernel   up to kGemvRows rows (decoding): every wave streams a few weight rows at once, 16 bytes per lane and row, the activation
//                         row sits in LDS; bf16 weights are widened exactly and multiplied in F32.  What runs inside the launch on the way in: what the row is still owed (a
//                         sublayer's normed output), an RMS norm; on the way out: a gated unit or an activation.
// Rows can be grouped (a mixture of experts: sorted rows of group g take matrix g) and gathered (row r reads activation row rows[r] / row_div).
// Group sizes live on the device, so the grid covers the worst case and workgroups outside their group's range leave at once.
// A second entry point (ntk_moe_few) runs all of a few tokens' chosen experts, the shared unit and their weighted sum in two row-streaming launches.
#include "common.hip.h"
#include "../../include/ntk_layers.h"

namespace ntk {

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float floatx4_t __attribute__((ext_vector_type(4)));
typedef uint32_t uintx4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ uint16_t f2bf(float f) {   // round to nearest even; NaN stays NaN
    uint32_t u = __float_as_uint(f);
    if ((u & 0x7fffffffu) > 0x7f800000u) return (uint16_t)((u >> 16) | 0x40u);
    u += 0x7fffu + ((u >> 16) & 1u);
    return (uint16_t)(u >> 16);
}
__device__ __forceinline__ float bf2f(uint16_t b) { return __uint_as_float((uint32_t)b << 16); }

struct DenseArgs {
    float* Y; int ldy;
    const float* X; int ldx;
    const void* W; long long wstride;
    const int* offsets;
    const int* rows; int row_div;
    int T, N, K, accumulate, G, vec, xvec;   // vec: weight rows 16-byte aligned, K % 8 == 0; xvec: activation rows (and norm_w) 16-byte aligned, K % 4 == 0
    int glu_ff; float glu_limit, glu_alpha, glu_up_offset, glu_cubic;   // few-row form only: outputs f < glu_ff = gated unit of rows f (gate) and glu_ff + f (up)
    const float* norm_w; float norm_eps, norm_offset;   // few-row form only: the activation row is RMS-normed with weight (offset + norm_w) first
    int act;                                            // NTK_ACT_*: on every output
    const float* add_y; int ld_add; const float* add_w; float add_eps, add_mult; float* x_out; int ldxo;   // few-row form only: see ntk_dense_desc
};

__device__ __forceinline__ bool group_range(const DenseArgs& a, int g, int& r0, int& r1) {
    if (a.offsets) { r0 = a.offsets[g]; r1 = a.offsets[g + 1]; } else { r0 = 0; r1 = a.T; }
    return r1 > r0;
}

__device__ __forceinline__ float activate(float v, int act) {
    if (act == NTK_ACT_RELU2) { const float p = fmaxf(v, 0.0f); return p * p; }
    return v;
}

// ---------------------------------------------------------------------------------------------------------------- bf16, matrix cores
// A workgroup of four waves (2 x 2) owns a TM x TN tile of Y; a wave owns (TM / 2) x (TN / 2) of it as 16 x 16 accumulator tiles.  K goes by in chunks
// of 32: the NEXT chunk's operands are requested into registers before the current one is multiplied out of LDS (global latency behind the MFMAs),
// activations are rounded to bfloat16 (nearest even, the hardware conversion) on their way into LDS.
constexpr int BK = 32, LDSK = BK + 8;   // LDS rows of 40 bf16 = 80 bytes: 16-byte aligned operand reads, rows 20 banks apart
typedef __bf16 bf16x2_t __attribute__((ext_vector_type(2)));
typedef float floatx2_t __attribute__((ext_vector_type(2)));

__device__ __forceinline__ uint32_t pack_bf16(float a, float b) {
    const bf16x2_t v = __builtin_convertvector(floatx2_t{a, b}, bf16x2_t);
    uint32_t u;
    __builtin_memcpy(&u, &v, 4);
    return u;
}

template <int TM, int TN, bool VEC>
__global__ __launch_bounds__(256) void dense_mfma_kernel(const DenseArgs a) {
    constexpr int PX = TM / 64, PW = TN / 64;        // loader passes of 64 rows
    constexpr int MI = TM / 32, NJ = TN / 32;        // 16 x 16 tiles per wave
    int r0, r1;
    if (!group_range(a, blockIdx.z, r0, r1)) return;
    const int row_base = r0 + blockIdx.y * TM;
    if (row_base >= r1) return;
    const int n_base = blockIdx.x * TN;
    const uint16_t* W = (const uint16_t*)a.W + (long long)blockIdx.z * a.wstride;
    __shared__ __attribute__((aligned(16))) uint16_t Xs[TM][LDSK];
    __shared__ __attribute__((aligned(16))) uint16_t Ws[TN][LDSK];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int wm = wave & 1, wn = wave >> 1;
    // loader: thread -> (row tid / 4 + 64 * pass, eight k from (tid & 3) * 8)
    const int lr = tid >> 2, lk = (tid & 3) * 8;
    const float* xrow[PX];
    const uint16_t* wrow[PW];
#pragma unroll
    for (int p = 0; p < PX; ++p) {
        const int xr = row_base + lr + 64 * p;
        xrow[p] = xr < r1 ? a.X + (long long)(a.rows ? a.rows[xr] / a.row_div : xr) * a.ldx : nullptr;
    }
#pragma unroll
    for (int p = 0; p < PW; ++p) {
        const int wr = n_base + lr + 64 * p;
        wrow[p] = wr < a.N ? W + (long long)wr * a.K : nullptr;
    }
    floatx4_t acc[MI][NJ];
#pragma unroll
    for (int i = 0; i < MI; ++i)
#pragma unroll
        for (int j = 0; j < NJ; ++j) acc[i][j] = floatx4_t{0.f, 0.f, 0.f, 0.f};
    uintx4_t xreg[PX], wreg[PW];
    auto fetch = [&](int k0) {
        const int k = k0 + lk;
#pragma unroll
        for (int p = 0; p < PX; ++p) {
            xreg[p] = uintx4_t{0u, 0u, 0u, 0u};
            if (xrow[p]) {
                if (VEC) {
                    if (k < a.K) {
                        const float4 v0 = *reinterpret_cast<const float4*>(xrow[p] + k), v1 = *reinterpret_cast<const float4*>(xrow[p] + k + 4);
                        xreg[p] = uintx4_t{pack_bf16(v0.x, v0.y), pack_bf16(v0.z, v0.w), pack_bf16(v1.x, v1.y), pack_bf16(v1.z, v1.w)};
                    }
                } else {
                    float v[8];
#pragma unroll
                    for (int j = 0; j < 8; ++j) v[j] = k + j < a.K ? xrow[p][k + j] : 0.0f;
                    xreg[p] = uintx4_t{pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]), pack_bf16(v[4], v[5]), pack_bf16(v[6], v[7])};
                }
            }
        }
#pragma unroll
        for (int p = 0; p < PW; ++p) {
            wreg[p] = uintx4_t{0u, 0u, 0u, 0u};
            if (wrow[p]) {
                if (VEC) {
                    if (k < a.K) wreg[p] = *reinterpret_cast<const uintx4_t*>(wrow[p] + k);
                } else {
                    uint32_t v[8];
#pragma unroll
                    for (int j = 0; j < 8; ++j) v[j] = k + j < a.K ? (uint32_t)wrow[p][k + j] : 0u;
                    wreg[p] = uintx4_t{v[0] | (v[1] << 16), v[2] | (v[3] << 16), v[4] | (v[5] << 16), v[6] | (v[7] << 16)};
                }
            }
        }
    };
    fetch(0);
    for (int k0 = 0; k0 < a.K; k0 += BK) {
        __syncthreads();   // the previous chunk's operand reads are done
#pragma unroll
        for (int p = 0; p < PX; ++p) *reinterpret_cast<uintx4_t*>(&Xs[lr + 64 * p][lk]) = xreg[p];
#pragma unroll
        for (int p = 0; p < PW; ++p) *reinterpret_cast<uintx4_t*>(&Ws[lr + 64 * p][lk]) = wreg[p];
        __syncthreads();
        if (k0 + BK < a.K) fetch(k0 + BK);
        bf16x8_t af[MI], bfr[NJ];
#pragma unroll
        for (int i = 0; i < MI; ++i) af[i] = *reinterpret_cast<const bf16x8_t*>(&Xs[wm * (TM / 2) + i * 16 + (lane & 15)][(lane >> 4) * 8]);
#pragma unroll
        for (int j = 0; j < NJ; ++j) bfr[j] = *reinterpret_cast<const bf16x8_t*>(&Ws[wn * (TN / 2) + j * 16 + (lane & 15)][(lane >> 4) * 8]);
#pragma unroll
        for (int i = 0; i < MI; ++i)
#pragma unroll
            for (int j = 0; j < NJ; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af[i], bfr[j], acc[i][j], 0, 0, 0);
    }
    // accumulator lane map: row 4 * (lane / 16) + r, column lane % 16.  What a sum is added onto is requested for a whole strip of tiles before the first store.
#pragma unroll
    for (int i = 0; i < MI; ++i) {
        const int row = row_base + wm * (TM / 2) + i * 16 + (lane >> 4) * 4;
        float* y = a.Y + (long long)row * a.ldy + n_base + wn * (TN / 2) + (lane & 15);
        const int n_left = a.N - (n_base + wn * (TN / 2) + (lane & 15));
        if (a.accumulate) {                                  // (uniform over the launch)
            float old[NJ][4];
#pragma unroll
            for (int j = 0; j < NJ; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r) old[j][r] = row + r < r1 && j * 16 < n_left ? y[(long long)r * a.ldy + j * 16] : 0.0f;
#pragma unroll
            for (int j = 0; j < NJ; ++j)
#pragma unroll
                for (int r = 0; r < 4; ++r) acc[i][j][r] += old[j][r];
        }
#pragma unroll
        for (int j = 0; j < NJ; ++j)
#pragma unroll
            for (int r = 0; r < 4; ++r)
                if (row + r < r1 && j * 16 < n_left) y[(long long)r * a.ldy + j * 16] = activate(acc[i][j][r], a.act);
    }
}

// ---------------------------------------------------------------------------------------------------------------- float32, vector FMA
constexpr int FK = 16, TM = 64, TN = 64;
__global__ __launch_bounds__(256) void dense_fma_kernel(const DenseArgs a) {
    int r0, r1;
    if (!group_range(a, blockIdx.z, r0, r1)) return;
    const int row_base = r0 + blockIdx.y * TM;
    if (row_base >= r1) return;
    const int n_base = blockIdx.x * TN;
    const float* W = (const float*)a.W + (long long)blockIdx.z * a.wstride;
    __shared__ __attribute__((aligned(16))) float Xs[FK][TM + 4];
    __shared__ __attribute__((aligned(16))) float Ws[FK][TN + 4];
    const int tid = threadIdx.x, ty = tid >> 4, tx = tid & 15;
    const int lr = tid >> 2, lk = (tid & 3) * 4;
    const int xr = row_base + lr;
    const bool x_ok = xr < r1;
    const float* xrow = nullptr;
    if (x_ok) xrow = a.X + (long long)(a.rows ? a.rows[xr] / a.row_div : xr) * a.ldx;
    const int wr = n_base + lr;
    const bool w_ok = wr < a.N;
    const float* wrow = W + (long long)wr * a.K;
    float acc[4][4] = {};
    for (int k0 = 0; k0 < a.K; k0 += FK) {
        float xv[4], wv[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int k = k0 + lk + j;
            xv[j] = (x_ok && k < a.K) ? xrow[k] : 0.0f;
            wv[j] = (w_ok && k < a.K) ? wrow[k] : 0.0f;
        }
        __syncthreads();
#pragma unroll
        for (int j = 0; j < 4; ++j) { Xs[lk + j][lr] = xv[j]; Ws[lk + j][lr] = wv[j]; }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < FK; ++k) {
            const float4 xa = *reinterpret_cast<const float4*>(&Xs[k][ty * 4]);
            const float4 wa = *reinterpret_cast<const float4*>(&Ws[k][tx * 4]);
            const float xs[4] = {xa.x, xa.y, xa.z, xa.w}, ws[4] = {wa.x, wa.y, wa.z, wa.w};
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(xs[i], ws[j], acc[i][j]);
        }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int row = row_base + ty * 4 + i, col = n_base + tx * 4 + j;
            if (row < r1 && col < a.N) {
                float* y = a.Y + (long long)row * a.ldy + col;
                *y = a.accumulate ? *y + acc[i][j] : activate(acc[i][j], a.act);
            }
        }
}

// ---------------------------------------------------------------------------------------------------------------- few rows: waves stream weight rows
// One workgroup per (group of 4 * RW outputs, activation row): the activation row sits in LDS, each wave owns RW consecutive weight rows and walks
// them together -- per step a lane requests the NEXT 16 bytes of each of its RW rows, then reads its 8 activations once and feeds RW sums from the bytes that
// have arrived; one DPP reduction per row at the end.  The first weights are requested together with the activation row and the weights of its norm, so they
// travel behind the norm's sum over the workgroup.  RW is picked so that the launch still has a few workgroups per CU.
constexpr int kGemvRows = 8;       // up to this many rows take this form
template <typename WT, int RW, bool GLU, bool ADD>
__global__ __launch_bounds__(256) void dense_gemv_kernel(const DenseArgs a) {
    extern __shared__ __attribute__((aligned(16))) float xs[];   // the activation row
    const int r = blockIdx.y;
    int g = 0;
    if (a.offsets) {
        if (r >= a.offsets[a.G]) return;
        while (r >= a.offsets[g + 1]) ++g;
    }
    const float* xrow = a.X + (long long)(a.rows ? a.rows[r] / a.row_div : r) * a.ldx;
    const WT* W = (const WT*)a.W + (long long)g * a.wstride;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    // GLU: the wave's RW rows are RW / 2 (gate, up) pairs of RW / 2 consecutive outputs
    constexpr int OUT = GLU ? RW / 2 : RW;
    const int n_out = GLU ? a.glu_ff : a.N;
    const int n0 = (blockIdx.x * 4 + wave) * OUT;
    const WT* w[RW];
#pragma unroll
    for (int i = 0; i < RW; ++i) {                          // rows past the end re-read the last one and are not stored
        const int row = GLU ? (i < OUT ? min(n0 + i, n_out - 1) : a.glu_ff + min(n0 + i - OUT, n_out - 1)) : min(n0 + i, n_out - 1);
        w[i] = W + (long long)row * a.K;
    }
    constexpr int NV = sizeof(WT) == 2 ? 1 : 2;             // 16-byte pieces of eight weights
    auto weights = [&](uintx4_t (&u)[RW][NV], int k) {
#pragma unroll
        for (int i = 0; i < RW; ++i)
#pragma unroll
            for (int p = 0; p < NV; ++p) u[i][p] = __builtin_nontemporal_load(reinterpret_cast<const uintx4_t*>(w[i] + k) + p);
    };
    __shared__ float red[16];
    float ss = 0.0f;
    uintx4_t first[RW][NV];
    if (a.xvec) {
        // the row's first 4096 entries stay in registers up to the norm; they, their norm weights and the wave's first weights are requested together
        constexpr int XV = 4;
        float4 xv[XV], nv[XV], yv[XV], aw[XV];
        const float* yrow = ADD ? a.add_y + (long long)r * a.ld_add : nullptr;
#pragma unroll
        for (int u = 0; u < XV; ++u) {
            const int k = 4 * (tid + 256 * u);
            if constexpr (ADD) {
                yv[u] = k < a.K ? *reinterpret_cast<const float4*>(yrow + k) : float4{0.0f, 0.0f, 0.0f, 0.0f};
                aw[u] = k < a.K ? *reinterpret_cast<const float4*>(a.add_w + k) : float4{0.0f, 0.0f, 0.0f, 0.0f};
            }
            xv[u] = k < a.K ? *reinterpret_cast<const float4*>(xrow + k) : float4{0.0f, 0.0f, 0.0f, 0.0f};
            nv[u] = a.norm_w && k < a.K ? *reinterpret_cast<const float4*>(a.norm_w + k) : float4{0.0f, 0.0f, 0.0f, 0.0f};
        }
        if (a.vec && lane * 8 < a.K) weights(first, lane * 8);
        for (int k = 4 * (tid + 256 * XV); k < a.K; k += 4 * 256) *reinterpret_cast<float4*>(xs + k) = *reinterpret_cast<const float4*>(xrow + k);
        float inv = 1.0f;
        if constexpr (ADD) {                                // what the row is still owed joins it; the first workgroup of the row leaves the sum
            float sy = 0.0f;
#pragma unroll
            for (int u = 0; u < XV; ++u) { sy = fmaf(yv[u].x, yv[u].x, sy); sy = fmaf(yv[u].y, yv[u].y, sy); sy = fmaf(yv[u].z, yv[u].z, sy); sy = fmaf(yv[u].w, yv[u].w, sy); }
            for (int k = 4 * (tid + 256 * XV); k < a.K; k += 4 * 256)
#pragma unroll
                for (int j = 0; j < 4; ++j) sy = fmaf(yrow[k + j], yrow[k + j], sy);
            const float iy = a.add_mult / sqrtf(block_sum(sy, red) / (float)a.K + a.add_eps);
            float* keep = blockIdx.x == 0 ? a.x_out + (long long)r * a.ldxo : nullptr;
#pragma unroll
            for (int u = 0; u < XV; ++u) {
                const int k = 4 * (tid + 256 * u);
                if (k >= a.K) continue;
                xv[u].x = fmaf(yv[u].x * iy, aw[u].x, xv[u].x); xv[u].y = fmaf(yv[u].y * iy, aw[u].y, xv[u].y);
                xv[u].z = fmaf(yv[u].z * iy, aw[u].z, xv[u].z); xv[u].w = fmaf(yv[u].w * iy, aw[u].w, xv[u].w);
                if (keep) *reinterpret_cast<float4*>(keep + k) = xv[u];
            }
            for (int k = 4 * (tid + 256 * XV); k < a.K; k += 4 * 256)
#pragma unroll
                for (int j = 0; j < 4; ++j) {               // (each thread rewrites what it wrote)
                    xs[k + j] = fmaf(yrow[k + j] * iy, a.add_w[k + j], xs[k + j]);
                    if (keep) keep[k + j] = xs[k + j];
                }
        }
        if (a.norm_w) {                                     // (uniform over the launch)
#pragma unroll
            for (int u = 0; u < XV; ++u) { ss = fmaf(xv[u].x, xv[u].x, ss); ss = fmaf(xv[u].y, xv[u].y, ss); ss = fmaf(xv[u].z, xv[u].z, ss); ss = fmaf(xv[u].w, xv[u].w, ss); }
            for (int k = 4 * (tid + 256 * XV); k < a.K; k += 4 * 256)
#pragma unroll
                for (int j = 0; j < 4; ++j) ss = fmaf(xs[k + j], xs[k + j], ss);
            inv = 1.0f / sqrtf(block_sum(ss, red) / (float)a.K + a.norm_eps);
            for (int k = 4 * (tid + 256 * XV); k < a.K; k += 4 * 256)
#pragma unroll
                for (int j = 0; j < 4; ++j) xs[k + j] = xs[k + j] * inv * (a.norm_offset + a.norm_w[k + j]);   // (each thread rewrites what it wrote)
        }
#pragma unroll
        for (int u = 0; u < XV; ++u) {
            const int k = 4 * (tid + 256 * u);
            if (k >= a.K) continue;
            float4 v = xv[u];
            if (a.norm_w) { v.x = v.x * inv * (a.norm_offset + nv[u].x); v.y = v.y * inv * (a.norm_offset + nv[u].y); v.z = v.z * inv * (a.norm_offset + nv[u].z); v.w = v.w * inv * (a.norm_offset + nv[u].w); }
            *reinterpret_cast<float4*>(xs + k) = v;
        }
    } else {
        if (a.vec && lane * 8 < a.K) weights(first, lane * 8);
        if constexpr (ADD) {
            const float* yrow = a.add_y + (long long)r * a.ld_add;
            float sy = 0.0f;
            for (int k = tid; k < a.K; k += 256) { xs[k] = xrow[k]; sy = fmaf(yrow[k], yrow[k], sy); }
            const float iy = a.add_mult / sqrtf(block_sum(sy, red) / (float)a.K + a.add_eps);
            float* keep = blockIdx.x == 0 ? a.x_out + (long long)r * a.ldxo : nullptr;
            for (int k = tid; k < a.K; k += 256) {
                const float v = fmaf(yrow[k] * iy, a.add_w[k], xs[k]);
                xs[k] = v;
                ss = fmaf(v, v, ss);
                if (keep) keep[k] = v;
            }
        } else {
            for (int k = tid; k < a.K; k += 256) { const float v = xrow[k]; xs[k] = v; ss = fmaf(v, v, ss); }
        }
        if (a.norm_w) {
            ss = block_sum(ss, red);
            const float inv = 1.0f / sqrtf(ss / (float)a.K + a.norm_eps);
            for (int k = tid; k < a.K; k += 256) xs[k] = xs[k] * inv * (a.norm_offset + a.norm_w[k]);   // (each thread rewrites what it wrote)
        }
    }
    __syncthreads();
    if (n0 >= n_out) return;                                // uniform per wave
    float s[RW];
#pragma unroll
    for (int i = 0; i < RW; ++i) s[i] = 0.0f;
    if (a.vec) {
        uintx4_t cur[RW][NV], next[RW][NV];
#pragma unroll
        for (int i = 0; i < RW; ++i)
#pragma unroll
            for (int p = 0; p < NV; ++p) cur[i][p] = first[i][p];
        for (int k = lane * 8; k < a.K; k += 64 * 8) {
            if (k + 64 * 8 < a.K) weights(next, k + 64 * 8);        // the next pass's weights behind this pass's sums
            float wv[RW][8];
#pragma unroll
            for (int i = 0; i < RW; ++i) {
                if constexpr (sizeof(WT) == 2) {
                    const uint32_t uu[4] = {cur[i][0].x, cur[i][0].y, cur[i][0].z, cur[i][0].w};
#pragma unroll
                    for (int j = 0; j < 4; ++j) { wv[i][2 * j] = __uint_as_float(uu[j] << 16); wv[i][2 * j + 1] = __uint_as_float(uu[j] & 0xffff0000u); }
                } else {
#pragma unroll
                    for (int p = 0; p < 2; ++p) {
                        wv[i][4 * p] = __uint_as_float(cur[i][p].x); wv[i][4 * p + 1] = __uint_as_float(cur[i][p].y);
                        wv[i][4 * p + 2] = __uint_as_float(cur[i][p].z); wv[i][4 * p + 3] = __uint_as_float(cur[i][p].w);
                    }
                }
            }
            const float4 x0 = *reinterpret_cast<const float4*>(xs + k), x1 = *reinterpret_cast<const float4*>(xs + k + 4);
            const float xv[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
#pragma unroll
            for (int i = 0; i < RW; ++i)
#pragma unroll
                for (int j = 0; j < 8; ++j) s[i] = fmaf(wv[i][j], xv[j], s[i]);
#pragma unroll
            for (int i = 0; i < RW; ++i)
#pragma unroll
                for (int p = 0; p < NV; ++p) cur[i][p] = next[i][p];
        }
    } else {
        for (int k = lane; k < a.K; k += 64) {
            const float xv = xs[k];
#pragma unroll
            for (int i = 0; i < RW; ++i) {
                float wv;
                if constexpr (sizeof(WT) == 2) wv = bf2f(((const uint16_t*)w[i])[k]); else wv = ((const float*)w[i])[k];
                s[i] = fmaf(wv, xv, s[i]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < RW; ++i) s[i] = wave_sum_lane63(s[i]);
#pragma unroll
    for (int i = 0; i < OUT; ++i) {
        if (lane == 63 && n0 + i < n_out) {
            float t = s[i];
            if constexpr (GLU) {
                const float gg = fminf(s[i], a.glu_limit), uu = fminf(fmaxf(s[i + OUT], -a.glu_limit), a.glu_limit);
                const float zz = a.glu_cubic != 0.0f ? fmaf(a.glu_cubic * gg * gg, gg, gg) : gg;
                t = gg * (1.0f / (1.0f + expf(-a.glu_alpha * zz))) * (uu + a.glu_up_offset);
            }
            float* y = a.Y + (long long)r * a.ldy + n0 + i;
            *y = a.accumulate ? *y + t : activate(t, a.act);
        }
    }
}

// ---------------------------------------------------------------------------------------------------------------- a few tokens' experts
// Two launches for everything between a router and the sum of its experts (see ntk_moe_few).  Both stream weight rows like dense_gemv_kernel: a wave owns RW rows, the
// next pass's 16 bytes per lane and row are requested before the current ones are used, the first ones ahead of the activations' way into LDS.
struct MoeFewArgs {
    float* out; int ldo;
    const float* h; int ldh;
    const int* ids; const float* wts; int top, experts;
    const void *up, *down, *shared_up, *shared_down; int ff, shared_ff;
    const float* sgate;
    int act; float* mid; int n, vec;
};

template <typename WT> struct WeightPiece {                  // eight weights of a row
    static constexpr int NV = sizeof(WT) == 2 ? 1 : 2;
    uintx4_t u[NV];
    __device__ __forceinline__ void load(const WT* p) {
#pragma unroll
        for (int i = 0; i < NV; ++i) u[i] = __builtin_nontemporal_load(reinterpret_cast<const uintx4_t*>(p) + i);
    }
    __device__ __forceinline__ void clear() {
#pragma unroll
        for (int i = 0; i < NV; ++i) u[i] = uintx4_t{0u, 0u, 0u, 0u};
    }
    __device__ __forceinline__ float dot(const float* x, float s) const {      // s + the eight products, k ascending; x 16-byte aligned
        const float4 x0 = *reinterpret_cast<const float4*>(x), x1 = *reinterpret_cast<const float4*>(x + 4);
        const float xv[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
        if constexpr (sizeof(WT) == 2) {
            const uint32_t w[4] = {u[0].x, u[0].y, u[0].z, u[0].w};
#pragma unroll
            for (int j = 0; j < 4; ++j) { s = fmaf(__uint_as_float(w[j] << 16), xv[2 * j], s); s = fmaf(__uint_as_float(w[j] & 0xffff0000u), xv[2 * j + 1], s); }
        } else {
#pragma unroll
            for (int p = 0; p < 2; ++p) {
                s = fmaf(__uint_as_float(u[p].x), xv[4 * p], s); s = fmaf(__uint_as_float(u[p].y), xv[4 * p + 1], s);
                s = fmaf(__uint_as_float(u[p].z), xv[4 * p + 2], s); s = fmaf(__uint_as_float(u[p].w), xv[4 * p + 3], s);
            }
        }
        return s;
    }
};
template <typename WT> __device__ __forceinline__ float weight_value(const WT* p) {
    if constexpr (sizeof(WT) == 2) return bf2f(*p); else return *p;
}

// mid[t][slot * ff + f] = act(U_e h)[f] times the expert's weight for the token's chosen experts, then the shared unit's times its gate; grid (rows / (4 RW), T)
template <typename WT, int RW>
__global__ __launch_bounds__(256) void moe_few_up_kernel(const MoeFewArgs a) {
    extern __shared__ __attribute__((aligned(16))) float xs[];   // the token's row
    const int t = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int routed = a.top * a.ff, rows = routed + a.shared_ff, m0 = (blockIdx.x * 4 + wave) * RW;
    const int* ids = a.ids + (long long)t * a.top;
    const WT* w[RW];
    bool any = false;
#pragma unroll
    for (int i = 0; i < RW; ++i) {                            // rows of identity experts and rows past the end: nothing to read
        const int m = m0 + i;
        w[i] = nullptr;
        if (m < routed) {
            const int e = ids[m / a.ff];
            if (e >= 0 && e < a.experts) w[i] = (const WT*)a.up + ((long long)e * a.ff + m % a.ff) * a.n;
        } else if (m < rows) {
            w[i] = (const WT*)a.shared_up + (long long)(m - routed) * a.n;
        }
        any = any || w[i];
    }
    WeightPiece<WT> cur[RW], next[RW];
    auto request = [&](WeightPiece<WT>(&p)[RW], int k) {
#pragma unroll
        for (int i = 0; i < RW; ++i) { if (w[i]) p[i].load(w[i] + k); else p[i].clear(); }
    };
    if (a.vec && lane * 8 < a.n) request(cur, lane * 8);
    const float* x = a.h + (long long)t * a.ldh;
    if (a.vec)
        for (int k = 4 * tid; k < a.n; k += 4 * 256) *reinterpret_cast<float4*>(xs + k) = *reinterpret_cast<const float4*>(x + k);
    else
        for (int k = tid; k < a.n; k += 256) xs[k] = x[k];
    __syncthreads();
    if (!any) return;                                         // (uniform over the wave)
    float s[RW];
#pragma unroll
    for (int i = 0; i < RW; ++i) s[i] = 0.0f;
    if (a.vec) {
        for (int k = lane * 8; k < a.n; k += 512) {
            if (k + 512 < a.n) request(next, k + 512);
#pragma unroll
            for (int i = 0; i < RW; ++i) { s[i] = cur[i].dot(xs + k, s[i]); cur[i] = next[i]; }
        }
    } else {
        for (int k = lane; k < a.n; k += 64)
#pragma unroll
            for (int i = 0; i < RW; ++i)
                if (w[i]) s[i] = fmaf(weight_value(w[i] + k), xs[k], s[i]);
    }
#pragma unroll
    for (int i = 0; i < RW; ++i) {
        s[i] = wave_sum_lane63(s[i]);
        if (lane == 63 && w[i]) {
            const float wt = m0 + i < routed ? a.wts[(long long)t * a.top + (m0 + i) / a.ff] : a.sgate ? a.sgate[t] : 1.0f;
            a.mid[(long long)t * rows + m0 + i] = activate(s[i], a.act) * wt;
        }
    }
}

// out[t][i] = one row of weights [D_e0[i] | D_e1[i] | ... | Ds[i]] against the weighted activations side by side; grid (n / (4 RW), T).  A wave goes through the
// row in passes of 512 entries inside one segment (a chosen expert, the shared unit; identity experts are passed over), with the requests of DEPTH passes under way.
template <typename WT, int RW, int DEPTH>
__global__ __launch_bounds__(256) void moe_few_down_kernel(const MoeFewArgs a) {
    extern __shared__ __attribute__((aligned(16))) float xs[];   // [top * ff + shared_ff]
    const int t = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int routed = a.top * a.ff, K = routed + a.shared_ff, i0 = (blockIdx.x * 4 + wave) * RW;
    const int* ids = a.ids + (long long)t * a.top;
    const float* mid = a.mid + (long long)t * K;
    long long row[RW];
#pragma unroll
    for (int i = 0; i < RW; ++i) row[i] = min(i0 + i, a.n - 1);     // (rows past the end re-read the last one and are not stored)
    // the pass that is requested next: segment (`top` = the shared unit, top + 1 = past the end), its matrix, the pass's first entry in it -- uniform over the wave
    int seg = -1, k0 = 0, len = 0;
    const WT* mat = nullptr;
    auto next_segment = [&]() {
        for (++seg, k0 = 0; seg < a.top; ++seg) {
            const int e = ids[seg];
            if (e >= 0 && e < a.experts) { mat = (const WT*)a.down + (long long)e * a.n * a.ff; len = a.ff; return; }
        }
        if (seg == a.top && a.shared_ff > 0) { mat = (const WT*)a.shared_down; len = a.shared_ff; return; }
        seg = a.top + 1;
    };
    WeightPiece<WT> piece[DEPTH][RW];
    int at[DEPTH];                                            // the lane's first activation of the pass (-1: none; -2: no pass)
    auto request = [&](WeightPiece<WT>(&p)[RW], int& x_at) {
        x_at = -2;
        if (seg > a.top) return;
        const int k = k0 + lane * 8;
        x_at = k < len ? (seg < a.top ? seg * a.ff : routed) + k : -1;
        if (x_at >= 0)
#pragma unroll
            for (int i = 0; i < RW; ++i) p[i].load(mat + row[i] * len + k);
        k0 += 512;
        if (k0 >= len) next_segment();
    };
    next_segment();
    if (a.vec)
#pragma unroll
        for (int d = 0; d < DEPTH; ++d) request(piece[d], at[d]);
    if (a.vec) {
        for (int m = 4 * tid; m < K; m += 4 * 256) *reinterpret_cast<float4*>(xs + m) = *reinterpret_cast<const float4*>(mid + m);
    } else {
        for (int m = tid; m < K; m += 256) xs[m] = mid[m];
    }
    __syncthreads();
    if (i0 >= a.n) return;                                    // (uniform over the wave)
    float s[RW];
#pragma unroll
    for (int i = 0; i < RW; ++i) s[i] = 0.0f;
    if (a.vec) {
        bool more = true;
        while (more) {
#pragma unroll
            for (int d = 0; d < DEPTH; ++d) {
                if (at[d] >= 0) {
#pragma unroll
                    for (int i = 0; i < RW; ++i) s[i] = piece[d][i].dot(xs + at[d], s[i]);
                }
                more = at[d] != -2;
                if (more) request(piece[d], at[d]);
            }
        }
    } else {
        for (; seg <= a.top; next_segment())
            for (int k = lane; k < len; k += 64)
#pragma unroll
                for (int i = 0; i < RW; ++i) s[i] = fmaf(weight_value(mat + row[i] * len + k), xs[(seg < a.top ? seg * a.ff : routed) + k], s[i]);
    }
    float ident = 0.0f;                                       // the weights of the token's identity experts
    for (int sl = 0; sl < a.top; ++sl)
        if (ids[sl] >= a.experts) ident += a.wts[(long long)t * a.top + sl];
#pragma unroll
    for (int i = 0; i < RW; ++i) {
        s[i] = wave_sum_lane63(s[i]);
        if (lane == 63 && i0 + i < a.n) a.out[(long long)t * a.ldo + i0 + i] = ident != 0.0f ? fmaf(ident, a.h[(long long)t * a.ldh + i0 + i], s[i]) : s[i];
    }
}

constexpr int kMoeDepth = 8;
template <typename WT>
static void launch_moe_few(const MoeFewArgs& a, int T, hipStream_t s) {
    const int rows = a.top * a.ff + a.shared_ff;
    const size_t lu = ((size_t)a.n * 4 + 15) & ~(size_t)15, ld = ((size_t)rows * 4 + 15) & ~(size_t)15;
    hipLaunchKernelGGL((moe_few_up_kernel<WT, 2>), dim3((rows + 7) / 8, T), dim3(256), lu, s, a);
    if ((long long)a.n * T >= 4096) hipLaunchKernelGGL((moe_few_down_kernel<WT, 2, kMoeDepth>), dim3((a.n + 7) / 8, T), dim3(256), ld, s, a);
    else hipLaunchKernelGGL((moe_few_down_kernel<WT, 1, kMoeDepth>), dim3((a.n + 3) / 4, T), dim3(256), ld, s, a);
}

template <typename WT, bool ADD>
static void launch_gemv(const DenseArgs& a, int rows, hipStream_t s) {
    const size_t lds = ((size_t)a.K * 4 + 15) & ~(size_t)15;
    // Rows per wave, measured over layer-like shapes (2048 .. 64000 outputs of 768 .. 4096 inputs, 1 .. 6 activation rows): two rows per wave are
    // the best or within noise everywhere from 4096 outputs x rows on (a 64000 x 4096 head: 84 us against 98 with one or eight), one below; launches
    // under ~20 MB sit at 4 - 6 us whatever the choice.  The GLU form keeps pairs: 4 pairs per wave for the large expert launches.
    const long long work = (long long)a.N * rows;
    int rw = work >= 4096 ? 2 : 1;
    if (const int force = NTK_TUNE_ENV_INT("NTK_DENSE_GEMV_RW", 0)) rw = force;   // (tuning builds only)
    if (a.glu_ff > 0) {
        const int out = work >= 4 * 8 * 512 ? 4 : work >= 4 * 4 * 512 ? 2 : 1;   // (gate, up) pairs per wave
        const dim3 grid((a.glu_ff + 4 * out - 1) / (4 * out), rows, 1);
        if (out == 4) hipLaunchKernelGGL((dense_gemv_kernel<WT, 8, true, ADD>), grid, dim3(256), lds, s, a);
        else if (out == 2) hipLaunchKernelGGL((dense_gemv_kernel<WT, 4, true, ADD>), grid, dim3(256), lds, s, a);
        else hipLaunchKernelGGL((dense_gemv_kernel<WT, 2, true, ADD>), grid, dim3(256), lds, s, a);
        return;
    }
    const dim3 grid((a.N + 4 * rw - 1) / (4 * rw), rows, 1);
    if (rw == 8) hipLaunchKernelGGL((dense_gemv_kernel<WT, 8, false, ADD>), grid, dim3(256), lds, s, a);
    else if (rw == 4) hipLaunchKernelGGL((dense_gemv_kernel<WT, 4, false, ADD>), grid, dim3(256), lds, s, a);
    else if (rw == 2) hipLaunchKernelGGL((dense_gemv_kernel<WT, 2, false, ADD>), grid, dim3(256), lds, s, a);
    else hipLaunchKernelGGL((dense_gemv_kernel<WT, 1, false, ADD>), grid, dim3(256), lds, s, a);
}

}  // namespace ntk

using namespace ntk;

int ntk_dense(const ntk_dense_desc* d, void* stream) {
    if (!d || !d->Y || !d->X || !d->W) return NTK_E_NULL;
    if (d->wdtype != NTK_DT_BF16 && d->wdtype != NTK_DT_F32) return NTK_E_DTYPE;
    if (d->T < 0 || d->N <= 0 || d->K <= 0 || d->ldx < d->K || d->ldy < (d->glu_ff > 0 ? d->glu_ff : d->N)) return NTK_E_SHAPE;
    if (d->offsets && d->G <= 0) return NTK_E_SHAPE;
    if (d->rows && d->row_div <= 0) return NTK_E_SHAPE;
    if (d->glu_ff > 0 && (d->T > kGemvRows || d->N != 2 * d->glu_ff || d->accumulate)) return NTK_E_SHAPE;
    if (d->norm_w && d->T > kGemvRows) return NTK_E_SHAPE;
    if ((d->act != NTK_ACT_NONE && d->act != NTK_ACT_RELU2) || (d->act && (d->accumulate || d->glu_ff > 0))) return NTK_E_SHAPE;
    if (d->add_y && (!d->add_w || !d->x_out)) return NTK_E_NULL;
    if (d->add_y && (d->T > kGemvRows || d->rows || d->offsets || d->ld_add < d->K || d->ldxo < d->K || d->x_out == d->X || d->x_out == d->add_y)) return NTK_E_SHAPE;
    if (d->T == 0) return NTK_OK;
    const int G = d->offsets ? d->G : 1;
    DenseArgs a{d->Y, d->ldy, d->X, d->ldx, d->W, d->wstride, d->offsets, d->rows, d->rows ? d->row_div : 1, d->T, d->N, d->K, d->accumulate, G, 0, 0, 0, 0.0f, 0.0f, 0.0f, 0.0f, nullptr, 0.0f, 0.0f, d->act, nullptr, 0, nullptr, 0.0f, 0.0f, nullptr, 0};
    hipStream_t s = resolve_stream(stream);
    if (d->T <= kGemvRows) {
        if ((size_t)d->K * 4 > 160 * 1024 - 1024) return NTK_E_SHAPE;
        a.glu_ff = d->glu_ff; a.glu_limit = d->glu_limit; a.glu_alpha = d->glu_alpha; a.glu_up_offset = d->glu_up_offset; a.glu_cubic = d->glu_cubic;
        a.norm_w = d->norm_w; a.norm_eps = d->norm_eps; a.norm_offset = d->norm_offset;
        a.vec = (d->K % 8 == 0) && !((uintptr_t)d->W & 15) && !((d->wstride * (d->wdtype == NTK_DT_BF16 ? 2 : 4)) & 15);
        a.xvec = (d->K % 4 == 0) && (d->ldx % 4 == 0) && !((uintptr_t)d->X & 15) && !((uintptr_t)d->norm_w & 15);
        if (d->add_y) {
            a.add_y = d->add_y; a.ld_add = d->ld_add; a.add_w = d->add_w; a.add_eps = d->add_eps; a.add_mult = d->add_mult; a.x_out = d->x_out; a.ldxo = d->ldxo;
            a.xvec = a.xvec && (d->ld_add % 4 == 0) && (d->ldxo % 4 == 0) && !(((uintptr_t)d->add_y | (uintptr_t)d->add_w | (uintptr_t)d->x_out) & 15);
            if (d->wdtype == NTK_DT_BF16) launch_gemv<uint16_t, true>(a, d->T, s);
            else launch_gemv<float, true>(a, d->T, s);
            return last_launch_status();
        }
        if (d->wdtype == NTK_DT_BF16) launch_gemv<uint16_t, false>(a, d->T, s);
        else launch_gemv<float, false>(a, d->T, s);
        return last_launch_status();
    }
    if (d->wdtype == NTK_DT_BF16) {
        const bool vec = (d->K % 8 == 0) && (d->ldx % 4 == 0) && !((uintptr_t)d->X & 15) && !((uintptr_t)d->W & 15) && (d->wstride % 8 == 0);
        // 128 x 128 tiles where a group has the rows and the launch still fills the chip; 64-row tiles for short groups (experts, short portions)
        const int rows_per_group = d->T / G;
        const bool big = rows_per_group >= 192 && d->N >= 128 && (long long)((d->T + 127) / 128) * ((d->N + 127) / 128) >= 224;
        if (big) {
            const dim3 grid((d->N + 127) / 128, (d->T + 127) / 128, G);
            if (vec) hipLaunchKernelGGL((dense_mfma_kernel<128, 128, true>), grid, dim3(256), 0, s, a);
            else hipLaunchKernelGGL((dense_mfma_kernel<128, 128, false>), grid, dim3(256), 0, s, a);
        } else if (d->N >= 128) {
            const dim3 grid((d->N + 127) / 128, (d->T + 63) / 64, G);
            if (vec) hipLaunchKernelGGL((dense_mfma_kernel<64, 128, true>), grid, dim3(256), 0, s, a);
            else hipLaunchKernelGGL((dense_mfma_kernel<64, 128, false>), grid, dim3(256), 0, s, a);
        } else {
            const dim3 grid((d->N + 63) / 64, (d->T + 63) / 64, G);
            if (vec) hipLaunchKernelGGL((dense_mfma_kernel<64, 64, true>), grid, dim3(256), 0, s, a);
            else hipLaunchKernelGGL((dense_mfma_kernel<64, 64, false>), grid, dim3(256), 0, s, a);
        }
    } else {
        const dim3 grid((d->N + TN - 1) / TN, (d->T + TM - 1) / TM, G);
        hipLaunchKernelGGL(dense_fma_kernel, grid, dim3(256), 0, s, a);
    }
    return last_launch_status();
}

int ntk_moe_few(const ntk_moe_few_desc* d, void* stream) {
    if (!d || !d->out || !d->h || !d->ids || !d->wts || !d->up || !d->down || !d->mid || (d->shared_ff > 0 && (!d->shared_up || !d->shared_down))) return NTK_E_NULL;
    if (d->wdtype != NTK_DT_BF16 && d->wdtype != NTK_DT_F32) return NTK_E_DTYPE;
    if (d->act != NTK_ACT_NONE && d->act != NTK_ACT_RELU2) return NTK_E_SHAPE;
    if (d->T < 0 || d->T > kGemvRows || d->n <= 0 || d->top <= 0 || d->experts <= 0 || d->ff <= 0 || d->shared_ff < 0 || d->ldo < d->n || d->ldh < d->n) return NTK_E_SHAPE;
    if ((long long)d->top * d->ff + d->shared_ff > NTK_MOE_FEW_MID || d->n > NTK_MOE_FEW_MID) return NTK_E_SHAPE;
    if (d->T == 0) return NTK_OK;
    MoeFewArgs a{d->out, d->ldo, d->h, d->ldh, d->ids, d->wts, d->top, d->experts, d->up, d->down, d->shared_up, d->shared_down, d->ff, d->shared_ff, d->sgate, d->act, d->mid, d->n, 0};
    a.vec = d->n % 8 == 0 && d->ff % 8 == 0 && d->shared_ff % 8 == 0 && d->ldh % 4 == 0 &&
            !(((uintptr_t)d->h | (uintptr_t)d->up | (uintptr_t)d->down | (uintptr_t)d->shared_up | (uintptr_t)d->shared_down) & 15);
    static bool raised = false;     // (idempotent: a race sets the same attributes twice)
    if (!raised) {
        const void* fn[] = {(const void*)moe_few_up_kernel<uint16_t, 2>, (const void*)moe_few_up_kernel<float, 2>, 
                            (const void*)moe_few_down_kernel<uint16_t, 2, kMoeDepth>, (const void*)moe_few_down_kernel<float, 2, kMoeDepth>,
                            (const void*)moe_few_down_kernel<uint16_t, 1, kMoeDepth>, (const void*)moe_few_down_kernel<float, 1, kMoeDepth>};
        for (const void* f : fn) NTK_HIP_TRY(hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, NTK_MOE_FEW_MID * 4));
        raised = true;
    }
    if (d->wdtype == NTK_DT_BF16) launch_moe_few<uint16_t>(a, d->T, resolve_stream(stream));
    else launch_moe_few<float>(a, d->T, resolve_stream(stream));
    return last_launch_status();
}

int ntk_dense_few_rows(void) { return kGemvRows; }

int ntk_dense_linear(float* Y, int ldy, const float* X, int ldx, const void* W, int wdtype, int T, int N, int K, int accumulate, void* stream) {
    ntk_dense_desc d{};
    d.Y = Y; d.ldy = ldy; d.X = X; d.ldx = ldx; d.W = W; d.wstride = 0; d.wdtype = wdtype; d.offsets = nullptr; d.G = 1; d.rows = nullptr; d.row_div = 1;
    d.T = T; d.N = N; d.K = K; d.accumulate = accumulate;
    return ntk_dense(&d, stream);
}
