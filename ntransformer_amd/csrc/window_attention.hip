// window_attention.hip -- grouped-query softmax attention over a cache of rotated keys and values: causal, optional sliding window, one or two score
// maps per head over the same values (two maps: the differential pair out = a_0 - lambda * a_1), optional unit norm of every head's output, optional
// learned bias by bucketed distance on the scaled score (a table of distances -> buckets, a table of buckets x heads) or a bias that falls with the distance at
// a rate of the head's, optional cap on the score
// (cap * tanh(score / cap)), optional sink (a key without a value in every softmax: of score 0, or of a learned score per head), optional gate on the output
// (element by element or one number per head); beside the sliding window the first `keep_first` positions can stay visible for ever, and instead of it there is a
// mask of chunks (a query sees the keys of its own chunk of `window` positions, counted from position 0, up to itself).
//
// Cache row of a position: [G][maps][dn] rotated keys | [G][dv] values, F32.  Scores, softmax, weights and sums are F32 on the vector units.
// A workgroup owns 16 (token, head) rows of ONE key/value head -- consecutive tokens times the heads that share it, so a key or value slab that was
// staged in LDS serves every query head of the group -- and walks the visible keys in chunks of 64: lane = key for the scores (key slabs of 64 entries
// in LDS), online softmax per row and map, lane = value column for the weighted sums (the value slab is loaded once for both maps).  When few rows
// face many keys (decoding), the chunks go round `splits` workgroups and a second launch merges their (max, sum, vector) states.
#include <algorithm>
#include "common.hip.h"
#include "../../include/ntk_layers.h"

namespace ntk {

// one workgroup per token: q rotated in place, k rotated into the cache row, v copied behind.  Angles in double (position times frequency), applied in F32.
// Optional: what the projections left to their consumer -- bias vectors on q, k and v, and a query temperature that grows with the position --, and an RMS norm
// over the token's WHOLE q (and whole k) ahead of the rotation.  k == NULL: queries only (a layer that reads another layer's cache rows).
struct PrepareArgs {
    float* cache; int row;
    float* q; int ldq; const float* k; int ldk; const float* v; int ldv;
    int nq, nk, dn, nv;                      // vectors of dn entries in q and in k (heads x maps), value entries
    const double* freq; float mag; int dims, halves, pos0;
    const float *qb, *kb, *vb; float temp_coef; double temp_every;
    const float* v_other; int ld_other; float v_blend; float* v_keep; int ld_keep;
    const float *q_norm, *k_norm; float norm_eps;
};

template <int NT>
__global__ __launch_bounds__(NT) void window_prepare_kernel(const PrepareArgs a) {
    extern __shared__ float cs[];   // [dims / 2] cos, [dims / 2] sin
    const int t = blockIdx.x, pos = a.pos0 + t, dn = a.dn;
    const int half = a.dims / 2;
    float* qt = a.q + (long long)t * a.ldq;
    const float* kt = a.k ? a.k + (long long)t * a.ldk : nullptr;
    if (a.qb || a.temp_coef != 0.0f) {     // (uniform over the launch) q = (q + bias) * temperature, ahead of the rotation: a thread rewrites its own entries
        const float temp = a.temp_coef != 0.0f ? 1.0f + a.temp_coef * logf((float)floor((double)(pos + 1) / a.temp_every) + 1.0f) : 1.0f;
        for (int j = threadIdx.x; j < a.nq * dn; j += NT) qt[j] = (qt[j] + (a.qb ? a.qb[j] : 0.0f)) * temp;
        __syncthreads();
    }
    for (int i = threadIdx.x; i < half; i += NT) {
        const double ang = (double)pos * a.freq[i];
        cs[i] = (float)(cos(ang) * (double)a.mag);
        cs[half + i] = (float)(sin(ang) * (double)a.mag);
    }
    float qs = 1.0f, ks = 1.0f;            // one over the root mean square of the whole q / k
    if (a.q_norm || a.k_norm) {            // (uniform over the launch)
        __shared__ float red[16];
        float sq = 0.0f, sk = 0.0f;
        if (a.q_norm) for (int j = threadIdx.x; j < a.nq * dn; j += NT) sq = fmaf(qt[j], qt[j], sq);
        if (a.k_norm && kt)
            for (int j = threadIdx.x; j < a.nk * dn; j += NT) { const float x = kt[j] + (a.kb ? a.kb[j] : 0.0f); sk = fmaf(x, x, sk); }
        if (a.q_norm) qs = 1.0f / sqrtf(block_sum(sq, red) / (float)(a.nq * dn) + a.norm_eps);
        if (a.k_norm && kt) ks = 1.0f / sqrtf(block_sum(sk, red) / (float)(a.nk * dn) + a.norm_eps);
    }
    __syncthreads();
    auto q_at = [&](int o) { return a.q_norm ? qt[o] * qs * a.q_norm[o] : qt[o]; };
    auto k_at = [&](int o) { const float x = kt[o] + (a.kb ? a.kb[o] : 0.0f); return a.k_norm ? x * ks * a.k_norm[o] : x; };
    const int pair = a.halves ? half : 1, step = a.halves ? 1 : 2;   // pair i = entries (i * step, i * step + pair)
    const int rest = dn - a.dims;
    for (int j = threadIdx.x; j < a.nq * half; j += NT) {       // nq = heads x maps vectors of dn
        const int o = (j / half) * dn + step * (j % half);
        float ra, rb;
        rope_rotate(q_at(o), q_at(o + pair), cs[j % half], cs[half + j % half], ra, rb);
        qt[o] = ra;
        qt[o + pair] = rb;
    }
    if (a.q_norm)
        for (int j = threadIdx.x; j < a.nq * rest; j += NT) {
            const int o = (j / rest) * dn + a.dims + j % rest;
            qt[o] = q_at(o);
        }
    if (!kt) return;
    float* dst = a.cache + (long long)pos * a.row;
    const float* vt = a.v + (long long)t * a.ldv;
    for (int j = threadIdx.x; j < a.nk * half; j += NT) {
        const int o = (j / half) * dn + step * (j % half);
        float ra, rb;
        rope_rotate(k_at(o), k_at(o + pair), cs[j % half], cs[half + j % half], ra, rb);
        dst[o] = ra;
        dst[o + pair] = rb;
    }
    for (int j = threadIdx.x; j < a.nk * rest; j += NT) {
        const int o = (j / rest) * dn + a.dims + j % rest;
        dst[o] = k_at(o);
    }
    for (int j = threadIdx.x; j < a.nv; j += NT) {
        float vv = vt[j] + (a.vb ? a.vb[j] : 0.0f);
        if (a.v_keep) a.v_keep[(long long)t * a.ld_keep + j] = vv;
        if (a.v_other) vv = fmaf(a.v_blend, a.v_other[(long long)t * a.ld_other + j], (1.0f - a.v_blend) * vv);
        dst[a.nk * dn + j] = vv;
    }
}

// One wave per (token, vector): RMS norm of every head's vector on its own with one shared weight, query temperature behind the norm, rotation; the values are copied
// (they may be the keys as they were projected).  A lane re-reads and rewrites its own entries or pairs only, after the wave's sum has used all of them.
__global__ __launch_bounds__(256) void window_prepare_heads_kernel(const PrepareArgs a, int G) {
    const int lane = threadIdx.x & 63, j = blockIdx.y * 4 + (threadIdx.x >> 6), dn = a.dn, dv = a.nv / G;
    const int t = blockIdx.x, pos = a.pos0 + t, nk = a.k ? a.nk : 0;
    if (j >= a.nq + nk + (a.k ? G : 0)) return;
    if (j >= a.nq + nk) {                                     // a value vector
        const int o = (j - a.nq - nk) * dv;
        const float* vt = a.v + (long long)t * a.ldv + o;
        float* dst = a.cache + (long long)pos * a.row + nk * dn + o;
        for (int i = lane; i < dv; i += 64) dst[i] = vt[i] + (a.vb ? a.vb[o + i] : 0.0f);
        return;
    }
    const bool is_q = j < a.nq;
    const int o = (is_q ? j : j - a.nq) * dn;
    const float* src = is_q ? a.q + (long long)t * a.ldq + o : a.k + (long long)t * a.ldk + o;
    float* dst = is_q ? a.q + (long long)t * a.ldq + o : a.cache + (long long)pos * a.row + o;
    const float* b = is_q ? a.qb : a.kb;
    const float* w = is_q ? a.q_norm : a.k_norm;
    constexpr int KEEP = 4;                                   // a lane's first entries stay in registers
    float v[KEEP];
    float ss = 0.0f;
#pragma unroll
    for (int u = 0; u < KEEP; ++u) {
        const int i = lane + 64 * u;
        v[u] = i < dn ? src[i] + (b ? b[o + i] : 0.0f) : 0.0f;
        ss = fmaf(v[u], v[u], ss);
    }
    for (int i = lane + 64 * KEEP; i < dn; i += 64) { const float x = src[i] + (b ? b[o + i] : 0.0f); ss = fmaf(x, x, ss); }
    const float inv = w ? 1.0f / sqrtf(wave_sum(ss) / (float)dn + a.norm_eps) : 1.0f;
    const float temp = is_q && a.temp_coef != 0.0f ? 1.0f + a.temp_coef * logf((float)floor((double)(pos + 1) / a.temp_every) + 1.0f) : 1.0f;
    auto formed = [&](float x, int i) { x = w ? x * inv * w[i] : x; return is_q ? x * temp : x; };
    if (a.dims == 0) {
#pragma unroll
        for (int u = 0; u < KEEP; ++u)
            if (lane + 64 * u < dn) dst[lane + 64 * u] = formed(v[u], lane + 64 * u);
        for (int i = lane + 64 * KEEP; i < dn; i += 64) dst[i] = formed(src[i] + (b ? b[o + i] : 0.0f), i);
        return;
    }
    const int half = a.dims / 2, pair = a.halves ? half : 1, step = a.halves ? 1 : 2;   // pair i = entries (i * step, i * step + pair)
    for (int i = lane; i < half; i += 64) {
        const int e = step * i;
        const double ang = (double)pos * a.freq[i];
        float ra, rb;
        rope_rotate(formed(src[e] + (b ? b[o + e] : 0.0f), e), formed(src[e + pair] + (b ? b[o + e + pair] : 0.0f), e + pair), (float)(cos(ang) * (double)a.mag),
                    (float)(sin(ang) * (double)a.mag), ra, rb);
        dst[e] = ra;
        dst[e + pair] = rb;
    }
    for (int i = a.dims + lane; i < dn; i += 64) dst[i] = formed(src[i] + (b ? b[o + i] : 0.0f), i);
}

struct WinArgs {
    float* out; int ldo;
    const float* q; int ldq;
    const float* cache; int row;
    int H, G, dn, dv, pos0, T, window;
    float scale, lambda;
    int sub_norm; float eps, out_scale;
    int splits; float* scratch;       // splits > 1: states [T * H][splits][maps][2 + dv]
    const float* rel; const int* bucket_of; int n_dist;   // rel != NULL: rel[bucket_of[min(distance, n_dist - 1)] * H + head] joins the scaled score
    int chunks; float softcap; int sink;                  // chunks != 0: `window` is a chunk size
    const float* gate; int ldg, head_gate;                // gate != NULL: out[t][h][c] *= sigmoid(gate[t * ldg + h * dv + c]), or gate[t * ldg + h] with head_gate
    int keep;                                             // positions 0 .. keep - 1 stay visible behind the sliding window
    const float* sinks;                                   // the sink's score per head (NULL with `sink`: 0)
    const float* slopes;                                  // slopes[head] * distance comes off the scaled score
};

// first key a query at position p sees
__device__ __forceinline__ int first_visible(int p, int window, int chunks) {
    if (window <= 0) return 0;
    return chunks ? (p / window) * window : max(0, p - window + 1);
}

constexpr int WROWS = 16, WQPW = 4, WKCH = 64, WSLAB = 64, WMAXC = 8;   // dv <= WMAXC * WSLAB

// the gate of row (t, h): its first entry and the distance to the next column's (0: one gate for the head)
__device__ __forceinline__ const float* gate_of(const WinArgs& a, int t, int h) {
    return a.gate ? a.gate + (long long)t * a.ldg + (a.head_gate ? h : h * a.dv) : nullptr;
}

// the differential pair, the unit norm and the scale on a row whose lanes hold columns c * 64 + lane
template <int M>
__device__ __forceinline__ void finish_row(float (&a)[M][WMAXC], int lane, int dv, float lambda, int sub_norm, float eps, float out_scale, float* o, const float* gate, int gate_step) {
    float r[WMAXC];
    float ss = 0.0f;
#pragma unroll
    for (int c = 0; c < WMAXC; ++c) {
        float x = a[0][c];
        if constexpr (M == 2) x = x - lambda * a[1][c];
        if (c * WSLAB + lane >= dv) x = 0.0f;
        r[c] = x;
        ss = fmaf(x, x, ss);
    }
    float mul = out_scale;
    if (sub_norm) mul = out_scale / sqrtf(wave_sum(ss) / (float)dv + eps);
#pragma unroll
    for (int c = 0; c < WMAXC; ++c)
        if (c * WSLAB + lane < dv) o[c * WSLAB + lane] = gate ? r[c] * mul / (1.0f + expf(-gate[(c * WSLAB + lane) * gate_step])) : r[c] * mul;
}

template <int M>
__global__ __launch_bounds__(256) void window_attention_kernel(const WinArgs a) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int DNP = (a.dn + 3) & ~3;
    float* Qs = lds;                               // [WROWS][M][DNP]
    float* Sl = Qs + WROWS * M * DNP;              // [WKCH][WSLAB + 1] key slab / [WKCH][WSLAB] value slab
    float* Ps = Sl + WKCH * (WSLAB + 1);           // [M][WROWS][WKCH]
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int g = blockIdx.y, R = a.H / a.G, n_rows = a.T * R;
    const int row0 = blockIdx.x * WROWS;
    const int last = min(row0 + WROWS, n_rows) - 1;
    const int pmin = a.pos0 + row0 / R, pmax = a.pos0 + last / R;
    const int jlo = first_visible(pmin, a.window, a.chunks);
    const int jhi = pmax;   // inclusive
    // the keys walked: positions 0 .. kept - 1 (those of the kept first ones that lie before the window), then jlo .. jhi; key number i of the walk is position
    // i, or i + skip from `kept` on
    const int kept = min(a.keep, jlo), skip = jlo - kept, n_keys = kept + jhi - jlo + 1;
    // queries into LDS
    for (int e0 = threadIdx.x; e0 < WROWS * M * DNP; e0 += 256 * 4) {     // (four of a thread's entries asked for before the first is stored)
        float qv[4];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
            const int e = e0 + 256 * u, i = e / (M * DNP), md = e % (M * DNP), m = md / DNP, d = md % DNP;
            const int rho = row0 + i;
            qv[u] = (e < WROWS * M * DNP && rho < n_rows && d < a.dn) ? a.q[(long long)(rho / R) * a.ldq + ((long long)(g * R + rho % R) * M + m) * a.dn + d] : 0.0f;
        }
#pragma unroll
        for (int u = 0; u < 4; ++u)
            if (e0 + 256 * u < WROWS * M * DNP) Qs[e0 + 256 * u] = qv[u];
    }
    float mx[M][WQPW], l[M][WQPW], acc[M][WQPW][WMAXC];
    int rpos[WQPW], rhead[WQPW];
    float slope[WQPW];
#pragma unroll
    for (int i = 0; i < WQPW; ++i) {
        const int rho = row0 + wave * WQPW + i;
        rpos[i] = rho < n_rows ? a.pos0 + rho / R : -1;
        rhead[i] = g * R + rho % R;
        slope[i] = a.slopes ? a.slopes[rhead[i]] : 0.0f;
        // the sink is a key without a value: the running maximum and sum start from it (in the first part only when the keys are split)
        const bool sunk = (a.sink || a.sinks) && (a.splits <= 1 || blockIdx.z == 0);
        const float sink_score = a.sinks ? a.sinks[rhead[i]] : 0.0f;
#pragma unroll
        for (int m = 0; m < M; ++m) {
            mx[m][i] = sunk ? sink_score : -INFINITY; l[m][i] = sunk ? 1.0f : 0.0f;
#pragma unroll
            for (int c = 0; c < WMAXC; ++c) acc[m][i][c] = 0.0f;
        }
    }
    const int vbase = a.G * M * a.dn + g * a.dv;
    int chunk = 0;
    for (int i0 = 0; i0 < n_keys; i0 += WKCH, ++chunk) {
        if (a.splits > 1 && chunk % a.splits != (int)blockIdx.z) continue;     // (uniform over the workgroup)
        const int nk = min(WKCH, n_keys - i0);
        auto key_pos = [&](int k) { return i0 + k + (i0 + k >= kept ? skip : 0); };   // position of the chunk's key k
        const int j = key_pos(lane);
#pragma unroll
        for (int m = 0; m < M; ++m) {
            float s[WQPW];
#pragma unroll
            for (int i = 0; i < WQPW; ++i) s[i] = 0.0f;
            // ---- scores of map m: slabs of WSLAB key entries
            for (int d0 = 0; d0 < a.dn; d0 += WSLAB) {
                const int nd = min(WSLAB, a.dn - d0);
                __syncthreads();
                {   // thread -> (key wave + 4 u, entry lane): the sixteen requests of a thread in flight before the first is stored
                    const float* src = a.cache + (g * M + m) * a.dn + d0 + lane;
                    float v[16];
#pragma unroll
                    for (int u = 0; u < 16; ++u) {
                        const int k = wave + 4 * u;
                        v[u] = (k < nk && lane < nd) ? src[(long long)key_pos(k) * a.row] : 0.0f;
                    }
#pragma unroll
                    for (int u = 0; u < 16; ++u) Sl[(wave + 4 * u) * (WSLAB + 1) + lane] = v[u];
                }
                __syncthreads();
                const float* kr = Sl + lane * (WSLAB + 1);
                for (int d = 0; d < nd; d += 4) {      // (entries past nd are zero in the slab, past dn in the queries)
                    const float k0 = kr[d], k1 = kr[d + 1], k2 = kr[d + 2], k3 = kr[d + 3];
#pragma unroll
                    for (int i = 0; i < WQPW; ++i) {
                        const float4 q4 = *reinterpret_cast<const float4*>(Qs + ((wave * WQPW + i) * M + m) * DNP + d0 + d);
                        s[i] = fmaf(q4.x, k0, s[i]); s[i] = fmaf(q4.y, k1, s[i]); s[i] = fmaf(q4.z, k2, s[i]); s[i] = fmaf(q4.w, k3, s[i]);
                    }
                }
            }
            // ---- online softmax of map m, weights to LDS
#pragma unroll
            for (int i = 0; i < WQPW; ++i) {
                const bool vis = lane < nk && rpos[i] >= 0 && j <= rpos[i] && (j >= first_visible(rpos[i], a.window, a.chunks) || j < a.keep);
                float sv = vis ? s[i] * a.scale : -INFINITY;
                if (a.rel && vis) sv += a.rel[(long long)a.bucket_of[min(rpos[i] - j, a.n_dist - 1)] * a.H + rhead[i]];
                if (a.slopes && vis) sv -= slope[i] * (float)(rpos[i] - j);
                if (a.softcap > 0.0f && vis) sv = a.softcap * tanhf(sv / a.softcap);
                const float mn = fmaxf(mx[m][i], wave_max(sv));
                const float ms = mn == -INFINITY ? 0.0f : mn;
                const float p = vis ? expf(sv - ms) : 0.0f;
                const float corr = mx[m][i] == -INFINITY ? 0.0f : expf(mx[m][i] - ms);
                l[m][i] = l[m][i] * corr + wave_sum(p);
                mx[m][i] = mn;
#pragma unroll
                for (int c = 0; c < WMAXC; ++c) acc[m][i][c] *= corr;
                Ps[(m * WROWS + wave * WQPW + i) * WKCH + lane] = p;
            }
        }
        // ---- weighted sums: slabs of WSLAB value columns, lane = column, one slab for all maps
#pragma unroll
        for (int c = 0; c < WMAXC; ++c) {
            const int v0 = c * WSLAB;
            if (v0 < a.dv) {
                const int nvv = min(WSLAB, a.dv - v0);
                __syncthreads();
                {
                    const float* src = a.cache + vbase + v0 + lane;
                    float v[16];
#pragma unroll
                    for (int u = 0; u < 16; ++u) {
                        const int k = wave + 4 * u;
                        v[u] = (k < nk && lane < nvv) ? src[(long long)key_pos(k) * a.row] : 0.0f;
                    }
#pragma unroll
                    for (int u = 0; u < 16; ++u) Sl[(wave + 4 * u) * WSLAB + lane] = v[u];
                }
                __syncthreads();
                for (int k = 0; k < nk; k += 4) {      // (weights and value rows past nk are zero)
                    const float x0 = Sl[k * WSLAB + lane], x1 = Sl[(k + 1) * WSLAB + lane], x2 = Sl[(k + 2) * WSLAB + lane], x3 = Sl[(k + 3) * WSLAB + lane];
#pragma unroll
                    for (int m = 0; m < M; ++m)
#pragma unroll
                        for (int i = 0; i < WQPW; ++i) {
                            const float4 p4 = *reinterpret_cast<const float4*>(Ps + (m * WROWS + wave * WQPW + i) * WKCH + k);
                            acc[m][i][c] = fmaf(p4.x, x0, acc[m][i][c]); acc[m][i][c] = fmaf(p4.y, x1, acc[m][i][c]);
                            acc[m][i][c] = fmaf(p4.z, x2, acc[m][i][c]); acc[m][i][c] = fmaf(p4.w, x3, acc[m][i][c]);
                        }
                }
            }
        }
    }
    // ---- results
#pragma unroll
    for (int i = 0; i < WQPW; ++i) {
        const int rho = row0 + wave * WQPW + i;
        if (rho >= n_rows) continue;
        const int t = rho / R, h = g * R + rho % R;
        if (a.splits > 1) {
#pragma unroll
            for (int m = 0; m < M; ++m) {
                float* st = a.scratch + ((((long long)t * a.H + h) * a.splits + blockIdx.z) * M + m) * (2 + a.dv);
                if (lane == 0) { st[0] = mx[m][i]; st[1] = l[m][i]; }
#pragma unroll
                for (int c = 0; c < WMAXC; ++c)
                    if (c * WSLAB + lane < a.dv) st[2 + c * WSLAB + lane] = acc[m][i][c];
            }
            continue;
        }
        float r[M][WMAXC];
#pragma unroll
        for (int m = 0; m < M; ++m) {
            const float inv = l[m][i] > 0.0f ? 1.0f / l[m][i] : 0.0f;
#pragma unroll
            for (int c = 0; c < WMAXC; ++c) r[m][c] = acc[m][i][c] * inv;
        }
        finish_row<M>(r, lane, a.dv, a.lambda, a.sub_norm, a.eps, a.out_scale, a.out + (long long)t * a.ldo + (long long)h * a.dv,
                      gate_of(a, t, h), a.head_gate ? 0 : 1);
    }
}

// merge of the partial states of one (token, head) row, one wave per row: lane = part for the weights exp(max_s - max) and the sum (splits <= 64), then
// lane = column for the weighted vectors, the parts in order with their loads independent of each other
template <int M>
__global__ __launch_bounds__(64) void window_attention_merge_kernel(const WinArgs a) {
    const int lane = threadIdx.x, row = blockIdx.x;       // row = t * H + h
    float r[M][WMAXC];
#pragma unroll
    for (int m = 0; m < M; ++m) {
        const float* st = a.scratch + ((long long)row * a.splits * M + m) * (2 + a.dv);
        const long long step = (long long)M * (2 + a.dv);
        const float ms = lane < a.splits ? st[lane * step] : -INFINITY;
        const float ls = lane < a.splits ? st[lane * step + 1] : 0.0f;
        const float mm = wave_max(ms);
        const float w = ms == -INFINITY ? 0.0f : expf(ms - mm);
        const float L = wave_sum(w * ls);
#pragma unroll
        for (int c = 0; c < WMAXC; ++c) r[m][c] = 0.0f;
        const int nc = (a.dv + WSLAB - 1) / WSLAB;
        for (int s0 = 0; s0 < a.splits; s0 += 8) {       // eight parts' loads in flight before the first is used
            for (int c = 0; c < nc; ++c) {
                float x[8];
#pragma unroll
                for (int u = 0; u < 8; ++u) x[u] = (s0 + u < a.splits && c * WSLAB + lane < a.dv) ? st[(s0 + u) * step + 2 + c * WSLAB + lane] : 0.0f;
#pragma unroll
                for (int u = 0; u < 8; ++u) {
                    const float ws = __shfl(w, (s0 + u) & 63, 64);
#pragma unroll
                    for (int cc = 0; cc < WMAXC; ++cc)
                        if (cc == c) r[m][cc] = fmaf(ws, x[u], r[m][cc]);
                }
            }
        }
        const float inv = L > 0.0f ? 1.0f / L : 0.0f;
#pragma unroll
        for (int c = 0; c < WMAXC; ++c) r[m][c] *= inv;
    }
    finish_row<M>(r, lane, a.dv, a.lambda, a.sub_norm, a.eps, a.out_scale, a.out + (long long)(row / a.H) * a.ldo + (long long)(row % a.H) * a.dv,
                  gate_of(a, row / a.H, row % a.H), a.head_gate ? 0 : 1);
}

// parts the key chunks of a row tile go round: only when few tiles face many chunks
static int window_splits(int T, int H, int G, int nkeys) {
    const int tiles = ((T * (H / G) + WROWS - 1) / WROWS) * G;
    const int chunks = (nkeys + WKCH - 1) / WKCH + 1;
    if (tiles >= 128 || chunks < 4) return 1;
    int s = 256 / tiles;
    if (s > chunks) s = chunks;
    if (s > 64) s = 64;
    return s < 2 ? 1 : s;
}
static int window_keys(int pos0, int T, int window, int chunks, int keep) {
    const int all = pos0 + T;
    if (chunks && window > 0) return all - (pos0 / window) * window;     // from the start of the first token's chunk
    return window > 0 && (long long)window + T - 1 + keep < all ? window + T - 1 + keep : all;
}

}  // namespace ntk

using namespace ntk;

int ntk_window_prepare(float* cache, int row, float* q, int ldq, const float* k, int ldk, const float* v, int ldv, int H, int G, int maps, int dn, int dv,
                       const ntk_rotary* rot, int pos0, int T, void* stream) {
    return ntk_window_prepare_biased(cache, row, q, ldq, k, ldk, v, ldv, H, G, maps, dn, dv, rot, nullptr, nullptr, nullptr, 0.0f, 1.0, pos0, T, stream);
}

int ntk_window_prepare_biased(float* cache, int row, float* q, int ldq, const float* k, int ldk, const float* v, int ldv, int H, int G, int maps, int dn, int dv,
                              const ntk_rotary* rot, const float* qb, const float* kb, const float* vb, float temp_coef, double temp_every, int pos0, int T,
                              void* stream) {
    ntk_window_prepare_desc d{};
    d.cache = cache; d.row = row; d.q = q; d.ldq = ldq; d.k = k; d.ldk = ldk; d.v = v; d.ldv = ldv; d.H = H; d.G = G; d.maps = maps; d.dn = dn; d.dv = dv; d.rot = rot;
    d.qb = qb; d.kb = kb; d.vb = vb; d.temp_coef = temp_coef; d.temp_every = temp_every; d.pos0 = pos0; d.T = T;
    return ntk_window_prepare_ex(&d, stream);
}

int ntk_window_prepare_ex(const ntk_window_prepare_desc* d, void* stream) {
    if (!d || !d->q || !d->rot || (d->rot->dims > 0 && !d->rot->freq)) return NTK_E_NULL;
    if (d->k ? (!d->cache || !d->v) : (d->v || d->kb || d->vb || d->v_other || d->v_keep || d->k_norm)) return NTK_E_NULL;   // (without k: queries only)
    const ntk_rotary* rot = d->rot;
    if (d->temp_coef != 0.0f && !(d->temp_every > 0.0)) return NTK_E_SHAPE;
    if (d->T < 0 || d->H <= 0 || d->G <= 0 || d->H % d->G || d->maps < 1 || d->dn <= 0 || d->dv <= 0 || d->pos0 < 0) return NTK_E_SHAPE;
    if (rot->dims < 0 || (rot->dims & 1) || rot->dims > d->dn || (rot->layout != NTK_ROT_NEIGHBOURS && rot->layout != NTK_ROT_HALVES)) return NTK_E_SHAPE;
    if (d->ldq < d->H * d->maps * d->dn) return NTK_E_SHAPE;
    if (d->k && (d->row < d->G * (d->maps * d->dn + d->dv) || d->ldk < d->G * d->maps * d->dn || d->ldv < d->G * d->dv)) return NTK_E_SHAPE;
    if ((d->v_other && d->ld_other < d->G * d->dv) || (d->v_keep && d->ld_keep < d->G * d->dv)) return NTK_E_SHAPE;
    if (d->T == 0) return NTK_OK;
    if (rot->dims > 16384) return NTK_E_SHAPE;     // (the angles' cos and sin sit in LDS)
    const PrepareArgs a{d->cache, d->row, d->q, d->ldq, d->k, d->ldk, d->v, d->ldv, d->H * d->maps, d->G * d->maps, d->dn, d->G * d->dv, rot->freq, rot->mag, rot->dims,
                        rot->layout == NTK_ROT_HALVES ? 1 : 0, d->pos0, d->qb, d->kb, d->vb, d->temp_coef, d->temp_every, d->v_other, d->ld_other, d->v_blend, d->v_keep,
                        d->ld_keep, d->q_norm, d->k_norm, d->norm_eps};
    const size_t lds = (size_t)(rot->dims + 2) * sizeof(float);
    if (d->head_norm) {
        if (d->v_other || d->v_keep) return NTK_E_SHAPE;      // (that form does not blend values)
        const int vectors = d->H * d->maps + (d->k ? d->G * d->maps + d->G : 0);
        hipLaunchKernelGGL(window_prepare_heads_kernel, dim3(d->T, (vectors + 3) / 4), dim3(256), 0, resolve_stream(stream), a, d->G);
        return last_launch_status();
    }
    // a normed row is read twice, the second time behind a sum over the workgroup: few tokens (decoding) take workgroups of 1024
    if ((d->q_norm || d->k_norm) && d->T <= 32) hipLaunchKernelGGL(window_prepare_kernel<1024>, dim3(d->T), dim3(1024), lds, resolve_stream(stream), a);
    else hipLaunchKernelGGL(window_prepare_kernel<256>, dim3(d->T), dim3(256), lds, resolve_stream(stream), a);
    return last_launch_status();
}

size_t ntk_window_attention_scratch(int T, int H, int maps, int dv, int nkeys) {
    // rows x splits <= 16 x 256: a launch is only split while it has fewer than 128 row tiles, into at most 256 / tiles (and 64) parts
    const size_t states = std::min<size_t>((size_t)T * H * 64, 4096);
    return nkeys > 0 ? states * maps * (2 + dv) : 0;
}

int ntk_window_attention(const ntk_window_attention_desc* d, void* stream) {
    if (!d || !d->out || !d->q || !d->cache) return NTK_E_NULL;
    if (d->T < 0 || d->H <= 0 || d->G <= 0 || d->H % d->G || d->dn <= 0 || d->dv <= 0 || d->pos0 < 0) return NTK_E_SHAPE;
    if (d->maps != 1 && d->maps != 2) return NTK_E_SHAPE;
    if (d->dv > WMAXC * WSLAB) return NTK_E_SHAPE;
    if (d->row < d->G * (d->maps * d->dn + d->dv) || d->ldq < d->H * d->maps * d->dn || d->ldo < d->H * d->dv) return NTK_E_SHAPE;
    if (d->T == 0) return NTK_OK;
    WinArgs a{};
    a.out = d->out; a.ldo = d->ldo; a.q = d->q; a.ldq = d->ldq; a.cache = d->cache; a.row = d->row; a.H = d->H; a.G = d->G; a.dn = d->dn; a.dv = d->dv;
    a.pos0 = d->pos0; a.T = d->T; a.window = d->window; a.scale = d->scale; a.lambda = d->lambda; a.sub_norm = d->sub_norm; a.eps = d->eps; a.out_scale = d->out_scale;
    if ((d->mask_mode != NTK_MASK_SLIDING && d->mask_mode != NTK_MASK_CHUNKS) || d->softcap < 0.0f) return NTK_E_SHAPE;
    a.chunks = d->mask_mode == NTK_MASK_CHUNKS; a.softcap = d->softcap; a.sink = d->sink;
    if (d->gate && d->ldg < (d->head_gate ? d->H : d->H * d->dv)) return NTK_E_SHAPE;
    a.gate = d->gate; a.ldg = d->ldg; a.head_gate = d->head_gate ? 1 : 0;
    if (d->keep_first < 0 || (d->keep_first > 0 && a.chunks)) return NTK_E_SHAPE;
    a.keep = d->keep_first; a.sinks = d->sinks; a.slopes = d->slopes;
    a.splits = d->scratch ? window_splits(d->T, d->H, d->G, window_keys(d->pos0, d->T, d->window, a.chunks, a.keep)) : 1;
    a.scratch = d->scratch;
    a.rel = d->rel; a.bucket_of = d->bucket_of; a.n_dist = d->n_dist;
    if (a.rel && (!a.bucket_of || a.n_dist <= 0)) return NTK_E_NULL;
    const int DNP = (d->dn + 3) & ~3;
    const size_t lds = ((size_t)WROWS * d->maps * DNP + WKCH * (WSLAB + 1) + (size_t)d->maps * WROWS * WKCH) * sizeof(float);
    if (lds > 150 * 1024) return NTK_E_SHAPE;
    hipStream_t s = resolve_stream(stream);
    const dim3 grid((d->T * (d->H / d->G) + WROWS - 1) / WROWS, d->G, a.splits);
    if (lds > 48 * 1024) {
        static bool raised = false;   // (idempotent: a race sets the same attribute twice)
        if (!raised) {
            NTK_HIP_TRY(hipFuncSetAttribute((const void*)window_attention_kernel<1>, hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024));
            NTK_HIP_TRY(hipFuncSetAttribute((const void*)window_attention_kernel<2>, hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024));
            raised = true;
        }
    }
    if (d->maps == 1) hipLaunchKernelGGL(window_attention_kernel<1>, grid, dim3(256), lds, s, a);
    else hipLaunchKernelGGL(window_attention_kernel<2>, grid, dim3(256), lds, s, a);
    int st = last_launch_status();
    if (st != NTK_OK || a.splits == 1) return st;
    if (d->maps == 1) hipLaunchKernelGGL(window_attention_merge_kernel<1>, dim3(d->T * d->H), dim3(64), 0, s, a);
    else hipLaunchKernelGGL(window_attention_merge_kernel<2>, dim3(d->T * d->H), dim3(64), 0, s, a);
    return last_launch_status();
}
