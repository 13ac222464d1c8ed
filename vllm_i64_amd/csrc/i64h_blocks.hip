// Kernels of libi64hip_dense.so for gated linear recurrences and mixtures of experts (include/i64h_dense.h):
//   gla_gates_kernel   : query activation and bounded forget gate, in place on the projection rows
//   gdn_gates_kernel / gdn_scan_kernel : gated delta rule - unit-vector queries and keys, write strength and decay; the recurrence with the
//                        correction S^T k summed over the DPP row before the write, the read-out after it; a decay per head or per key channel;
//                        without the correction: gated linear attention, with keys of its own or one minus the decay as the key
//   gdn_tile_kernel    : the same recurrence for long runs, tokens staged through LDS
//   route_topk_kernel  : softmax scores (over all entries or the chosen ones) or sigmoid scores, corrected choice, groups of
//                        neighbours, top-k and normalised (or raw) weights, one wave per row (few rows: a workgroup per row)
//   moe_plan_kernel    : (token, choice) pairs grouped by expert: offsets, the token of every grouped row, the row of every pair
//   moe_combine_kernel : weighted sum of the chosen experts' rows, pass-through entries and the shared expert's row
// A row continues the row before it iff slot and position say so; state is taken as empty at position 0.  All arithmetic fp32.
#include "i64h_common.h"
#include "i64h_dense.h"

__device__ __forceinline__ float bl_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }

// ---------------------------------------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void gla_gates_kernel(const i64h_gla_args p) {
    const int64_t t = blockIdx.y;
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= p.heads * p.dim) return;
    float* row = p.P + t * p.ldp;
    if (p.q_act) {
        const float q = row[p.q_off + c];
        row[p.q_off + c] = q * bl_sigmoid(q);
    }
    const float lo = p.lower ? p.lower[c] : 0.0f;
    row[p.f_off + c] = lo + (1.0f - lo) * bl_sigmoid(row[p.f_off + c]);
}

// ---------------------------------------------------------------------------------------------------------------------------
// Gated delta rule.  gdn_gates_kernel: one workgroup per token - a wave per query / key head makes the head a unit vector in place (the
// query also scaled), and the first threads turn the raw gate projections into the write strength and the decay of every head.
__device__ __forceinline__ float bl_softplus(float x) { return x > 20.0f ? x : log1pf(expf(x)); }

__global__ __launch_bounds__(256) void gdn_gates_kernel(const i64h_gdn_args p) {
    const int64_t t = blockIdx.x;
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    float* row = p.X + t * p.ldx;
    if (p.unit_eps >= 0.0f || p.q_scale != 1.0f) {
        for (int u = wid; u < 2 * p.kv_heads; u += 4) {
            const bool isq = u < p.kv_heads;
            float* x = row + (isq ? p.q_off + u * p.dim : p.k_off + (u - p.kv_heads) * p.dim);
            float s = 0.0f;
            for (int d = lane; d < p.dim; d += 64) s += x[d] * x[d];
            s = wave_sum(s);
            float f = p.unit_eps >= 0.0f ? 1.0f / sqrtf(s + p.unit_eps) : 1.0f;
            if (isq) f *= p.q_scale;
            for (int d = lane; d < p.dim; d += 64) x[d] *= f;
        }
    }
    for (int a = threadIdx.x; a < p.heads; a += 256) {
        const float* r = p.R + t * p.ldr;
        p.G[t * 2 * p.heads + a] = bl_sigmoid(r[p.b_off + a]);
        if (p.a_off >= 0) p.G[t * 2 * p.heads + p.heads + a] = expf(-expf(p.A_log[a]) * bl_softplus(r[p.a_off + a] + p.dt_bias[a]));
    }
}

// gdn_scan_kernel: one workgroup per (head, 16 * CPT value columns, run of rows); the 16 lanes of a DPP row share CPT value columns and hold
// KPT key channels of each in registers, a wave has four such rows.  Per token the state decays, the row sums S^T k with DPP
// moves (every lane of the row ends with the sum), the correction along k is written, and a second row sum reads the state out with
// the query - after the write.  No LDS and no barrier, the tokens of a run strictly in their order (the same sums in the same order however
// a prompt is cut); loads run TG tokens ahead in two alternating register sets.  State layout [slot, head, value column, key channel].
// CHD: a decay per head and key channel (F) in the place of one per head.  RULE: the delta rule's correction and write strength, or gated
// linear attention: the token writes k v^T as it is, the read-out is multiplied by q_scale; the keys are the row's own or one minus the decay.
enum { GD_DELTA = 0, GD_KEYS = 1, GD_FORGET = 2 };
// TG is chosen so that two waves fit a SIMD's registers (the loads in flight are most of them); one where every run is a single row.
// A lane's KPT channels: four neighbours in every stripe of 64 (so that 16 lanes read 256 consecutive bytes at a time).
template <int KPT>
__device__ __forceinline__ int gd_channel(int nlane, int k) {
    return KPT >= 4 ? 4 * (nlane + 16 * (k >> 2)) + (k & 3) : nlane * KPT + k;
}
template <int KPT, int CPT, bool CHD, int TG, int RULE>
__global__ __launch_bounds__(256) void gdn_scan_kernel(const i64h_gdn_args p, const int ctiles, const int vec) {
    const int N = p.dim, P = p.vdim;
    const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
    const int nlane = lane & 15, cl = lane >> 4;
    const int a = blockIdx.x / ctiles, seg = blockIdx.y;
    const int kh = a / (p.heads / p.kv_heads);
    const int cbase = (blockIdx.x % ctiles) * 16 * CPT + (w * 4 + cl) * CPT;
    const int64_t r0 = p.seg_start[seg], r1 = p.seg_start[seg + 1];
    if (r1 <= r0) return;
    float S[CPT][KPT];
    float* gS = p.state + ((int64_t)p.slot_ids[r0] * p.heads + a) * P * N;      // + column * N
    const bool fresh = p.positions[r0] == 0;
#pragma unroll
    for (int j = 0; j < CPT; ++j) {
        const bool cok = cbase + j < P;
        const float* src = gS + (int64_t)(cok ? cbase + j : 0) * N;
#pragma unroll
        for (int k = 0; k < KPT; ++k) S[j][k] = 0.0f;
        if (!fresh && cok) {
            if (vec) {
#pragma unroll
                for (int k = 0; k < KPT; k += 4)
                    if (gd_channel<KPT>(nlane, k) < N) {
                        const float4 v = *(const float4*)(src + gd_channel<KPT>(nlane, k));
                        S[j][k] = v.x, S[j][k + 1] = v.y, S[j][k + 2] = v.z, S[j][k + 3] = v.w;
                    }
            } else {
#pragma unroll
                for (int k = 0; k < KPT; ++k)
                    if (gd_channel<KPT>(nlane, k) < N) S[j][k] = src[gd_channel<KPT>(nlane, k)];
            }
        }
    }
    const int qoff = p.q_off + kh * N, koff = p.k_off + kh * N, foff = a * N;
    struct Tok {
        float q[KPT], k[RULE == GD_FORGET ? 1 : KPT], f[CHD ? KPT : 1], v[CPT], beta;
    };
    auto fetch = [&](int64_t t, Tok& u) {
        if (t >= r1) return;
        const float* row = p.X + t * p.ldx;
        if (vec) {      // KPT % 4 == 0 and every slice starts at a multiple of four floats and lies inside the row
#pragma unroll
            for (int k = 0; k < KPT; k += 4) {
                float4 q = make_float4(0, 0, 0, 0), kk = q, f = RULE == GD_FORGET ? make_float4(1, 1, 1, 1) : q;
                if (gd_channel<KPT>(nlane, k) < N) {
                    q = *(const float4*)(row + qoff + gd_channel<KPT>(nlane, k));
                    if (RULE != GD_FORGET) kk = *(const float4*)(row + koff + gd_channel<KPT>(nlane, k));
                    if (CHD) f = *(const float4*)(p.F + t * p.ldf + foff + gd_channel<KPT>(nlane, k));
                }
                u.q[k] = q.x, u.q[k + 1] = q.y, u.q[k + 2] = q.z, u.q[k + 3] = q.w;
                if (RULE != GD_FORGET) u.k[k] = kk.x, u.k[k + 1] = kk.y, u.k[k + 2] = kk.z, u.k[k + 3] = kk.w;
                if (CHD) u.f[k] = f.x, u.f[k + 1] = f.y, u.f[k + 2] = f.z, u.f[k + 3] = f.w;
            }
        } else {
#pragma unroll
            for (int k = 0; k < KPT; ++k) {
                const int c = gd_channel<KPT>(nlane, k);
                const bool ok = c < N;
                u.q[k] = ok ? row[qoff + c] : 0.0f;
                if (RULE != GD_FORGET) u.k[k] = ok ? row[koff + c] : 0.0f;
                if (CHD) u.f[k] = ok ? p.F[t * p.ldf + foff + c] : (RULE == GD_FORGET ? 1.0f : 0.0f);
            }
        }
#pragma unroll
        for (int j = 0; j < CPT; ++j) u.v[j] = cbase + j < P ? row[p.v_off + a * P + cbase + j] : 0.0f;
        if (RULE == GD_DELTA) u.beta = p.G[t * 2 * p.heads + a];
        if (!CHD) u.f[0] = p.G[t * 2 * p.heads + p.heads + a];
    };
    auto step = [&](int64_t t, const Tok& u) {
        if (t >= r1) return;
#pragma unroll
        for (int j = 0; j < CPT; ++j) {
            float part = 0.0f;
            if constexpr (RULE == GD_DELTA) {
                float seen = 0.0f;
#pragma unroll
                for (int k = 0; k < KPT; ++k) {
                    S[j][k] *= u.f[CHD ? k : 0];
                    seen = fmaf(S[j][k], u.k[k], seen);
                }
                seen = group_sum(seen, 16);
                const float d = u.beta * (u.v[j] - seen);
#pragma unroll
                for (int k = 0; k < KPT; ++k) {
                    S[j][k] = fmaf(u.k[k], d, S[j][k]);
                    part = fmaf(S[j][k], u.q[k], part);
                }
            } else {
#pragma unroll
                for (int k = 0; k < KPT; ++k) {
                    const float kk = RULE == GD_FORGET ? 1.0f - u.f[CHD ? k : 0] : u.k[RULE == GD_FORGET ? 0 : k];
                    S[j][k] = fmaf(u.f[CHD ? k : 0], S[j][k], kk * u.v[j]);
                    part = fmaf(S[j][k], u.q[k], part);
                }
            }
            part = group_sum(part, 16);
            if (nlane == 0 && cbase + j < P) p.out[t * p.ldo + a * P + cbase + j] = RULE == GD_DELTA ? part : part * p.q_scale;
        }
    };
    Tok A[TG], B[TG];
#pragma unroll
    for (int i = 0; i < TG; ++i) fetch(r0 + i, A[i]);
    for (int64_t t = r0; t < r1; t += 2 * TG) {
#pragma unroll
        for (int i = 0; i < TG; ++i) fetch(t + TG + i, B[i]);
#pragma unroll
        for (int i = 0; i < TG; ++i) step(t + i, A[i]);
#pragma unroll
        for (int i = 0; i < TG; ++i) fetch(t + 2 * TG + i, A[i]);
#pragma unroll
        for (int i = 0; i < TG; ++i) step(t + TG + i, B[i]);
    }
#pragma unroll
    for (int j = 0; j < CPT; ++j) {
        if (cbase + j >= P) continue;
        float* dst = gS + (int64_t)(cbase + j) * N;
        if (vec) {
#pragma unroll
            for (int k = 0; k < KPT; k += 4)
                if (gd_channel<KPT>(nlane, k) < N) *(float4*)(dst + gd_channel<KPT>(nlane, k)) = make_float4(S[j][k], S[j][k + 1], S[j][k + 2], S[j][k + 3]);
        } else {
#pragma unroll
            for (int k = 0; k < KPT; ++k)
                if (gd_channel<KPT>(nlane, k) < N) dst[gd_channel<KPT>(nlane, k)] = S[j][k];
        }
    }
}

// gdn_tile_kernel: the same recurrence, bit for bit, for runs of many rows.  What every wave of a workgroup reads of a token (query, key,
// decays) is loaded once per workgroup, TT tokens at a time, into one of two LDS tiles while the other one is computed: the loads of a
// tile have the arithmetic of a whole tile to arrive, and the waves read 16 bytes per lane from LDS one token ahead.  Needs 16-byte rows.
template <int KPT, int CPT, bool CHD, int RULE>
__global__ __launch_bounds__(256) void gdn_tile_kernel(const i64h_gdn_args p, const int ctiles) {
    static_assert(KPT % 4 == 0, "whole 16-byte slices per lane");
    constexpr int TT = KPT > 8 ? 8 : 16;      // tokens per tile
    constexpr int NP = 16 * KPT, PARTS = CHD && RULE != GD_FORGET ? 3 : 2, LPP = TT * NP / 4 / 256, WC = 16 * CPT;     // LPP: 16-byte loads per thread and part
    constexpr int VPT = (TT * WC + 255) / 256;
    __shared__ __attribute__((aligned(16))) float sX[2][PARTS][TT][NP];
    __shared__ float sV[2][TT][WC];
    __shared__ float sG[2][TT][2];      // write strength, decay per head
    const int N = p.dim, P = p.vdim;
    const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
    const int nlane = lane & 15, cl = lane >> 4;
    const int a = blockIdx.x / ctiles, seg = blockIdx.y;
    const int kh = a / (p.heads / p.kv_heads);
    const int wg0 = (blockIdx.x % ctiles) * WC, cw = (w * 4 + cl) * CPT, cbase = wg0 + cw;
    const int64_t r0 = p.seg_start[seg], r1 = p.seg_start[seg + 1];
    if (r1 <= r0) return;      // (the whole workgroup)
    float S[CPT][KPT];
    float* gS = p.state + ((int64_t)p.slot_ids[r0] * p.heads + a) * P * N;
    const bool fresh = p.positions[r0] == 0;
#pragma unroll
    for (int j = 0; j < CPT; ++j) {
        const bool cok = cbase + j < P;
        const float* src = gS + (int64_t)(cok ? cbase + j : 0) * N;
#pragma unroll
        for (int k = 0; k < KPT; k += 4) {
            const int c = gd_channel<KPT>(nlane, k);
            float4 v = make_float4(0, 0, 0, 0);
            if (!fresh && cok && c < N) v = *(const float4*)(src + c);
            S[j][k] = v.x, S[j][k + 1] = v.y, S[j][k + 2] = v.z, S[j][k + 3] = v.w;
        }
    }
    float4 st[PARTS][LPP];
    float sv[VPT], sg = 0.0f;
    auto gload = [&](int64_t t0) {
#pragma unroll
        for (int u = 0; u < LPP; ++u) {
            const int e = tid + 256 * u, c = (e % (NP / 4)) * 4;
            const int64_t t = t0 + e / (NP / 4);
            const bool ok = t < r1 && c < N;
            const float* row = p.X + t * p.ldx;
            st[0][u] = ok ? *(const float4*)(row + p.q_off + kh * N + c) : make_float4(0, 0, 0, 0);
            if (RULE != GD_FORGET) st[1][u] = ok ? *(const float4*)(row + p.k_off + kh * N + c) : make_float4(0, 0, 0, 0);
            const float pad = RULE == GD_FORGET ? 1.0f : 0.0f;
            if (CHD) st[PARTS - 1][u] = ok ? *(const float4*)(p.F + t * p.ldf + a * N + c) : make_float4(pad, pad, pad, pad);
        }
#pragma unroll
        for (int u = 0; u < VPT; ++u) {
            const int e = tid + 256 * u, c = wg0 + e % WC;
            const int64_t t = t0 + e / WC;
            sv[u] = (t < r1 && c < P) ? p.X[t * p.ldx + p.v_off + a * P + c] : 0.0f;
        }
        if (tid < 2 * TT) {
            const int64_t t = t0 + (tid >> 1);
            sg = (t < r1 && (RULE == GD_DELTA || (tid & 1)) && !(CHD && (tid & 1))) ? p.G[t * 2 * p.heads + (tid & 1) * p.heads + a] : 0.0f;
        }
    };
    auto lstore = [&](int b) {
#pragma unroll
        for (int u = 0; u < LPP; ++u) {
            const int e = tid + 256 * u;
#pragma unroll
            for (int x = 0; x < PARTS; ++x) *(float4*)&sX[b][x][e / (NP / 4)][(e % (NP / 4)) * 4] = st[x][u];
        }
#pragma unroll
        for (int u = 0; u < VPT; ++u)
            if (tid + 256 * u < TT * WC) sV[b][(tid + 256 * u) / WC][(tid + 256 * u) % WC] = sv[u];
        if (tid < 2 * TT) sG[b][tid >> 1][tid & 1] = sg;
    };
    struct Tok {
        float q[KPT], k[RULE == GD_FORGET ? 1 : KPT], f[CHD ? KPT : 1], v[CPT], beta;
    };
    auto fetch = [&](int b, int i, Tok& u) {
#pragma unroll
        for (int k = 0; k < KPT; k += 4) {
            const int c = gd_channel<KPT>(nlane, k);
            const float4 q = *(const float4*)&sX[b][0][i][c];
            u.q[k] = q.x, u.q[k + 1] = q.y, u.q[k + 2] = q.z, u.q[k + 3] = q.w;
            if (RULE != GD_FORGET) {
                const float4 kk = *(const float4*)&sX[b][1][i][c];
                u.k[k] = kk.x, u.k[k + 1] = kk.y, u.k[k + 2] = kk.z, u.k[k + 3] = kk.w;
            }
            if (CHD) {
                const float4 f = *(const float4*)&sX[b][PARTS - 1][i][c];
                u.f[k] = f.x, u.f[k + 1] = f.y, u.f[k + 2] = f.z, u.f[k + 3] = f.w;
            }
        }
#pragma unroll
        for (int j = 0; j < CPT; ++j) u.v[j] = sV[b][i][cw + j];
        u.beta = sG[b][i][0];
        if (!CHD) u.f[0] = sG[b][i][1];
    };
    auto step = [&](int64_t t, const Tok& u) {
        float seen[CPT], part[CPT], d[CPT];
        if constexpr (RULE != GD_DELTA) {
#pragma unroll
            for (int j = 0; j < CPT; ++j) {
                part[j] = 0.0f;
#pragma unroll
                for (int k = 0; k < KPT; ++k) {
                    const float kk = RULE == GD_FORGET ? 1.0f - u.f[CHD ? k : 0] : u.k[RULE == GD_FORGET ? 0 : k];
                    S[j][k] = fmaf(u.f[CHD ? k : 0], S[j][k], kk * u.v[j]);
                    part[j] = fmaf(S[j][k], u.q[k], part[j]);
                }
            }
#pragma unroll
            for (int j = 0; j < CPT; ++j) {
                const float o = group_sum(part[j], 16);
                if (nlane == 0 && cbase + j < P) p.out[t * p.ldo + a * P + cbase + j] = o * p.q_scale;
            }
        } else {
#pragma unroll
            for (int j = 0; j < CPT; ++j) {
                seen[j] = 0.0f;
#pragma unroll
                for (int k = 0; k < KPT; ++k) {
                    S[j][k] *= u.f[CHD ? k : 0];
                    seen[j] = fmaf(S[j][k], u.k[k], seen[j]);
                }
            }
#pragma unroll
            for (int j = 0; j < CPT; ++j) d[j] = u.beta * (u.v[j] - group_sum(seen[j], 16));
#pragma unroll
            for (int j = 0; j < CPT; ++j) {
                part[j] = 0.0f;
#pragma unroll
                for (int k = 0; k < KPT; ++k) {
                    S[j][k] = fmaf(u.k[k], d[j], S[j][k]);
                    part[j] = fmaf(S[j][k], u.q[k], part[j]);
                }
            }
#pragma unroll
            for (int j = 0; j < CPT; ++j) {
                const float o = group_sum(part[j], 16);
                if (nlane == 0 && cbase + j < P) p.out[t * p.ldo + a * P + cbase + j] = o;
            }
        }
    };
    gload(r0);
    lstore(0);
    __syncthreads();
    int b = 0;
    for (int64_t t0 = r0; t0 < r1; t0 += TT, b ^= 1) {
        const int cnt = (int)min((int64_t)TT, r1 - t0);
        const bool more = t0 + TT < r1;
        if (more) gload(t0 + TT);
        Tok A, B;
        fetch(b, 0, A);
        for (int i = 0; i < cnt; i += 2) {
            fetch(b, i + 1, B);            // (a tile has TT rows, an even number: zeros past the run's end)
            step(t0 + i, A);
            if (i + 1 < cnt) {
                if (i + 2 < cnt) fetch(b, i + 2, A);
                step(t0 + i + 1, B);
            }
        }
        if (more) lstore(b ^ 1);
        __syncthreads();
    }
#pragma unroll
    for (int j = 0; j < CPT; ++j) {
        if (cbase + j >= P) continue;
        float* dst = gS + (int64_t)(cbase + j) * N;
#pragma unroll
        for (int k = 0; k < KPT; k += 4) {
            const int c = gd_channel<KPT>(nlane, k);
            if (c < N) *(float4*)(dst + c) = make_float4(S[j][k], S[j][k + 1], S[j][k + 2], S[j][k + 3]);
        }
    }
}

// ---------------------------------------------------------------------------------------------------------------------------
// the lane that holds the largest value, ties to the lower index; (value, index) pairs with index < 0 do not take part
__device__ __forceinline__ int bl_wave_argmax(float v, int idx, float& best) {
    best = wave_max(idx >= 0 ? v : -INFINITY);
    const int cand = (idx >= 0 && v == best) ? idx : 0x7fffffff;
    return -wave_max_i(-cand);
}

#define RT_MAX_TOP 32
#define RT_SPLIT_ROWS 512      // launches of at most so many rows give every row a workgroup
// SPLIT: a workgroup per row - its four waves share the columns of the router's products, the first one goes on with their sums (few
// rows: one wave's chain of loads is what a launch would wait for).
template <bool SPLIT>
__global__ __launch_bounds__(256) void route_topk_kernel(const i64h_route_args p) {
    extern __shared__ float rt_lds[];   // per wave: [E] scores, [E] choice values, [groups] group flags; SPLIT: once, and [4][E + 1] partial products
    const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6;
    const int64_t t = SPLIT ? (int64_t)blockIdx.x : (int64_t)blockIdx.x * 4 + wid;
    if (t >= p.n) return;     // (a whole wave leaves; without SPLIT there is no workgroup barrier below)
    const int E = p.E, G = p.groups > 1 ? p.groups : 1, gsz = E / G;
    // volatile: lanes read what another lane of the wave wrote (one wave: program order is enough, no barrier)
    volatile float* sc = rt_lds + (SPLIT ? 0 : (size_t)wid * (2 * E + G));
    float* part = rt_lds + 2 * E + G;
    volatile float* ch = sc + E;
    volatile float* gflag = ch + E;
    if (p.W) {      // the router's own products: eight entries at a time, every lane a share of the columns, fp32 throughout
        const float* h = p.h + t * p.ldh;
        const uint16_t* W = (const uint16_t*)p.W;
        const int K = p.K;
        const bool vec = (K & 3) == 0 && (p.ldh & 3) == 0 && ((uintptr_t)p.h & 15) == 0 && ((uintptr_t)p.W & 7) == 0;
        const int rows = p.gate_out ? E + 1 : E;
        for (int e0 = 0; e0 < rows; e0 += 8) {
            float acc[8] = {0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f, 0.0f};
            if (vec) {
                for (int k = (SPLIT ? threadIdx.x : lane) * 4; k < K; k += SPLIT ? 1024 : 256) {
                    const float4 x = *(const float4*)(h + k);
#pragma unroll
                    for (int j = 0; j < 8; ++j) {
                        if (e0 + j < rows) {
                            const uint2 w = *(const uint2*)(W + (int64_t)(e0 + j) * K + k);
                            acc[j] = fmaf(x.x, __uint_as_float(w.x << 16), acc[j]);
                            acc[j] = fmaf(x.y, __uint_as_float(w.x & 0xffff0000u), acc[j]);
                            acc[j] = fmaf(x.z, __uint_as_float(w.y << 16), acc[j]);
                            acc[j] = fmaf(x.w, __uint_as_float(w.y & 0xffff0000u), acc[j]);
                        }
                    }
                }
            } else {
                for (int k = SPLIT ? threadIdx.x : lane; k < K; k += SPLIT ? 256 : 64) {
                    const float x = h[k];
#pragma unroll
                    for (int j = 0; j < 8; ++j)
                        if (e0 + j < rows) acc[j] = fmaf(x, __uint_as_float((uint32_t)W[(int64_t)(e0 + j) * K + k] << 16), acc[j]);
                }
            }
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const float v = wave_sum(acc[j]);
                if (SPLIT) {
                    if (lane == 0 && e0 + j < rows) part[wid * rows + e0 + j] = v;
                    continue;
                }
                if (lane == 0 && e0 + j < E) ch[e0 + j] = p.bias ? v + p.bias[e0 + j] : v;
                if (lane == 0 && e0 + j == E && p.gate_out) p.gate_out[t] = bl_sigmoid(v);
            }
        }
        if (SPLIT) {
            __syncthreads();
            if (wid > 0) return;
            for (int e = lane; e < rows; e += 64) {
                const float v = (part[e] + part[rows + e]) + (part[2 * rows + e] + part[3 * rows + e]);
                if (e < E) ch[e] = p.bias ? v + p.bias[e] : v;
                else p.gate_out[t] = bl_sigmoid(v);
            }
        }
    } else {
        const float* z = p.logits + t * p.ld;
        for (int e = lane; e < E; e += 64) ch[e] = p.bias ? z[e] + p.bias[e] : z[e];
    }
    if (p.sigmoid_scores) {     // scores of their own, in the logits' order: the choice falls on the logits unless it is corrected
        for (int e = lane; e < E; e += 64) {
            const float s = bl_sigmoid(ch[e]);
            sc[e] = s;
            if (p.correction) ch[e] = s + p.correction[e];
        }
    } else if (p.chosen_softmax) {     // the choice falls on the logits themselves
        for (int e = lane; e < E; e += 64) {
            const float s = ch[e];
            sc[e] = s;
            if (p.correction) ch[e] = s + p.correction[e];
        }
    } else {
        float mx = -INFINITY;
        for (int e = lane; e < E; e += 64) mx = fmaxf(mx, ch[e]);
        mx = wave_max(mx);
        float sum = 0.0f;
        for (int e = lane; e < E; e += 64) {
            const float v = expf(ch[e] - mx);
            sc[e] = v;
            sum += v;
        }
        sum = wave_sum(sum);
        for (int e = lane; e < E; e += 64) {
            const float s = sc[e] / sum;
            sc[e] = s;
            ch[e] = p.correction ? s + p.correction[e] : s;
        }
    }
    if (G > 1) {   // a group's score: its largest choice value; the `keep` best groups stay, the entries of the others cannot be chosen
        for (int g = lane; g < G; g += 64) {
            float b = -INFINITY;
            for (int i = 0; i < gsz; ++i) b = fmaxf(b, ch[g * gsz + i]);
            gflag[g] = b;
        }
        // (LDS traffic of one wave needs program order only)
        for (int r = 0; r < p.keep; ++r) {
            float bv = -INFINITY;
            int bi = -1;
            for (int g = lane; g < G; g += 64) {
                const float v = gflag[g];
                if (!(v != v) && v != INFINITY && (bi < 0 || v > bv)) bv = v, bi = g;     // +inf marks a group already kept
            }
            float best;
            const int pick = bl_wave_argmax(bv, bi, best);
            if (pick != 0x7fffffff && lane == 0) gflag[pick] = INFINITY;
        }
        for (int e = lane; e < E; e += 64)
            if (gflag[e / gsz] != INFINITY) ch[e] = -INFINITY;
    }
    float wsum = 0.0f;
    float mine_w = 0.0f;      // lane k keeps the k-th choice
    int mine_i = 0;
    for (int k = 0; k < p.top; ++k) {
        float bv = -INFINITY;
        int bi = -1;
        for (int e = lane; e < E; e += 64) {
            const float v = ch[e];
            if (v == v && (bi < 0 || v > bv)) bv = v, bi = e;
        }
        float best;
        int pick = bl_wave_argmax(bv, bi, best);
        if (pick == 0x7fffffff) pick = 0;
        const float s = sc[pick];
        wsum += s;
        if (lane == k) mine_w = s, mine_i = pick;
        if (lane == 0) ch[pick] = __builtin_nanf("");     // taken: out of every later comparison
    }
    if (p.chosen_softmax) {     // ... and the weights are the softmax over the chosen ones
        const float top1 = wave_max(lane < p.top ? mine_w : -INFINITY);
        mine_w = lane < p.top ? expf(mine_w - top1) : 0.0f;
        wsum = wave_sum(mine_w);
    }
    if (lane < p.top) {
        p.idx[t * p.top + lane] = mine_i;
        p.wgt[t * p.top + lane] = (p.raw_weights ? mine_w : mine_w / (wsum + 1e-20f)) * p.scale;
    }
}

// ---------------------------------------------------------------------------------------------------------------------------
__global__ __launch_bounds__(1024) void moe_plan_kernel(const i64h_moe_plan_args p) {
    extern __shared__ int pl_lds[];   // [experts + 1] counts, then offsets; [experts] cursors
    int* cnt = pl_lds;
    int* cur = pl_lds + p.experts + 1;
    const int tid = threadIdx.x;
    const int64_t pairs = p.n * p.top;
    for (int e = tid; e <= p.experts; e += 1024) cnt[e] = 0;
    __syncthreads();
    for (int64_t i = tid; i < pairs; i += 1024) {
        const int e = p.idx[i];
        if (e >= 0 && e < p.experts) atomicAdd(&cnt[e], 1);
    }
    __syncthreads();
    if (tid == 0) {
        int run = 0;
        for (int e = 0; e < p.experts; ++e) {
            const int c = cnt[e];
            cnt[e] = run;
            cur[e] = run;
            run += c;
        }
        cnt[p.experts] = run;
    }
    __syncthreads();
    for (int e = tid; e <= p.experts; e += 1024) p.group_off[e] = cnt[e];
    for (int64_t i = tid; i < pairs; i += 1024) {
        const int e = p.idx[i];
        int r = -1;
        if (e >= 0 && e < p.experts) {
            r = atomicAdd(&cur[e], 1);
            p.pair_token[r] = (int)(i / p.top);
            if (p.pair_wgt) p.pair_wgt[r] = p.wgt[i];
        }
        p.pair_row[i] = r;
    }
}

__global__ __launch_bounds__(256) void moe_combine_kernel(const i64h_moe_combine_args p) {
    const int64_t t = blockIdx.x;
    const int W = p.W;
    for (int c = threadIdx.x; c < W; c += 256) {
        float a = 0.0f;
        for (int k = 0; k < p.top; ++k) {
            const int r = p.pair_row[t * p.top + k];
            const float v = r >= 0 ? p.Y[(int64_t)r * W + c] : p.h[t * W + c];
            a += p.wgt ? p.wgt[t * p.top + k] * v : v;
        }
        if (p.shared) a += p.shared_gate ? p.shared_gate[t] * p.shared[t * W + c] : p.shared[t * W + c];
        p.out[t * W + c] = a;
    }
}

// ---------------------------------------------------------------------------------------------------------------------------
extern "C" {

static int gla_check(const i64h_gla_args& d, const char* what) {
    I64H_CHECK_ARG(d.heads > 0 && d.dim > 0 && d.vdim > 0 && d.n >= 0, "%s: heads %d, dim %d, vdim %d", what, d.heads, d.dim, d.vdim);
    I64H_CHECK_ARG(d.P && d.q_off >= 0 && d.f_off >= 0 && d.v_off >= 0, "%s: null operand or negative column", what);
    return 0;
}

int i64h_gla_gates(const i64h_gla_args* dp, void* stream) {
    I64H_CHECK_ARG(dp != nullptr, "gla_gates: no descriptor");
    const i64h_gla_args& d = *dp;
    if (gla_check(d, "gla_gates")) return 1;
    I64H_CHECK_ARG(d.n <= 65535, "gla_gates: %lld rows in one launch (at most 65535)", (long long)d.n);
    if (d.n == 0) return 0;
    hipLaunchKernelGGL(gla_gates_kernel, dim3((unsigned)((d.heads * d.dim + 255) / 256), (unsigned)d.n), dim3(256), 0, (hipStream_t)stream, d);
    I64H_CHECK_LAUNCH();
    return 0;
}

static int gdn_check(const i64h_gdn_args& d, const char* what) {
    I64H_CHECK_ARG(d.heads > 0 && d.kv_heads > 0 && d.heads % d.kv_heads == 0 && d.dim > 0 && d.vdim > 0 && d.n >= 0, "%s: heads %d, query / key heads %d, dim %d, vdim %d",
                   what, d.heads, d.kv_heads, d.dim, d.vdim);
    I64H_CHECK_ARG(d.X && d.q_off >= 0 && d.k_off >= 0 && d.v_off >= 0, "%s: null operand or negative column", what);
    return 0;
}

int i64h_gdn_gates(const i64h_gdn_args* dp, void* stream) {
    I64H_CHECK_ARG(dp != nullptr, "gdn_gates: no descriptor");
    const i64h_gdn_args& d = *dp;
    if (gdn_check(d, "gdn_gates")) return 1;
    I64H_CHECK_ARG(d.G && d.R && d.b_off >= 0 && (d.a_off < 0 || (d.A_log && d.dt_bias)), "gdn_gates: null operand or negative column");
    if (d.n == 0) return 0;
    hipLaunchKernelGGL(gdn_gates_kernel, dim3((unsigned)d.n), dim3(256), 0, (hipStream_t)stream, d);
    I64H_CHECK_LAUNCH();
    return 0;
}

static int g_gdn_form = 0;
int i64h_set_gdn_scan_form(int32_t form) {
    I64H_CHECK_ARG(form >= 0 && form <= 4, "gdn_scan: form %d", form);
    g_gdn_form = form;
    return 0;
}

// the recurrence's launch, with the delta rule's correction or (a decay per key channel, every head its own keys) without it
extern "C++" {
template <int RULE>
static int gdn_launch(const i64h_gdn_args& d, void* stream) {
    const int kpt = (d.dim + 15) / 16;
    auto vec_ok = [&](int K) {
        return K % 4 == 0 && d.dim % 4 == 0 && d.ldx % 4 == 0 && d.q_off % 4 == 0 && d.k_off % 4 == 0 && (uintptr_t)d.X % 16 == 0 && (uintptr_t)d.state % 16 == 0 &&
               (!d.F || (d.ldf % 4 == 0 && (uintptr_t)d.F % 16 == 0));
    };
    const int kround = kpt <= 4 ? 4 : (kpt <= 8 ? 8 : 16);
    if (g_gdn_form != 1 && vec_ok(kround) && (g_gdn_form > 1 || d.n >= 8 * (int64_t)d.nseg)) {
        // one value column per lane while that is at most two workgroups per CU, two (fewer reads of the tile) beyond
        const int cpt = g_gdn_form > 1 ? (g_gdn_form == 4 ? 4 : g_gdn_form - 1) : ((int64_t)d.heads * ((d.vdim + 15) / 16) * d.nseg <= 512 ? 1 : 2);
        const int ctiles = (d.vdim + 16 * cpt - 1) / (16 * cpt);
        const dim3 grid((unsigned)(d.heads * ctiles), (unsigned)d.nseg);
        auto launch = [&](auto kern) { hipLaunchKernelGGL(kern, grid, dim3(256), 0, (hipStream_t)stream, d, ctiles); };
#define GDN_TILE(C, CHD)                                            \
    if (kround == 4) launch(gdn_tile_kernel<4, C, CHD, RULE>);      \
    else if (kround == 8) launch(gdn_tile_kernel<8, C, CHD, RULE>); \
    else launch(gdn_tile_kernel<16, C, CHD, RULE>);
        if (RULE != GD_DELTA || d.F) {
            if (cpt == 1) { GDN_TILE(1, true) } else if (cpt == 2) { GDN_TILE(2, true) } else { GDN_TILE(4, true) }
        } else if constexpr (RULE == GD_DELTA) {
            if (cpt == 1) { GDN_TILE(1, false) } else if (cpt == 2) { GDN_TILE(2, false) } else { GDN_TILE(4, false) }
        }
#undef GDN_TILE
        I64H_CHECK_LAUNCH();
        return 0;
    }
    // columns per lane: query and key are loaded once for both - unless the launch would then leave most of the chip idle
    // (two columns also give the two row sums of a token independent work to overlap: measured faster from 256 workgroups on)
    const int cpt = (d.vdim > 16 && (int64_t)d.heads * ((d.vdim + 31) / 32) * d.nseg >= 256) ? 2 : 1;
    const int ctiles = (d.vdim + 16 * cpt - 1) / (16 * cpt);
    const dim3 grid((unsigned)(d.heads * ctiles), (unsigned)d.nseg);
    auto launch = [&](auto kern, int K) {
        const int vec = vec_ok(K);
        hipLaunchKernelGGL(kern, grid, dim3(256), 0, (hipStream_t)stream, d, ctiles, vec);
    };
#define GDN_PICK(C, CHD, ONE)                                                                    \
    if (kpt <= 1) launch(gdn_scan_kernel<1, C, CHD, ONE ? 1 : 4, RULE>, 1);                       \
    else if (kpt <= 2) launch(gdn_scan_kernel<2, C, CHD, ONE ? 1 : 4, RULE>, 2);                  \
    else if (kpt <= 4) launch(gdn_scan_kernel<4, C, CHD, ONE ? 1 : 4, RULE>, 4);                  \
    else if (kpt <= 8) launch(gdn_scan_kernel<8, C, CHD, ONE ? 1 : (CHD ? 2 : 4), RULE>, 8);      \
    else launch(gdn_scan_kernel<16, C, CHD, ONE ? 1 : (CHD ? 1 : 2), RULE>, 16);
#define GDN_PICK2(C, CHD) \
    if (d.nseg == d.n) { GDN_PICK(C, CHD, true) } else { GDN_PICK(C, CHD, false) }
    if (RULE != GD_DELTA || d.F) {
        if (cpt == 2) { GDN_PICK2(2, true) } else { GDN_PICK2(1, true) }
    } else if constexpr (RULE == GD_DELTA) {
        if (cpt == 2) { GDN_PICK2(2, false) } else { GDN_PICK2(1, false) }
    }
#undef GDN_PICK2
#undef GDN_PICK
    I64H_CHECK_LAUNCH();
    return 0;
}
}

int i64h_gdn_scan(const i64h_gdn_args* dp, void* stream) {
    I64H_CHECK_ARG(dp != nullptr, "gdn_scan: no descriptor");
    const i64h_gdn_args& d = *dp;
    if (gdn_check(d, "gdn_scan")) return 1;
    I64H_CHECK_ARG(d.G && d.seg_start && d.positions && d.slot_ids && d.state && d.out, "gdn_scan: null operand");
    I64H_CHECK_ARG(d.dim <= 16 * 16, "gdn_scan: dim %d above 256", d.dim);
    I64H_CHECK_ARG(d.nseg <= 65535, "gdn_scan: %d runs in one launch", d.nseg);
    if (d.nseg <= 0 || d.n == 0) return 0;
    return gdn_launch<GD_DELTA>(d, stream);
}

int i64h_gla_scan(const i64h_gla_args* dp, void* stream) {
    I64H_CHECK_ARG(dp != nullptr, "gla_scan: no descriptor");
    const i64h_gla_args& d = *dp;
    if (gla_check(d, "gla_scan")) return 1;
    I64H_CHECK_ARG(d.seg_start && d.positions && d.slot_ids && d.state && d.out, "gla_scan: null operand");
    I64H_CHECK_ARG(d.dim <= 16 * 16, "gla_scan: dim %d above 256", d.dim);
    I64H_CHECK_ARG(d.nseg <= 65535, "gla_scan: %d runs in one launch", d.nseg);
    I64H_CHECK_ARG(!d.F || d.ldf >= d.f_off + (int64_t)d.heads * d.dim, "gla_scan: the decays' rows are shorter than their columns");
    if (d.nseg <= 0 || d.n == 0) return 0;
    i64h_gdn_args a = {};
    a.X = d.P, a.ldx = d.ldp, a.q_off = d.q_off, a.k_off = d.k_off >= 0 ? d.k_off : 0, a.v_off = d.v_off, a.heads = a.kv_heads = d.heads, a.dim = d.dim, a.vdim = d.vdim;
    a.F = (d.F ? d.F : d.P) + d.f_off, a.ldf = d.F ? d.ldf : d.ldp, a.q_scale = d.q_scale, a.seg_start = d.seg_start, a.nseg = d.nseg;
    a.positions = d.positions, a.slot_ids = d.slot_ids, a.state = d.state, a.out = d.out, a.ldo = d.ldo, a.n = d.n;
    return d.k_off >= 0 ? gdn_launch<GD_KEYS>(a, stream) : gdn_launch<GD_FORGET>(a, stream);
}

int i64h_route_topk(const i64h_route_args* dp, void* stream) {
    I64H_CHECK_ARG(dp != nullptr, "route_topk: no descriptor");
    const i64h_route_args& d = *dp;
    I64H_CHECK_ARG(d.E > 0 && d.E <= 1024 && d.top > 0 && d.top <= RT_MAX_TOP && d.top <= d.E, "route_topk: %d entries (at most 1024), top %d (at most %d)", d.E, d.top, RT_MAX_TOP);
    I64H_CHECK_ARG(d.groups <= 1 || (d.E % d.groups == 0 && d.keep >= 1 && d.keep <= d.groups), "route_topk: %d entries in %d groups, %d kept", d.E, d.groups, d.keep);
    I64H_CHECK_ARG(!d.sigmoid_scores || !d.chosen_softmax, "route_topk: sigmoid scores, or the softmax over the chosen logits");
    I64H_CHECK_ARG(!d.gate_out || d.W, "route_topk: the gate's row lies behind the router's rows");
    I64H_CHECK_ARG(d.groups <= 1 || d.keep * (d.E / d.groups) >= d.top, "route_topk: %d kept groups of %d entries hold fewer than top %d", d.keep, d.E / (d.groups > 0 ? d.groups : 1), d.top);
    I64H_CHECK_ARG(d.idx && d.wgt && ((d.logits && d.ld >= d.E) || (d.W && d.h && d.K > 0 && d.ldh >= d.K)), "route_topk: null operand or row stride below the row");
    if (d.n == 0) return 0;
    const size_t own = (size_t)(2 * d.E + (d.groups > 1 ? d.groups : 1));
    if (d.W && d.n <= RT_SPLIT_ROWS)
        hipLaunchKernelGGL(route_topk_kernel<true>, dim3((unsigned)d.n), dim3(256), (own + 4 * (size_t)(d.E + 1)) * 4, (hipStream_t)stream, d);
    else
        hipLaunchKernelGGL(route_topk_kernel<false>, dim3((unsigned)((d.n + 3) / 4)), dim3(256), 4 * own * 4, (hipStream_t)stream, d);
    I64H_CHECK_LAUNCH();
    return 0;
}

int i64h_moe_plan(const i64h_moe_plan_args* dp, void* stream) {
    I64H_CHECK_ARG(dp != nullptr, "moe_plan: no descriptor");
    const i64h_moe_plan_args& d = *dp;
    I64H_CHECK_ARG(d.experts > 0 && d.experts <= 4096 && d.top > 0 && d.n >= 0, "moe_plan: %d experts (at most 4096), top %d", d.experts, d.top);
    I64H_CHECK_ARG(d.idx && d.group_off && d.pair_token && d.pair_row, "moe_plan: null operand");
    I64H_CHECK_ARG(d.n * d.top < (1ll << 31), "moe_plan: too many pairs");
    I64H_CHECK_ARG(!d.pair_wgt || d.wgt, "moe_plan: weights per row come from the weights per choice");
    hipLaunchKernelGGL(moe_plan_kernel, dim3(1), dim3(1024), (size_t)(2 * d.experts + 1) * 4, (hipStream_t)stream, d);
    I64H_CHECK_LAUNCH();
    return 0;
}

int i64h_moe_combine(const i64h_moe_combine_args* dp, void* stream) {
    I64H_CHECK_ARG(dp != nullptr, "moe_combine: no descriptor");
    const i64h_moe_combine_args& d = *dp;
    I64H_CHECK_ARG(d.top > 0 && d.W > 0 && d.n >= 0, "moe_combine: top %d, width %d", d.top, d.W);
    I64H_CHECK_ARG(d.Y && d.pair_row && d.h && d.out, "moe_combine: null operand");
    if (d.n == 0) return 0;
    hipLaunchKernelGGL(moe_combine_kernel, dim3((unsigned)d.n), dim3(256), 0, (hipStream_t)stream, d);
    I64H_CHECK_LAUNCH();
    return 0;
}

}  // extern "C"
