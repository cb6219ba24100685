// kernels_step.hip -- one token per sequence: projections as weight-streaming GEMVs or skinny MFMA products
// (up to 16 rows) of any size with the surrounding steps fused (streams' read + grouped norm in front; convolution step, minGRU step, gated
// activation, streams' update or argmax behind), and the selective-scan step.
#include <algorithm>

#include "act.h"
#include "decoder.h"

namespace pgmi {

namespace {

constexpr int UN = 4;  // K steps (512 elements each) whose weight loads are in flight together

// eight activations as loaded
struct X8b { uint4 q; };
struct X8f { float4 a, b; };
template <typename T> struct X8 { typedef X8b type; };
template <> struct X8<float> { typedef X8f type; };
__device__ __forceinline__ void ldx(const uint16_t* p, X8b& x) { x.q = *reinterpret_cast<const uint4*>(p); }
__device__ __forceinline__ void ldx(const float* p, X8f& x) {
    x.a = *reinterpret_cast<const float4*>(p);
    x.b = *reinterpret_cast<const float4*>(p + 4);
}
__device__ __forceinline__ float dotx(const uint4 w, const X8b& x, float acc) { return dot8(w, x.q, acc); }
__device__ __forceinline__ float dotx(const uint4 w, const X8f& x, float acc) {
    const uint32_t q[4] = {w.x, w.y, w.z, w.w};
    const float v[8] = {x.a.x, x.a.y, x.a.z, x.a.w, x.b.x, x.b.y, x.b.z, x.b.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        acc = fmaf(__uint_as_float(q[i] << 16), v[2 * i], acc);
        acc = fmaf(__uint_as_float(q[i] & 0xFFFF0000u), v[2 * i + 1], acc);
    }
    return acc;
}

constexpr int unit_rows(int mode) { return mode == GR_GRU ? 3 : 2; }
// outputs a unit covers (plain modes: two rows; GRU, SwiGLU: one channel)
constexpr int unit_outs(int mode) { return mode == GR_GRU || mode == GR_SWIGLU ? 1 : 2; }

// The step that follows a projection, for output n of row b (v: its sum over K; GR_GRU: v = z, v1 = u, v2 = g;
// GR_SWIGLU: v = gate, v1 = up).  Every (n, b) is handled by one thread.
template <typename T, int MODE>
__device__ __forceinline__ void step_epilogue(const GemvRtArgs& a, int n, int b, float v, float v1, float v2) {
    if constexpr (MODE == GR_ACT) {
        if (a.bias) v += bf2f(a.bias[n]);
        stf(reinterpret_cast<T*>(a.out) + (long)b * a.ldo + n, v);
    } else if constexpr (MODE == GR_LOGITS || MODE == GR_F32) {
        reinterpret_cast<float*>(a.out)[(long)b * a.ldo + n] = v;
    } else if constexpr (MODE == GR_CONV) {
        if (n < a.C) {
            const int KT = a.taps_k;
            float* tp = a.state + (long)a.slot[b] * (KT - 1) * a.C + n;
            const bool first = a.pos[b] == 0;
            const uint16_t* cw = a.cw + (long)n * KT;
            float y = fmaf(bf2f(cw[KT - 1]), v, bf2f(a.cb[n]));
            for (int j = 0; j < KT - 1; ++j) {
                const float o = first ? 0.0f : tp[(long)j * a.C];
                y = fmaf(bf2f(cw[j]), o, y);
                if (j > 0) tp[(long)(j - 1) * a.C] = o;
            }
            if (KT > 1) tp[(long)(KT - 2) * a.C] = v;
            stf(reinterpret_cast<T*>(a.out) + (long)b * a.ldo + n, siluf_(y));
        } else {
            stf(reinterpret_cast<T*>(a.out2) + (long)b * a.ldo2 + n - a.C, v);
        }
    } else if constexpr (MODE == GR_GRU) {
        const float z = sigmoidf_(v + bf2f(a.bias[n]));
        float* st = a.state + (long)a.slot[b] * a.N + n;
        const float S = fmaf(1.0f - z, a.pos[b] > 0 ? *st : 0.0f, z * gru_candidate(v1 + bf2f(a.bias[a.N + n])));
        *st = S;
        stf(reinterpret_cast<T*>(a.out) + (long)b * a.ldo + n, S * siluf_(v2));
    } else if constexpr (MODE == GR_SWIGLU) {
        stf(reinterpret_cast<T*>(a.out) + (long)b * a.ldo + n, siluf_(v) * v1);
    } else {  // GR_STREAMS: the whole column of streams at once
        float* Xr = a.X + (long)b * a.S * a.D + n;
        if (!a.mix) {
            *Xr = fmaf(a.mult, v, *Xr);
            return;
        }
        float x[8];
#pragma unroll
        for (int s = 0; s < 8; ++s) x[s] = s < a.S ? Xr[(long)s * a.D] : 0.0f;
        for (int t = 0; t < a.S; ++t) {
            float y = bf2f(a.wout[t]) * v;
#pragma unroll
            for (int s = 0; s < 8; ++s)
                if (s < a.S) y = fmaf(bf2f(a.mix[s * a.S + t]), x[s], y);
            Xr[(long)t * a.D] = y;
        }
    }
}

// the columns that pad an activation row to a multiple of 8 are zero
template <typename T, int MODE>
__device__ __forceinline__ void step_pads(const GemvRtArgs& a) {
    if constexpr (MODE == GR_GRU || MODE == GR_SWIGLU || MODE == GR_CONV) {
        const int n = MODE == GR_CONV ? a.C : a.N;
        if (blockIdx.x == 0 && (int)threadIdx.x < a.B)
            for (int k = n; k < a.ldo; ++k) stf(reinterpret_cast<T*>(a.out) + (long)threadIdx.x * a.ldo + k, 0.0f);
    }
}

// WK: waves of the workgroup that share a unit, each a K slice.  XG: the input is rows of activations, loaded with the
// weights; else the streams' read and norm, staged in LDS by the prologue.
template <typename T, int NB, int MODE, int WK, bool XG>
__global__ void __launch_bounds__(256) k_gemv_rt(GemvRtArgs a) {
    constexpr int RW = unit_rows(MODE), UO = unit_outs(MODE), UPB = 4 / WK;
    extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
    T* xs = reinterpret_cast<T*>(smem);  // [NB][K]
    __shared__ float red[64];
    __shared__ float part[WK > 1 ? 4 : 1][RW * NB];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int nunit = (a.N + UO - 1) / UO, K = a.K;
    const int ustep = gridDim.x * UPB, kw = wave % WK;
    int unit = blockIdx.x * UPB + wave / WK;
    uint4 w[2][RW][UN];
    typename X8<T>::type xr[2][XG ? NB : 1][XG ? UN : 1];
    auto xload = [&](int buf, int k0) {
        if constexpr (XG) {
#pragma unroll
            for (int b = 0; b < NB; ++b) {
                const T* p = reinterpret_cast<const T*>(a.x) + (long)(b < a.B ? b : 0) * a.ldx;
#pragma unroll
                for (int i = 0; i < UN; ++i) {
                    const int k = k0 + (i * WK + kw) * 512 + lane * 8;
                    ldx(p + (k < K ? k : 0), xr[buf][b][i]);
                }
            }
        }
    };
    auto wload = [&](uint4 (&q)[RW][UN], int u, int k0) {
        const int uu = u < nunit ? u : nunit - 1;
#pragma unroll
        for (int r = 0; r < RW; ++r) {
            int n;
            if constexpr (UO == 1) n = r * a.N + uu;
            else { n = uu * 2 + r; n = n < a.N ? n : a.N - 1; }
            const uint16_t* p = a.W + (long)n * a.ldw;
#pragma unroll
            for (int i = 0; i < UN; ++i) {
                const int k = k0 + (i * WK + kw) * 512 + lane * 8;
                q[r][i] = ldg16_sel(p + k, k < K, p);
            }
        }
    };
    wload(w[0], unit, 0);  // in flight during the prologue
    if constexpr (XG) {
        xload(0, 0);
    } else {
        // the streams' read and grouped norm of each row, as streams_norm
        float* u_ = reinterpret_cast<float*>(smem + (size_t)NB * K * sizeof(T));  // [D], then [groups]
        float* inv = u_ + a.D;
        const int P = a.D / a.groups, D = a.D;
        for (int b = 0; b < NB && b < a.B; ++b) {
            const float* Xr = a.X + (long)b * a.S * D;
            if (P % 256 == 0 && D <= 8192) {
                // a wave's 64 x 4 elements lie in one group: one partial per (piece, wave)
                constexpr int PC = 8;
                const int np = (D + 1023) / 1024;
                float4 u[PC];
                ushort4 nw[PC];
#pragma unroll
                for (int i = 0; i < PC; ++i) {
                    u[i] = make_float4(0.f, 0.f, 0.f, 0.f);
                    nw[i] = make_ushort4(0, 0, 0, 0);
                    const int d = i * 1024 + tid * 4;
                    if (i < np && d < D) {
                        nw[i] = *reinterpret_cast<const ushort4*>(a.nw + d);
                        for (int s = 0; s < a.S; ++s) {
                            const float c = a.in ? bf2f(a.in[s]) : 1.0f;
                            const float4 q = *reinterpret_cast<const float4*>(Xr + (long)s * D + d);
                            u[i].x = fmaf(c, q.x, u[i].x); u[i].y = fmaf(c, q.y, u[i].y);
                            u[i].z = fmaf(c, q.z, u[i].z); u[i].w = fmaf(c, q.w, u[i].w);
                        }
                    }
                }
#pragma unroll
                for (int i = 0; i < PC; ++i)
                    if (i < np) {
                        const float q = wave_sum(u[i].x * u[i].x + u[i].y * u[i].y + u[i].z * u[i].z + u[i].w * u[i].w);
                        if (lane == 0) red[i * 4 + wave] = q;
                    }
                __syncthreads();
#pragma unroll
                for (int i = 0; i < PC; ++i) {
                    const int d = i * 1024 + tid * 4;
                    if (i < np && d < D) {
                        const int p0 = d / P * (P / 256);
                        float q = 0.0f;
                        for (int t = 0; t < P / 256; ++t) q += red[p0 + t];
                        const float f = 1.0f / sqrtf(q / (float)P + a.eps);
                        T* o = xs + b * K + d;
                        stf(o, u[i].x * f * bf2f(nw[i].x));
                        stf(o + 1, u[i].y * f * bf2f(nw[i].y));
                        stf(o + 2, u[i].z * f * bf2f(nw[i].z));
                        stf(o + 3, u[i].w * f * bf2f(nw[i].w));
                    }
                }
                __syncthreads();
                continue;
            }
            for (int d = tid; d < D; d += 256) {
                float u = 0.0f;
                for (int s = 0; s < a.S; ++s) u = fmaf(a.in ? bf2f(a.in[s]) : 1.0f, Xr[(long)s * D + d], u);
                u_[d] = u;
            }
            __syncthreads();
            for (int g = wave; g < a.groups; g += 4) {
                float q = 0.0f;
                for (int i = lane; i < P; i += 64) q = fmaf(u_[g * P + i], u_[g * P + i], q);
                q = wave_sum(q);
                if (lane == 0) inv[g] = 1.0f / sqrtf(q / (float)P + a.eps);
            }
            __syncthreads();
            for (int d = tid; d < K; d += 256) stf(xs + b * K + d, d < D ? u_[d] * inv[d / P] * bf2f(a.nw[d]) : 0.0f);
            __syncthreads();
        }
    }
    float best[NB];
    int bi[NB];
#pragma unroll
    for (int b = 0; b < NB; ++b) { best[b] = -INFINITY; bi[b] = 0x7fffffff; }
    float acc[RW][NB];
    auto mac = [&](int buf, int k0) {
#pragma unroll
        for (int i = 0; i < UN; ++i) {
            const int k = k0 + (i * WK + kw) * 512 + lane * 8;
            if (k < K) {
#pragma unroll
                for (int b = 0; b < NB; ++b) {
                    typename X8<T>::type x;
                    if constexpr (XG) x = xr[buf][b][i];
                    else ldx(xs + b * K + k, x);
#pragma unroll
                    for (int r = 0; r < RW; ++r) acc[r][b] = dotx(w[buf][r][i], x, acc[r][b]);
                }
            }
        }
    };
    constexpr int KB = UN * WK * 512;  // K elements per block
    // every wave of a workgroup runs the same number of rounds (WK > 1 meets at a barrier)
    for (int u0 = blockIdx.x * UPB; u0 < nunit; u0 += ustep, unit += ustep) {
#pragma unroll
        for (int r = 0; r < RW; ++r)
#pragma unroll
            for (int b = 0; b < NB; ++b) acc[r][b] = 0.0f;
        for (int k0 = 0; k0 < K; k0 += 2 * KB) {
            if (k0 + KB < K) {
                wload(w[1], unit, k0 + KB);
                xload(1, k0 + KB);
            }
            mac(0, k0);
            if (k0 + KB < K) {
                if (k0 + 2 * KB < K) {
                    wload(w[0], unit, k0 + 2 * KB);
                    xload(0, k0 + 2 * KB);
                }
                mac(1, k0 + KB);
            }
        }
        if (u0 + ustep < nunit) {
            wload(w[0], unit + ustep, 0);
            xload(0, 0);
        }
#pragma unroll
        for (int r = 0; r < RW; ++r)
#pragma unroll
            for (int b = 0; b < NB; ++b) acc[r][b] = wave_sum(acc[r][b]);
        if constexpr (WK > 1) {
            __syncthreads();
            if (lane == 0)
#pragma unroll
                for (int r = 0; r < RW; ++r)
#pragma unroll
                    for (int b = 0; b < NB; ++b) part[wave][r * NB + b] = acc[r][b];
            __syncthreads();
#pragma unroll
            for (int r = 0; r < RW; ++r)
#pragma unroll
                for (int b = 0; b < NB; ++b) {
                    float t = 0.0f;
#pragma unroll
                    for (int q = 0; q < WK; ++q) t += part[(wave / WK) * WK + q][r * NB + b];
                    acc[r][b] = t;
                }
        }
        if (unit >= nunit) continue;
        if constexpr (MODE == GR_LOGITS) {
#pragma unroll
            for (int r = 0; r < RW; ++r)
#pragma unroll
                for (int b = 0; b < NB; ++b) {
                    const int n = unit * 2 + r;
                    if (n < a.N && acc[r][b] > best[b]) { best[b] = acc[r][b]; bi[b] = n; }
                }
        }
        // lane (r, b) of the unit's first wave finishes output r of row b
        const int lr = lane / NB, lb = lane % NB;
        float v = 0.0f, v1 = 0.0f, v2 = 0.0f;
#pragma unroll
        for (int b = 0; b < NB; ++b) {
            if constexpr (UO == 1) {
                if (lb == b) { v = acc[0][b]; v1 = acc[1][b]; v2 = acc[RW - 1][b]; }
            } else {
#pragma unroll
                for (int r = 0; r < RW; ++r)
                    if (lr == r && lb == b) v = acc[r][b];
            }
        }
        const int n = unit * UO + lr;
        if (kw == 0 && lr < UO && lb < a.B && n < a.N) step_epilogue<T, MODE>(a, n, lb, v, v1, v2);
    }
    if constexpr (MODE == GR_LOGITS) {
        __shared__ float sv[4][NB];
        __shared__ int si[4][NB];
        if (lane == 0)
#pragma unroll
            for (int b = 0; b < NB; ++b) { sv[wave][b] = best[b]; si[wave][b] = bi[b]; }
        __syncthreads();
        if (tid < NB && tid < a.B) {
            float v = sv[0][tid];
            int ix = si[0][tid];
            for (int q = 1; q < 4; ++q)
                if (sv[q][tid] > v || (sv[q][tid] == v && si[q][tid] < ix)) { v = sv[q][tid]; ix = si[q][tid]; }
            a.pmax[(long)tid * gridDim.x + blockIdx.x] = v;
            a.pidx[(long)tid * gridDim.x + blockIdx.x] = ix;
        }
    }
    step_pads<T, MODE>(a);
}

int k_split(const GemvRtArgs& a, int mode) { return mode != GR_LOGITS && a.K >= 4096 ? 4 : 1; }

template <typename T, int NB, int MODE, int WK>
void run_wk(hipStream_t s, const GemvRtArgs& a) {
    const dim3 grid(gemv_rt_blocks(a, (GemvRtMode)MODE));
    if (a.x) {
        hipLaunchKernelGGL((k_gemv_rt<T, NB, MODE, WK, true>), grid, dim3(256), 0, s, a);
        return;
    }
    const size_t lds = (size_t)NB * a.K * sizeof(T) + (size_t)(a.D + a.groups) * sizeof(float);
    if (lds > 60 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&k_gemv_rt<T, NB, MODE, WK, false>),
                                  hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL((k_gemv_rt<T, NB, MODE, WK, false>), grid, dim3(256), lds, s, a);
}

template <typename T, int NB, int MODE>
void run(hipStream_t s, const GemvRtArgs& a) {
    if (MODE != GR_LOGITS && k_split(a, MODE) == 4) run_wk<T, NB, MODE, MODE == GR_LOGITS ? 1 : 4>(s, a);
    else run_wk<T, NB, MODE, 1>(s, a);
}

template <typename T, int NB>
void run_mode(hipStream_t s, GemvRtMode mode, const GemvRtArgs& a) {
    switch (mode) {
        case GR_ACT: run<T, NB, GR_ACT>(s, a); break;
        case GR_CONV: run<T, NB, GR_CONV>(s, a); break;
        case GR_GRU: run<T, NB, GR_GRU>(s, a); break;
        case GR_SWIGLU: run<T, NB, GR_SWIGLU>(s, a); break;
        case GR_STREAMS: run<T, NB, GR_STREAMS>(s, a); break;
        case GR_LOGITS: run<T, NB, GR_LOGITS>(s, a); break;
        case GR_F32: run<T, NB, GR_F32>(s, a); break;
    }
}

// ---------------------------------------------------------------- up to 16 rows: MFMA
// A workgroup owns 16 outputs (of each of the unit's matrices) and all rows; its 4 waves split K.  A lane reads 32
// contiguous bytes of its weight row per 64-deep step (4 lanes: one 128-byte line), so the two MFMAs of a step
// contract k = 16 lg .. 16 lg + 7 and 16 lg + 8 .. 16 lg + 15 of each lane group -- the activations (straight from
// L2, B fragments) use the same order.  After the waves' sums meet in LDS, thread (n, b) runs the step's epilogue.
// GR_F32 with gridDim.y > 1: K is cut over the y workgroups too, out holds their partial slabs [y][B][N].
template <int MODE>
__global__ void __launch_bounds__(256) k_skinny(GemvRtArgs a) {
    constexpr int NM = MODE == GR_GRU ? 3 : MODE == GR_SWIGLU ? 2 : 1;
    constexpr int U = NM == 1 ? 8 : 4;  // 64-deep steps in flight
    __shared__ float sums[4][NM][16][17];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int li = lane & 15, lg = lane >> 4, n0 = blockIdx.x * 16, K = a.K;
    const uint16_t* wp[NM];
#pragma unroll
    for (int m = 0; m < NM; ++m) {
        const int n = n0 + li < a.N ? n0 + li : a.N - 1;
        wp[m] = a.W + ((long)m * a.N + n) * a.ldw;
    }
    const uint16_t* xp = reinterpret_cast<const uint16_t*>(a.x) + (long)(li < a.B ? li : a.B - 1) * a.ldx;
    f32x4 acc[NM];
#pragma unroll
    for (int m = 0; m < NM; ++m) acc[m] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int nstep = (K + 63) / 64;
    const int per = (nstep + gridDim.y - 1) / gridDim.y, s_end = min(nstep, (int)(blockIdx.y + 1) * per);
    for (int s0 = blockIdx.y * per + wave; s0 < s_end; s0 += 4 * U) {
        uint4 w[U][NM][2], x[U][2];
#pragma unroll
        for (int i = 0; i < U; ++i) {
            const int k = (s0 + 4 * i) * 64 + lg * 16;
#pragma unroll
            for (int h = 0; h < 2; ++h) {
                const bool ok = s0 + 4 * i < s_end && k + 8 * h < K;
#pragma unroll
                for (int m = 0; m < NM; ++m) w[i][m][h] = ldg16_sel(wp[m] + k + 8 * h, ok, wp[m]);
                x[i][h] = ldg16_sel(xp + k + 8 * h, ok, xp);
            }
        }
#pragma unroll
        for (int i = 0; i < U; ++i)
#pragma unroll
            for (int h = 0; h < 2; ++h)
#pragma unroll
                for (int m = 0; m < NM; ++m)
                    acc[m] = mfma16(__builtin_bit_cast(short8, w[i][m][h]), __builtin_bit_cast(short8, x[i][h]), acc[m]);
    }
#pragma unroll
    for (int m = 0; m < NM; ++m)
#pragma unroll
        for (int r = 0; r < 4; ++r) sums[wave][m][4 * lg + r][li] = acc[m][r];
    __syncthreads();
    const int b = tid & 15, n = n0 + (tid >> 4);
    float v[3] = {0.f, 0.f, 0.f};
#pragma unroll
    for (int m = 0; m < NM; ++m)
#pragma unroll
        for (int q = 0; q < 4; ++q) v[m] += sums[q][m][tid >> 4][b];
    if constexpr (MODE == GR_F32) {
        if (b < a.B && n < a.N)
            reinterpret_cast<float*>(a.out)[((long)blockIdx.y * a.B + b) * a.ldo + n] = v[0];
        return;
    }
    if (b < a.B && n < a.N) step_epilogue<uint16_t, MODE>(a, n, b, v[0], v[1], v[2]);
    step_pads<uint16_t, MODE>(a);
}

void run_skinny(hipStream_t s, GemvRtMode mode, const GemvRtArgs& a) {
    const dim3 grid((a.N + 15) / 16), block(256);
    switch (mode) {
        case GR_ACT: hipLaunchKernelGGL((k_skinny<GR_ACT>), grid, block, 0, s, a); break;
        case GR_CONV: hipLaunchKernelGGL((k_skinny<GR_CONV>), grid, block, 0, s, a); break;
        case GR_GRU: hipLaunchKernelGGL((k_skinny<GR_GRU>), grid, block, 0, s, a); break;
        case GR_SWIGLU: hipLaunchKernelGGL((k_skinny<GR_SWIGLU>), grid, block, 0, s, a); break;
        case GR_STREAMS: hipLaunchKernelGGL((k_skinny<GR_STREAMS>), grid, block, 0, s, a); break;
        default: hipLaunchKernelGGL((k_skinny<GR_F32>), dim3(grid.x, a.split < 1 ? 1 : a.split), block, 0, s, a); break;
    }
}

// ---------------------------------------------------------------- convolution step
template <typename T>
__global__ void __launch_bounds__(256) k_conv_step(const T* __restrict__ xz, int ldxz, int C, int K,
                                                   const uint16_t* __restrict__ w, const uint16_t* __restrict__ cb,
                                                   float* __restrict__ taps, const int* __restrict__ slot,
                                                   const int* __restrict__ pos, T* __restrict__ out, int ldo) {
    const int b = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
    if (c >= ldo) return;
    float y = 0.0f;
    if (c < C) {
        float* tp = taps + (long)slot[b] * (K - 1) * C + c;
        const bool first = pos[b] == 0;
        const float v = ldf(xz + (long)b * ldxz + c);
        y = fmaf(bf2f(w[(long)c * K + K - 1]), v, bf2f(cb[c]));
        for (int j = 0; j < K - 1; ++j) {
            const float o = first ? 0.0f : tp[(long)j * C];
            y = fmaf(bf2f(w[(long)c * K + j]), o, y);
            if (j > 0) tp[(long)(j - 1) * C] = o;
        }
        if (K > 1) tp[(long)(K - 2) * C] = v;
        y = siluf_(y);
    }
    stf(out + (long)b * ldo + c, y);
}

// ---------------------------------------------------------------- selective-scan step
// LPC lanes per channel: they share the dt dot product over R and hold the channel's states
template <typename T, int LPC>
__global__ void __launch_bounds__(256) k_scan_step(ScanStepArgs a) {
    extern __shared__ float sm[];  // [R + 2N] of this sequence
    constexpr int CPB = 256 / LPC;
    const int b = blockIdx.y, tid = threadIdx.x, sub = tid % LPC;
    const int M = a.R + 2 * a.N;
    for (int i = tid; i < M; i += 256) {
        float v = 0.0f;
        for (int z = 0; z < a.split; ++z) v += a.slabs[((long)z * a.B + b) * M + i];
        sm[i] = v;
    }
    __syncthreads();
    const int c = blockIdx.x * CPB + tid / LPC;
    const bool ok = c < a.C;
    const int cc = ok ? c : a.C - 1;
    float dt = 0.0f;
    const uint16_t* wd = a.Wdt + (long)cc * a.ldwdt;
    for (int r = sub * 8; r < a.R; r += LPC * 8) {  // rows of Wdt are 16-byte aligned, zero past R
        float w[8];
        ld8(wd + r, w);
#pragma unroll
        for (int v = 0; v < 8; ++v)
            if (r + v < a.R) dt = fmaf(w[v], sm[r + v], dt);
    }
#pragma unroll
    for (int o = 1; o < LPC; o <<= 1) dt += __shfl_xor(dt, o, 64);
    dt = softplusf_(dt + bf2f(a.dtb[cc]));
    const float x = ldf(reinterpret_cast<const T*>(a.x) + (long)b * a.ldx + cc);
    const float dx = dt * x;
    const bool first = a.pos[b] == 0;
    float* st = a.state + ((long)a.slot[b] * a.C + cc) * a.N;
    const float* B = sm + a.R;
    const float* Cv = B + a.N;
    float y = 0.0f;
    for (int n = sub; n < a.N; n += LPC) {
        const float A = -expf(bf2f(a.A_log[(long)cc * a.N + n])) * 1.4426950408889634f;
        const float S = fmaf(__builtin_amdgcn_exp2f(dt * A), first ? 0.0f : st[n], dx * B[n]);
        if (ok) st[n] = S;
        y = fmaf(S, Cv[n], y);
    }
#pragma unroll
    for (int o = 1; o < LPC; o <<= 1) y += __shfl_xor(y, o, 64);
    if (sub == 0 && c < a.ldy) {
        y = fmaf(bf2f(a.Dw[cc]), x, y);
        stf(reinterpret_cast<T*>(a.y) + (long)b * a.ldy + c,
            ok ? y * siluf_(ldf(reinterpret_cast<const T*>(a.z) + (long)b * a.ldz + cc)) : 0.0f);
    }
}

template <typename T>
void scan_step_t(hipStream_t s, const ScanStepArgs& a) {
    const size_t lds = (size_t)(a.R + 2 * a.N) * sizeof(float);
    const int cols = std::max(a.C, a.ldy);
    if (a.N <= 16) hipLaunchKernelGGL((k_scan_step<T, 8>), dim3((cols + 31) / 32, a.B), dim3(256), lds, s, a);
    else hipLaunchKernelGGL((k_scan_step<T, 16>), dim3((cols + 15) / 16, a.B), dim3(256), lds, s, a);
}

// ---------------------------------------------------------------- minGRU step
template <typename T>
__global__ void __launch_bounds__(256) k_gru_step(const T* __restrict__ zug, int ld, int C, float* __restrict__ state,
                                                  const int* __restrict__ slot, const int* __restrict__ pos,
                                                  T* __restrict__ y, int ldy) {
    const int b = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
    if (c >= ldy) return;
    float v = 0.0f;
    if (c < C) {
        const T* r = zug + (long)b * ld + c;
        float* st = state + (long)slot[b] * C + c;
        const float z = sigmoidf_(ldf(r));
        const float S = fmaf(1.0f - z, pos[b] > 0 ? *st : 0.0f, z * gru_candidate(ldf(r + C)));
        *st = S;
        v = S * siluf_(ldf(r + 2 * C));
    }
    stf(y + (long)b * ldy + c, v);
}

// ---------------------------------------------------------------- end of a step
__global__ void __launch_bounds__(256) k_decode_finish(const float* __restrict__ pmax, const int* __restrict__ pidx,
                                                       int nparts, int64_t* __restrict__ next, int64_t* __restrict__ hist,
                                                       int* __restrict__ pos) {
    const int b = blockIdx.x, tid = threadIdx.x;
    __shared__ float sv[256];
    __shared__ int si[256];
    if (nparts > 0) {
        float best = -INFINITY;
        int bi = 0x7fffffff;
        for (int i = tid; i < nparts; i += 256) {
            const float v = pmax[(long)b * nparts + i];
            const int ix = pidx[(long)b * nparts + i];
            if (v > best || (v == best && ix < bi)) { best = v; bi = ix; }
        }
        sv[tid] = best;
        si[tid] = bi;
        __syncthreads();
        for (int o = 128; o > 0; o >>= 1) {
            if (tid < o && (sv[tid + o] > sv[tid] || (sv[tid + o] == sv[tid] && si[tid + o] < si[tid]))) {
                sv[tid] = sv[tid + o];
                si[tid] = si[tid + o];
            }
            __syncthreads();
        }
        // no finite logit: token 0 rather than an index out of the table
        if (tid == 0) next[b] = si[0] == 0x7fffffff ? 0 : si[0];
    }
    if (tid == 0) {
        if (hist) hist[b] = next[b];
        pos[b] += 1;
    }
}

}  // namespace

int gemv_rt_max_batch() { return 16; }
int gemv_rt_parts() { return 2 * 1024; }
GemvRtForm gemv_rt_form(int B, Act act, int streams, int width) {
    // fp32 activations: no MFMA form.  bf16: one row, while every workgroup's own read of the streams stays small;
    // measured, batch 1, 2 streams: width 1024 0.379 against 0.432 ms per step, 2048 0.802 / 0.818, 4096 0.828 / 0.661
    if (act == ACT_F32) return B <= 2 ? GF_STREAM : GF_NONE;
    if (B == 1 && streams * width <= 4096) return GF_STREAM;
    return B <= gemv_rt_max_batch() ? GF_SKINNY : GF_NONE;
}

bool gemv_rt_fits(GemvRtForm form, int K, Act act) {
    if (form == GF_STREAM) return (size_t)2 * K * (act == ACT_F32 ? 4 : 2) <= 96 * 1024;
    return form == GF_SKINNY;
}

int gemv_rt_split(GemvRtForm form, int N, int K) {
    if (form != GF_SKINNY) return 1;
    const int tiles = (N + 15) / 16, nstep = (K + 63) / 64;
    int split = 1;
    while (split < 8 && tiles * split < 512 && nstep / (split * 2) >= 4) split *= 2;
    const int per = (nstep + split - 1) / split;  // no empty slice
    return (nstep + per - 1) / per;
}

int gemv_rt_blocks(const GemvRtArgs& a, GemvRtMode mode) {
    const int units = (a.N + unit_outs(mode) - 1) / unit_outs(mode), upb = 4 / k_split(a, mode);
    return std::max(1, std::min((units + upb - 1) / upb, 1024));
}

void gemv_rt(hipStream_t s, Act act, GemvRtMode mode, const GemvRtArgs& a) {
    if (a.form == GF_SKINNY) run_skinny(s, mode, a);
    else if (act == ACT_BF16) run_mode<uint16_t, 1>(s, mode, a);
    else if (a.B <= 1) run_mode<float, 1>(s, mode, a);
    else run_mode<float, 2>(s, mode, a);
}

void conv_step(hipStream_t s, Act act, const void* xz, int ldxz, int B, int C, int K, const uint16_t* w,
               const uint16_t* b, float* taps, const int* slot, const int* pos, void* out, int ldo) {
    const dim3 grid((ldo + 255) / 256, B);
    if (act == ACT_F32)
        hipLaunchKernelGGL((k_conv_step<float>), grid, dim3(256), 0, s, reinterpret_cast<const float*>(xz), ldxz, C, K, w,
                           b, taps, slot, pos, reinterpret_cast<float*>(out), ldo);
    else
        hipLaunchKernelGGL((k_conv_step<uint16_t>), grid, dim3(256), 0, s, reinterpret_cast<const uint16_t*>(xz), ldxz, C,
                           K, w, b, taps, slot, pos, reinterpret_cast<uint16_t*>(out), ldo);
}

void scan_step(hipStream_t s, Act act, const ScanStepArgs& a) {
    if (act == ACT_F32) scan_step_t<float>(s, a);
    else scan_step_t<uint16_t>(s, a);
}

void gru_step(hipStream_t s, Act act, const void* zug, int ld, int B, int C, float* state, const int* slot,
              const int* pos, void* y, int ldy) {
    const dim3 grid((ldy + 255) / 256, B);
    if (act == ACT_F32)
        hipLaunchKernelGGL((k_gru_step<float>), grid, dim3(256), 0, s, reinterpret_cast<const float*>(zug), ld, C, state,
                           slot, pos, reinterpret_cast<float*>(y), ldy);
    else
        hipLaunchKernelGGL((k_gru_step<uint16_t>), grid, dim3(256), 0, s, reinterpret_cast<const uint16_t*>(zug), ld, C,
                           state, slot, pos, reinterpret_cast<uint16_t*>(y), ldy);
}

void decode_finish(hipStream_t s, int B, const float* pmax, const int* pidx, int nparts, int64_t* next, int64_t* hist,
                   int* pos) {
    hipLaunchKernelGGL(k_decode_finish, dim3(B), dim3(256), 0, s, pmax, pidx, nparts, next, hist, pos);
}

}  // namespace pgmi
