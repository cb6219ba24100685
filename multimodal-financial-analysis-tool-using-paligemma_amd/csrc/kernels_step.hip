// kernels_step.hip -- one token per sequence: projections as weight-streaming GEMVs of any size with the
// surrounding steps fused (streams' read + grouped norm in front; convolution step, minGRU step, gated
// activation, streams' update or argmax behind), and the selective-scan step.
#include <algorithm>

#include "act.h"
#include "decoder.h"

namespace pgmi {

namespace {

constexpr int UN = 4;  // K steps (512 elements each) whose weight loads are in flight together

__device__ __forceinline__ float dotx(const uint4 w, const uint16_t* x, float acc) {
    return dot8(w, *reinterpret_cast<const uint4*>(x), acc);
}
__device__ __forceinline__ float dotx(const uint4 w, const float* x, float acc) {
    const uint32_t q[4] = {w.x, w.y, w.z, w.w};
    float v[8];
    ld8(x, v);
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

template <typename T, int NB, int MODE>
__global__ void __launch_bounds__(256) k_gemv_rt(GemvRtArgs a) {
    constexpr int RW = unit_rows(MODE), UO = unit_outs(MODE);
    extern __shared__ __attribute__((aligned(16))) uint8_t smem[];
    T* xs = reinterpret_cast<T*>(smem);  // [NB][K]
    __shared__ float red[4];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int nunit = (a.N + UO - 1) / UO, K = a.K;
    int unit = blockIdx.x * 4 + wave;
    uint4 w[RW][UN];
    auto wrow = [&](int u, int r) -> long {
        int n;
        if constexpr (UO == 1) n = r * a.N + u;
        else { n = u * 2 + r; n = n < a.N ? n : a.N - 1; }
        return n;
    };
    auto wload = [&](int u, int k0) {
        const int uu = u < nunit ? u : nunit - 1;
#pragma unroll
        for (int r = 0; r < RW; ++r) {
            const uint16_t* p = a.W + wrow(uu, r) * a.ldw;
#pragma unroll
            for (int i = 0; i < UN; ++i) {
                const int k = k0 + i * 512 + lane * 8;
                w[r][i] = ldg16_sel(p + k, k < K, p);
            }
        }
    };
    wload(unit, 0);  // in flight during the prologue
    if (a.x) {
        for (int e = tid * 8; e < NB * K; e += 256 * 8) {
            const int b = e / K, k = e % K;
            float v[8];
            ld8(reinterpret_cast<const T*>(a.x) + (long)(b < a.B ? b : 0) * a.ldx + k, v);
            st8(xs + b * K + k, v);
        }
    } else {
        // the streams' read and grouped norm of each row (fp32 in registers / LDS), as streams_norm
        float* u_ = reinterpret_cast<float*>(smem + (size_t)NB * K * sizeof(T));  // [D], then [groups]
        float* inv = u_ + a.D;
        const int P = a.D / a.groups;
        for (int b = 0; b < NB && b < a.B; ++b) {
            const float* Xr = a.X + (long)b * a.S * a.D;
            for (int d = tid; d < a.D; d += 256) {
                float u = 0.0f;
                for (int s = 0; s < a.S; ++s) u = fmaf(a.in ? bf2f(a.in[s]) : 1.0f, Xr[(long)s * a.D + d], u);
                u_[d] = u;
            }
            __syncthreads();
            if (a.groups >= 4) {
                for (int g = wave; g < a.groups; g += 4) {
                    float q = 0.0f;
                    for (int i = lane; i < P; i += 64) q = fmaf(u_[g * P + i], u_[g * P + i], q);
                    q = wave_sum(q);
                    if (lane == 0) inv[g] = 1.0f / sqrtf(q / (float)P + a.eps);
                }
                __syncthreads();
            } else {
                for (int g = 0; g < a.groups; ++g) {
                    float q = 0.0f;
                    for (int i = tid; i < P; i += 256) q = fmaf(u_[g * P + i], u_[g * P + i], q);
                    q = wave_sum(q);
                    if (lane == 0) red[wave] = q;
                    __syncthreads();
                    if (tid == 0) inv[g] = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)P + a.eps);
                    __syncthreads();
                }
            }
            for (int d = tid; d < K; d += 256) stf(xs + b * K + d, d < a.D ? u_[d] * inv[d / P] * bf2f(a.nw[d]) : 0.0f);
            __syncthreads();
        }
    }
    __syncthreads();
    float best[NB];
    int bi[NB];
#pragma unroll
    for (int b = 0; b < NB; ++b) { best[b] = -INFINITY; bi[b] = 0x7fffffff; }
    for (; unit < nunit; unit += gridDim.x * 4) {
        float acc[RW][NB];
#pragma unroll
        for (int r = 0; r < RW; ++r)
#pragma unroll
            for (int b = 0; b < NB; ++b) acc[r][b] = 0.0f;
        for (int k0 = 0; k0 < K; k0 += UN * 512) {
#pragma unroll
            for (int i = 0; i < UN; ++i) {
                const int k = k0 + i * 512 + lane * 8;
                if (k < K) {
#pragma unroll
                    for (int b = 0; b < NB; ++b)
#pragma unroll
                        for (int r = 0; r < RW; ++r) acc[r][b] = dotx(w[r][i], xs + b * K + k, acc[r][b]);
                }
            }
            if (k0 + UN * 512 < K) wload(unit, k0 + UN * 512);
        }
        if (unit + (int)gridDim.x * 4 < nunit) wload(unit + gridDim.x * 4, 0);
#pragma unroll
        for (int r = 0; r < RW; ++r)
#pragma unroll
            for (int b = 0; b < NB; ++b) acc[r][b] = wave_sum(acc[r][b]);
        if constexpr (MODE == GR_GRU || MODE == GR_SWIGLU) {
            const int c = unit;
#pragma unroll
            for (int b = 0; b < NB; ++b) {
                if (lane == b && b < a.B) {
                    float y;
                    if constexpr (MODE == GR_GRU) {
                        float zr = acc[0][b] + bf2f(a.bias[c]), ur = acc[1][b] + bf2f(a.bias[a.N + c]);
                        const float z = sigmoidf_(zr);
                        float* st = a.state + (long)a.slot[b] * a.N + c;
                        const float S = fmaf(1.0f - z, a.pos[b] > 0 ? *st : 0.0f, z * gru_candidate(ur));
                        *st = S;
                        y = S * siluf_(acc[RW - 1][b]);
                    } else {
                        y = siluf_(acc[0][b]) * acc[1][b];
                    }
                    stf(reinterpret_cast<T*>(a.out) + (long)b * a.ldo + c, y);
                }
            }
        } else if constexpr (MODE == GR_STREAMS) {
            // lane (r, b, t): every lane of the wave has read its streams before any is written
            const int t = lane & 7, b = (lane >> 3) % NB, r = (lane >> 3) / NB;
            float y = 0.0f;
#pragma unroll
            for (int rr = 0; rr < RW; ++rr)
#pragma unroll
                for (int bb = 0; bb < NB; ++bb)
                    if (r == rr && b == bb) y = acc[rr][bb];
            const int n = unit * 2 + r;
            const bool ok = r < RW && b < a.B && t < a.S && n < a.N;
            float v = 0.0f;
            if (ok) {
                const float* Xr = a.X + (long)b * a.S * a.D + n;
                v = bf2f(a.wout[t]) * y;
                for (int s = 0; s < a.S; ++s) v = fmaf(bf2f(a.mix[s * a.S + t]), Xr[(long)s * a.D], v);
            }
            if (ok) a.X[((long)b * a.S + t) * a.D + n] = v;
        } else {
#pragma unroll
            for (int r = 0; r < RW; ++r)
#pragma unroll
                for (int b = 0; b < NB; ++b) {
                    const int n = unit * 2 + r;
                    if constexpr (MODE == GR_LOGITS) {
                        if (n < a.N && (acc[r][b] > best[b])) { best[b] = acc[r][b]; bi[b] = n; }
                    }
                    if (lane == r * NB + b && b < a.B && n < a.N) {
                        float v = acc[r][b];
                        if constexpr (MODE == GR_LOGITS || MODE == GR_F32) {
                            reinterpret_cast<float*>(a.out)[(long)b * a.ldo + n] = v;
                        } else if constexpr (MODE == GR_ACT) {
                            if (a.bias) v += bf2f(a.bias[n]);
                            stf(reinterpret_cast<T*>(a.out) + (long)b * a.ldo + n, v);
                        } else if constexpr (MODE == GR_CONV) {
                            if (n < a.C) {
                                const int KT = a.taps_k;
                                float* tp = a.state + (long)a.slot[b] * (KT - 1) * a.C + n;
                                const bool first = a.pos[b] == 0;
                                float y = fmaf(bf2f(a.cw[(long)n * KT + KT - 1]), v, bf2f(a.cb[n]));
                                for (int j = 0; j < KT - 1; ++j) {
                                    const float o = first ? 0.0f : tp[(long)j * a.C];
                                    y = fmaf(bf2f(a.cw[(long)n * KT + j]), o, y);
                                    if (j > 0) tp[(long)(j - 1) * a.C] = o;
                                }
                                if (KT > 1) tp[(long)(KT - 2) * a.C] = v;
                                stf(reinterpret_cast<T*>(a.out) + (long)b * a.ldo + n, siluf_(y));
                            } else {
                                stf(reinterpret_cast<T*>(a.out2) + (long)b * a.ldo2 + n - a.C, v);
                            }
                        }
                    }
                }
        }
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
    // activation outputs: the columns that pad a row to 8 are zero
    if constexpr (MODE == GR_GRU || MODE == GR_SWIGLU || MODE == GR_CONV) {
        const int n = MODE == GR_CONV ? a.C : a.N;
        if (blockIdx.x == 0 && tid < NB && tid < a.B)
            for (int k = n; k < a.ldo; ++k) stf(reinterpret_cast<T*>(a.out) + (long)tid * a.ldo + k, 0.0f);
    }
}

template <typename T, int NB, int MODE>
void run(hipStream_t s, const GemvRtArgs& a) {
    size_t lds = (size_t)NB * a.K * sizeof(T) + (a.x ? 0 : (size_t)(a.D + a.groups) * sizeof(float));
    if (lds > 64 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&k_gemv_rt<T, NB, MODE>),
                                  hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL((k_gemv_rt<T, NB, MODE>), dim3(gemv_rt_blocks(a, (GemvRtMode)MODE)), dim3(256), lds, s, a);
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

template <typename T>
void run_t(hipStream_t s, GemvRtMode mode, const GemvRtArgs& a) {
    if (a.B <= 1) run_mode<T, 1>(s, mode, a);
    else run_mode<T, 2>(s, mode, a);
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

int gemv_rt_max_batch() { return 2; }

bool gemv_rt_fits(int B, int K, Act act) {
    return B <= gemv_rt_max_batch() && (size_t)gemv_rt_max_batch() * K * (act == ACT_F32 ? 4 : 2) <= 96 * 1024;
}

int gemv_rt_blocks(const GemvRtArgs& a, GemvRtMode mode) {
    const int units = (a.N + unit_outs(mode) - 1) / unit_outs(mode);
    return std::max(1, std::min((units + 3) / 4, 2048));
}

void gemv_rt(hipStream_t s, Act act, GemvRtMode mode, const GemvRtArgs& a) {
    if (act == ACT_F32) run_t<float>(s, mode, a);
    else run_t<uint16_t>(s, mode, a);
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
