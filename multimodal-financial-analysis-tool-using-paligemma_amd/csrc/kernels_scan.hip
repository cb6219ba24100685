// kernels_scan.hip -- the recurrent mechanisms of the layered decoders, over packed rows of unequal sequences:
// the causal convolution and selective scan of Mamba, and the minimal gated recurrence (minGRU).
//
// A sequence's rows are cut into chunks.  With one chunk a workgroup walks it from the sequence's state.  With
// several, three launches run them in parallel: (A) every chunk but the last from a zero state (its end
// state and its total decay), (B) one short walk over the chunks that turns these into the chunks' entry states,
// (C) every chunk again from its entry state, writing the outputs; the last chunk leaves the sequence's state.
// The decay of a chunk is exp(A sum(dt)), so (A) keeps sums of steps and no products.
#include <algorithm>

#include "act.h"
#include "decoder.h"

namespace pgmi {

namespace {

// ---------------------------------------------------------------- causal convolution + silu
// the input at the sequence's relative row p < 0: the taps kept from earlier steps (zero at the start)
template <typename T>
__device__ __forceinline__ float tap_at(const SeqInfo& q, const float* taps, int K, int C, int p, int c) {
    const int j = K - 1 + p;
    return (q.start > 0 && j >= 0) ? taps[((long)q.slot * (K - 1) + j) * C + c] : 0.0f;
}

// V == 8: eight channels per lane, KT taps held in registers, each wave a run of consecutive rows.
// KT == 0: any number of taps, one channel per lane.
template <typename T, int KT>
__global__ void __launch_bounds__(256) k_conv_silu(const T* __restrict__ xz, int ldxz, int C, int K,
                                                   const uint16_t* __restrict__ w, const uint16_t* __restrict__ b,
                                                   const SeqInfo* __restrict__ seqs, const ChunkInfo* __restrict__ chunks,
                                                   const float* __restrict__ taps, T* __restrict__ out, int ldo) {
    const ChunkInfo ck = chunks[blockIdx.y];
    const SeqInfo q = seqs[ck.seq];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int run = (ck.len + 3) / 4, r0 = wave * run, r1 = min(ck.len, r0 + run);
    if constexpr (KT > 0) {
        const int c = (blockIdx.x * 64 + lane) * 8;
        if (c >= C || r0 >= r1) return;
        float wk[KT][8], bias[8], win[KT][8];
        {
            float f[KT * 8];
#pragma unroll
            for (int t = 0; t < KT; ++t) {
                float g[8];
                ld8(w + (long)c * KT + 8 * t, g);
#pragma unroll
                for (int v = 0; v < 8; ++v) f[8 * t + v] = g[v];
            }
#pragma unroll
            for (int t = 0; t < KT; ++t)
#pragma unroll
                for (int v = 0; v < 8; ++v) wk[t][v] = f[v * KT + t];
        }
        ld8(b + c, bias);
#pragma unroll
        for (int t = 0; t < KT - 1; ++t) {  // the KT - 1 inputs before the run
            const int p = ck.rel + r0 - (KT - 1) + t;
            if (p >= 0) {
                ld8(xz + (long)(q.off + p) * ldxz + c, win[t]);
            } else {
#pragma unroll
                for (int v = 0; v < 8; ++v) win[t][v] = tap_at<T>(q, taps, KT, C, p, c + v);
            }
        }
#pragma unroll 4
        for (int r = r0; r < r1; ++r) {
            ld8(xz + (long)(ck.row + r) * ldxz + c, win[KT - 1]);
            float y[8];
#pragma unroll
            for (int v = 0; v < 8; ++v) {
                y[v] = bias[v];
#pragma unroll
                for (int t = 0; t < KT; ++t) y[v] = fmaf(wk[t][v], win[t][v], y[v]);
                y[v] = siluf_(y[v]);
#pragma unroll
                for (int t = 0; t + 1 < KT; ++t) win[t][v] = win[t + 1][v];
            }
            st8(out + (long)(ck.row + r) * ldo + c, y);
        }
    } else {
        const int c = blockIdx.x * 64 + lane;
        if (c >= ldo) return;
        for (int r = r0; r < r1; ++r) {
            float y = 0.0f;
            if (c < C) {
                y = bf2f(b[c]);
                for (int k = 0; k < K; ++k) {
                    const int p = ck.rel + r - (K - 1) + k;
                    const float x = p >= 0 ? ldf(xz + (long)(q.off + p) * ldxz + c) : tap_at<T>(q, taps, K, C, p, c);
                    y = fmaf(bf2f(w[(long)c * K + k]), x, y);
                }
                y = siluf_(y);
            }
            stf(out + (long)(ck.row + r) * ldo + c, y);
        }
    }
}

// the last K - 1 inputs of each sequence become its taps (one thread per channel, ascending j: new tap j is
// an older tap at j + len, not yet overwritten, or a row of this step)
template <typename T>
__global__ void __launch_bounds__(256) k_conv_taps(const T* __restrict__ xz, int ldxz, int C, int K,
                                                   const SeqInfo* __restrict__ seqs, float* __restrict__ taps) {
    const SeqInfo q = seqs[blockIdx.y];
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= C) return;
    for (int j = 0; j < K - 1; ++j) {
        const int p = q.len - (K - 1) + j;
        const float v = p >= 0 ? ldf(xz + (long)(q.off + p) * ldxz + c) : tap_at<T>(q, taps, K, C, p, c);
        taps[((long)q.slot * (K - 1) + j) * C + c] = v;
    }
}

template <typename T>
__global__ void __launch_bounds__(256) k_scan_inputs(const float* __restrict__ slabs, int split, int rows, int R, int N,
                                                     T* __restrict__ dtl, int ldd, float* __restrict__ bc) {
    const int M = R + 2 * N;
    const int row = blockIdx.x;
    for (int i = threadIdx.x; i < M; i += 256) {
        float v = 0.0f;
        for (int z = 0; z < split; ++z) v += slabs[((long)z * rows + row) * M + i];
        if (i < R) stf(dtl + (long)row * ldd + i, v);
        else bc[(long)row * 2 * N + i - R] = v;
    }
    for (int i = R + threadIdx.x; i < ldd; i += 256) stf(dtl + (long)row * ldd + i, 0.0f);
}

// ---------------------------------------------------------------- selective scan
constexpr int kSub = 32;  // rows whose B | C are staged in LDS at a time
constexpr int kPre = 8;   // rows whose step, input and gate are in flight ahead of the recurrence

// LPC lanes per channel, NPL states per lane (N <= LPC * NPL; states past N are inert: B = C = 0).
// PHASE 0: (A) zero entry state, no output; 1: (C) / single-chunk walk.
template <typename T, int NPL, int LPC, int PHASE>
__global__ void __launch_bounds__(256) k_scan(ScanArgs a) {
    constexpr int CPB = 256 / LPC;  // channels per workgroup
    constexpr int NP = NPL * LPC;
    __shared__ __attribute__((aligned(16))) float sB[kSub][NP], sC[PHASE ? kSub : 1][PHASE ? NP : 4];
    const ChunkInfo ck = a.chunks[blockIdx.y];
    const bool last = ck.idx + 1 == ck.nch;
    if (PHASE == 0 && last) return;  // only earlier chunks feed others
    const SeqInfo q = a.seqs[ck.seq];
    const int tid = threadIdx.x, sub = tid % LPC;
    const int c = blockIdx.x * CPB + tid / LPC;
    const bool ok = c < a.C;
    const int cc = ok ? c : a.C - 1;
    const int n0 = sub * NPL;
    const int N = a.N;
    float A[NPL], S[NPL];
    const long sbase = ((long)q.slot * a.C + cc) * N, cbase = ((long)blockIdx.y * a.C + cc) * N;
#pragma unroll
    for (int i = 0; i < NPL; ++i) {
        const int n = n0 + i;
        // dt A in powers of two: exp(dt A) = exp2(dt A log2 e)
        A[i] = n < N ? -expf(bf2f(a.A_log[(long)cc * N + n])) * 1.4426950408889634f : 0.0f;
        S[i] = 0.0f;
        if (PHASE == 1 && n < N) {
            if (ck.nch > 1) S[i] = a.cstate[cbase + n];
            else if (q.start > 0) S[i] = a.state[sbase + n];
        }
    }
    const float bias = bf2f(a.dtb[cc]), Dc = bf2f(a.Dw[cc]);
    const float* __restrict__ dp = a.dt + (long)ck.row * a.C + cc;
    const T* __restrict__ xp = reinterpret_cast<const T*>(a.x) + (long)ck.row * a.ldx + cc;
    const T* __restrict__ zp = reinterpret_cast<const T*>(a.z) + (long)ck.row * a.ldz + cc;
    T* __restrict__ yp = reinterpret_cast<T*>(a.y) + (long)ck.row * a.ldy + c;
    float dsum = 0.0f;
    float pd[kPre];
    T px[kPre], pz[kPre];
    auto fetch = [&](int t0) {  // rows past the chunk repeat its last one (never used)
#pragma unroll
        for (int t = 0; t < kPre; ++t) {
            const long r = min(t0 + t, ck.len - 1);
            pd[t] = dp[r * a.C];
            px[t] = xp[r * a.ldx];
            if constexpr (PHASE == 1) pz[t] = zp[r * a.ldz];
        }
    };
    fetch(0);
    for (int t0 = 0; t0 < ck.len; t0 += kSub) {
        const int nt = min(kSub, ck.len - t0);
        __syncthreads();
        for (int i = tid; i < nt * NP; i += 256) {
            const int t = i / NP, n = i % NP;
            const float* r = a.bc + (long)(ck.row + t0 + t) * 2 * N;
            sB[t][n] = n < N ? r[n] : 0.0f;
            if constexpr (PHASE == 1) sC[t][n] = n < N ? r[N + n] : 0.0f;
        }
        __syncthreads();
        for (int tb = 0; tb < nt; tb += kPre) {
            float dt[kPre], x[kPre], g[kPre];
#pragma unroll
            for (int t = 0; t < kPre; ++t) {
                dt[t] = softplus_of<T>(pd[t] + bias);
                x[t] = ldf(&px[t]);
                g[t] = 0.0f;
                if constexpr (PHASE == 1) g[t] = siluf_(ldf(&pz[t]));
            }
            if (t0 + tb + kPre < ck.len) fetch(t0 + tb + kPre);
#pragma unroll
            for (int t = 0; t < kPre; ++t) {
                if (tb + t < nt) {
                    const float dx = dt[t] * x[t];
                    dsum += dt[t];
                    float y = 0.0f;
#pragma unroll
                    for (int i = 0; i < NPL; i += 4) {
                        const float4 B = *reinterpret_cast<const float4*>(&sB[tb + t][n0 + i]);
                        S[i] = fmaf(__builtin_amdgcn_exp2f(dt[t] * A[i]), S[i], dx * B.x);
                        S[i + 1] = fmaf(__builtin_amdgcn_exp2f(dt[t] * A[i + 1]), S[i + 1], dx * B.y);
                        S[i + 2] = fmaf(__builtin_amdgcn_exp2f(dt[t] * A[i + 2]), S[i + 2], dx * B.z);
                        S[i + 3] = fmaf(__builtin_amdgcn_exp2f(dt[t] * A[i + 3]), S[i + 3], dx * B.w);
                        if constexpr (PHASE == 1) {
                            const float4 Cv = *reinterpret_cast<const float4*>(&sC[tb + t][n0 + i]);
                            y = fmaf(S[i], Cv.x, y);
                            y = fmaf(S[i + 1], Cv.y, y);
                            y = fmaf(S[i + 2], Cv.z, y);
                            y = fmaf(S[i + 3], Cv.w, y);
                        }
                    }
                    if constexpr (PHASE == 1) {
#pragma unroll
                        for (int o = 1; o < LPC; o <<= 1) y += __shfl_xor(y, o, 64);
                        if (sub == 0 && c < a.ldy)  // columns C .. ldy - 1 are zero
                            stf(yp + (long)(t0 + tb + t) * a.ldy, ok ? fmaf(Dc, x[t], y) * g[t] : 0.0f);
                    }
                }
            }
        }
    }
    if (!ok) return;
    if constexpr (PHASE == 0) {
#pragma unroll
        for (int i = 0; i < NPL; ++i)
            if (n0 + i < N) a.cstate[cbase + n0 + i] = S[i];
        if (sub == 0) a.csum[(long)blockIdx.y * a.C + c] = dsum;
    } else if (last) {
#pragma unroll
        for (int i = 0; i < NPL; ++i)
            if (n0 + i < N) a.state[sbase + n0 + i] = S[i];
    }
}

// (B) the chunks' entry states, in place of their end states
__global__ void __launch_bounds__(256) k_scan_carry(ScanArgs a) {
    const ChunkInfo ck = a.chunks[blockIdx.y];
    if (ck.idx != 0 || ck.nch < 2) return;  // one walk per sequence, from its first chunk
    const SeqInfo q = a.seqs[ck.seq];
    const long i = (long)blockIdx.x * 256 + threadIdx.x, CN = (long)a.C * a.N;
    if (i >= CN) return;
    const int c = (int)(i / a.N);
    const float A = -expf(bf2f(a.A_log[i])) * 1.4426950408889634f;
    float S = q.start > 0 ? a.state[(long)q.slot * CN + i] : 0.0f;
    float* e = a.cstate + (long)blockIdx.y * CN + i;
    const float* ds = a.csum + (long)blockIdx.y * a.C + c;
    const int n = ck.nch - 1;  // the last chunk left no end state
    for (int k0 = 0; k0 <= n; k0 += kPre) {
        float end[kPre], f[kPre];
#pragma unroll
        for (int k = 0; k < kPre; ++k) {
            const long r = min(k0 + k, n - 1);
            end[k] = e[r * CN];
            f[k] = ds[r * a.C];
        }
#pragma unroll
        for (int k = 0; k < kPre; ++k)
            if (k0 + k <= n) {
                e[(long)(k0 + k) * CN] = S;
                S = fmaf(__builtin_amdgcn_exp2f(A * f[k]), S, end[k]);
            }
    }
}

template <typename T, int NPL, int LPC>
void launch_scan(hipStream_t s, const ScanArgs& a) {
    const int CPB = 256 / LPC;
    const dim3 grid((std::max(a.C, a.ldy) + CPB - 1) / CPB, a.nchunk);
    if (a.multi) {
        hipLaunchKernelGGL((k_scan<T, NPL, LPC, 0>), grid, dim3(256), 0, s, a);
        const long CN = (long)a.C * a.N;
        hipLaunchKernelGGL(k_scan_carry, dim3((unsigned)((CN + 255) / 256), a.nchunk), dim3(256), 0, s, a);
    }
    hipLaunchKernelGGL((k_scan<T, NPL, LPC, 1>), grid, dim3(256), 0, s, a);
}

template <typename T>
void scan_t(hipStream_t s, const ScanArgs& a) {
    if (a.N <= 8) launch_scan<T, 8, 1>(s, a);
    else if (a.N <= 16) launch_scan<T, 16, 1>(s, a);
    else if (a.N <= 32) launch_scan<T, 16, 2>(s, a);
    else if (a.N <= 64) launch_scan<T, 16, 4>(s, a);
    else if (a.N <= 128) launch_scan<T, 16, 8>(s, a);
    else launch_scan<T, 16, 16>(s, a);
}

// ---------------------------------------------------------------- minGRU
// V channels per lane (2 where rows allow it, else 1)
template <typename T, int PHASE, int V>
__global__ void __launch_bounds__(64) k_gru(GruArgs a) {
    const ChunkInfo ck = a.chunks[blockIdx.y];
    const bool last = ck.idx + 1 == ck.nch;
    if (PHASE == 0 && last) return;
    const SeqInfo q = a.seqs[ck.seq];
    const int c = (blockIdx.x * 64 + threadIdx.x) * V;
    const T* __restrict__ zp = reinterpret_cast<const T*>(a.zug) + (long)ck.row * a.ld + c;
    T* __restrict__ yp = reinterpret_cast<T*>(a.y) + (long)ck.row * a.ldy + c;
    if (c >= a.C) {  // columns C .. ldy - 1 are zero (V == 1 only)
        if (PHASE == 1 && c < a.ldy)
            for (int t = 0; t < ck.len; ++t) stf(yp + (long)t * a.ldy, 0.0f);
        return;
    }
    float S[V], keep[V];
    float* cs = a.cstate + ((long)blockIdx.y * 2) * a.C + c;
#pragma unroll
    for (int v = 0; v < V; ++v) {
        S[v] = 0.0f;
        keep[v] = 1.0f;
        if constexpr (PHASE == 1) {
            if (ck.nch > 1) S[v] = cs[v];
            else if (q.start > 0) S[v] = a.state[(long)q.slot * a.C + c + v];
        }
    }
    struct alignas(sizeof(T) * V) Raw { T v[V]; };
    Raw rz[kPre], ru[kPre], rg[PHASE ? kPre : 1];
    auto fetch = [&](int t0) {  // rows past the chunk repeat its last one (never used)
#pragma unroll
        for (int t = 0; t < kPre; ++t) {
            const T* r = zp + (long)min(t0 + t, ck.len - 1) * a.ld;
            rz[t] = *reinterpret_cast<const Raw*>(r);
            ru[t] = *reinterpret_cast<const Raw*>(r + a.C);
            if constexpr (PHASE == 1) rg[t] = *reinterpret_cast<const Raw*>(r + 2 * a.C);
        }
    };
    fetch(0);
    for (int t0 = 0; t0 < ck.len; t0 += kPre) {
        float z[kPre][V], u[kPre][V], g[kPre][V];
#pragma unroll
        for (int t = 0; t < kPre; ++t)
#pragma unroll
            for (int v = 0; v < V; ++v) {
                z[t][v] = ldf(&rz[t].v[v]);
                u[t][v] = ldf(&ru[t].v[v]);
                if constexpr (PHASE == 1) g[t][v] = ldf(&rg[t].v[v]);
            }
        if (t0 + kPre < ck.len) fetch(t0 + kPre);
#pragma unroll
        for (int t = 0; t < kPre; ++t) {
            if (t0 + t >= ck.len) break;
            float y[V];
#pragma unroll
            for (int v = 0; v < V; ++v) {
                const float zz = sigmoidf_(z[t][v]);
                S[v] = fmaf(1.0f - zz, S[v], zz * gru_candidate(u[t][v]));
                if constexpr (PHASE == 0) keep[v] *= 1.0f - zz;
                else y[v] = S[v] * siluf_(g[t][v]);
            }
            if constexpr (PHASE == 1) {
                Raw o;
#pragma unroll
                for (int v = 0; v < V; ++v) stf(&o.v[v], y[v]);
                *reinterpret_cast<Raw*>(yp + (long)(t0 + t) * a.ldy) = o;
            }
        }
    }
#pragma unroll
    for (int v = 0; v < V; ++v) {
        if constexpr (PHASE == 0) {
            cs[v] = S[v];
            cs[a.C + v] = keep[v];
        } else if (last) {
            a.state[(long)q.slot * a.C + c + v] = S[v];
        }
    }
}

__global__ void __launch_bounds__(64) k_gru_carry(GruArgs a) {
    const ChunkInfo ck = a.chunks[blockIdx.y];
    if (ck.idx != 0 || ck.nch < 2) return;
    const SeqInfo q = a.seqs[ck.seq];
    const int c = blockIdx.x * 64 + threadIdx.x;
    if (c >= a.C) return;
    float S = q.start > 0 ? a.state[(long)q.slot * a.C + c] : 0.0f;
    float* e = a.cstate + ((long)blockIdx.y * 2) * a.C + c;
    const int n = ck.nch - 1;
    for (int k0 = 0; k0 <= n; k0 += kPre) {
        float end[kPre], keep[kPre];
#pragma unroll
        for (int k = 0; k < kPre; ++k) {
            const long r = min(k0 + k, n - 1);
            end[k] = e[r * 2 * a.C];
            keep[k] = e[r * 2 * a.C + a.C];
        }
#pragma unroll
        for (int k = 0; k < kPre; ++k)
            if (k0 + k <= n) {
                e[(long)(k0 + k) * 2 * a.C] = S;
                S = fmaf(keep[k], S, end[k]);
            }
    }
}

template <typename T, int V>
void gru_v(hipStream_t s, const GruArgs& a) {
    const int cols = std::max(a.C, V == 1 ? a.ldy : a.C);
    const dim3 grid((cols + 64 * V - 1) / (64 * V), a.nchunk);
    if (a.multi) {
        hipLaunchKernelGGL((k_gru<T, 0, V>), grid, dim3(64), 0, s, a);
        hipLaunchKernelGGL(k_gru_carry, dim3((a.C + 63) / 64, a.nchunk), dim3(64), 0, s, a);
    }
    hipLaunchKernelGGL((k_gru<T, 1, V>), grid, dim3(64), 0, s, a);
}

template <typename T>
void gru_t(hipStream_t s, const GruArgs& a) {
    if (a.C % 8 == 0 && a.ld % 8 == 0) gru_v<T, 2>(s, a);
    else gru_v<T, 1>(s, a);
}

template <typename T>
void conv_t(hipStream_t s, const T* xz, int ldxz, int C, int K, const uint16_t* w, const uint16_t* b,
            const SeqInfo* seqs, int nseq, const ChunkInfo* chunks, int nchunk, float* taps, T* out, int ldo) {
    const dim3 gv((C / 8 + 63) / 64, nchunk), g1((ldo + 63) / 64, nchunk), blk(256);
#define CONV_(kt, grid) hipLaunchKernelGGL((k_conv_silu<T, kt>), grid, blk, 0, s, xz, ldxz, C, K, w, b, seqs, chunks, taps, out, ldo)
    const bool vec = C % 8 == 0 && ldxz % 8 == 0;
    if (vec && K == 2) CONV_(2, gv);
    else if (vec && K == 3) CONV_(3, gv);
    else if (vec && K == 4) CONV_(4, gv);
    else if (vec && K == 5) CONV_(5, gv);
    else CONV_(0, g1);
#undef CONV_
    if (K > 1)
        hipLaunchKernelGGL((k_conv_taps<T>), dim3((C + 255) / 256, nseq), dim3(256), 0, s, xz, ldxz, C, K, seqs, taps);
}

}  // namespace

int scan_max_state() { return 256; }

void conv_silu(hipStream_t s, Act act, const void* xz, int ldxz, int C, int K, const uint16_t* w, const uint16_t* b,
               const SeqInfo* seqs, int nseq, const ChunkInfo* chunks, int nchunk, float* taps, void* out, int ldo) {
    if (act == ACT_F32)
        conv_t(s, reinterpret_cast<const float*>(xz), ldxz, C, K, w, b, seqs, nseq, chunks, nchunk, taps,
               reinterpret_cast<float*>(out), ldo);
    else
        conv_t(s, reinterpret_cast<const uint16_t*>(xz), ldxz, C, K, w, b, seqs, nseq, chunks, nchunk, taps,
               reinterpret_cast<uint16_t*>(out), ldo);
}

void scan_inputs(hipStream_t s, Act act, const float* slabs, int split, int rows, int R, int N, void* dtl, int ldd,
                 float* bc) {
    if (act == ACT_F32)
        hipLaunchKernelGGL((k_scan_inputs<float>), dim3(rows), dim3(256), 0, s, slabs, split, rows, R, N,
                           reinterpret_cast<float*>(dtl), ldd, bc);
    else
        hipLaunchKernelGGL((k_scan_inputs<uint16_t>), dim3(rows), dim3(256), 0, s, slabs, split, rows, R, N,
                           reinterpret_cast<uint16_t*>(dtl), ldd, bc);
}

void selective_scan(hipStream_t s, Act act, const ScanArgs& a) {
    if (act == ACT_F32) scan_t<float>(s, a);
    else scan_t<uint16_t>(s, a);
}

void mingru_scan(hipStream_t s, Act act, const GruArgs& a) {
    if (act == ACT_F32) gru_t<float>(s, a);
    else gru_t<uint16_t>(s, a);
}

}  // namespace pgmi
