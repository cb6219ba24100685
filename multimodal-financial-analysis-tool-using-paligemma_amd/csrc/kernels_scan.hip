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

template <typename T, int V>
__global__ void __launch_bounds__(256) k_conv_silu(const T* __restrict__ xz, int ldxz, int C, int K,
                                                   const uint16_t* __restrict__ w, const uint16_t* __restrict__ b,
                                                   const SeqInfo* __restrict__ seqs, const ChunkInfo* __restrict__ chunks,
                                                   const float* __restrict__ taps, T* __restrict__ out, int ldo) {
    const ChunkInfo ck = chunks[blockIdx.y];
    const SeqInfo q = seqs[ck.seq];
    const int c = (blockIdx.x * 64 + (threadIdx.x & 63)) * V;
    if (c >= ldo) return;
    for (int r = threadIdx.x >> 6; r < ck.len; r += 4) {
        const int rel = ck.rel + r;
        float acc[V];
#pragma unroll
        for (int v = 0; v < V; ++v) acc[v] = c + v < C ? bf2f(b[c + v]) : 0.0f;
        for (int k = 0; k < K; ++k) {
            const int p = rel - (K - 1) + k;
            if constexpr (V == 8) {
                if (p >= 0) {
                    float x[8];
                    ld8(xz + (long)(q.off + p) * ldxz + c, x);
#pragma unroll
                    for (int v = 0; v < 8; ++v) acc[v] = fmaf(bf2f(w[(long)(c + v) * K + k]), x[v], acc[v]);
                } else {
#pragma unroll
                    for (int v = 0; v < 8; ++v)
                        acc[v] = fmaf(bf2f(w[(long)(c + v) * K + k]), tap_at<T>(q, taps, K, C, p, c + v), acc[v]);
                }
            } else if (c < C) {
                const float x = p >= 0 ? ldf(xz + (long)(q.off + p) * ldxz + c) : tap_at<T>(q, taps, K, C, p, c);
                acc[0] = fmaf(bf2f(w[(long)c * K + k]), x, acc[0]);
            }
        }
#pragma unroll
        for (int v = 0; v < V; ++v) acc[v] = c + v < C ? siluf_(acc[v]) : 0.0f;
        T* o = out + (long)(ck.row + r) * ldo + c;
        if constexpr (V == 8) st8(o, acc);
        else stf(o, acc[0]);
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

// LPC lanes per channel, NPL states per lane (N <= LPC * NPL; states past N are inert: B = C = 0).
// PHASE 0: (A) zero entry state, no output; 1: (C) / single-chunk walk.
template <typename T, int NPL, int LPC, int PHASE>
__global__ void __launch_bounds__(256) k_scan(ScanArgs a) {
    constexpr int CPB = 256 / LPC;  // channels per workgroup
    constexpr int NP = NPL * LPC;
    __shared__ float sB[kSub][NP], sC[PHASE ? kSub : 1][PHASE ? NP : 1];
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
    const T* xp = reinterpret_cast<const T*>(a.x);
    const T* zp = reinterpret_cast<const T*>(a.z);
    T* yp = reinterpret_cast<T*>(a.y);
    float dsum = 0.0f;
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
#pragma unroll 4
        for (int t = 0; t < nt; ++t) {
            const long row = ck.row + t0 + t;
            const float dt = softplusf_(a.dt[row * a.C + cc] + bias);
            const float x = ldf(xp + row * a.ldx + cc);
            const float dx = dt * x;
            dsum += dt;
            float y = 0.0f;
#pragma unroll
            for (int i = 0; i < NPL; ++i) {
                S[i] = fmaf(__builtin_amdgcn_exp2f(dt * A[i]), S[i], dx * sB[t][n0 + i]);
                if constexpr (PHASE == 1) y = fmaf(S[i], sC[t][n0 + i], y);
            }
            if constexpr (PHASE == 1) {
#pragma unroll
                for (int o = 1; o < LPC; o <<= 1) y += __shfl_xor(y, o, 64);
                if (sub == 0 && c < a.ldy) {  // columns C .. ldy - 1 are zero
                    y = fmaf(Dc, x, y);
                    stf(yp + row * a.ldy + c, ok ? y * siluf_(ldf(zp + row * a.ldz + cc)) : 0.0f);
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
    for (int k = 0; k < ck.nch; ++k) {
        float* e = a.cstate + (long)(blockIdx.y + k) * CN + i;
        const float end = k + 1 < ck.nch ? *e : 0.0f;
        *e = S;
        if (k + 1 < ck.nch)
            S = fmaf(__builtin_amdgcn_exp2f(A * a.csum[(long)(blockIdx.y + k) * a.C + c]), S, end);
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
    else if (a.N <= 16) launch_scan<T, 8, 2>(s, a);
    else if (a.N <= 32) launch_scan<T, 8, 4>(s, a);
    else if (a.N <= 64) launch_scan<T, 8, 8>(s, a);
    else if (a.N <= 128) launch_scan<T, 8, 16>(s, a);
    else launch_scan<T, 8, 32>(s, a);
}

// ---------------------------------------------------------------- minGRU
template <typename T, int PHASE>
__global__ void __launch_bounds__(256) k_gru(GruArgs a) {
    const ChunkInfo ck = a.chunks[blockIdx.y];
    const bool last = ck.idx + 1 == ck.nch;
    if (PHASE == 0 && last) return;
    const SeqInfo q = a.seqs[ck.seq];
    const int c = blockIdx.x * 256 + threadIdx.x;
    const T* zp = reinterpret_cast<const T*>(a.zug);
    T* yp = reinterpret_cast<T*>(a.y);
    if (c >= a.C) {
        if (PHASE == 1 && c < a.ldy)
            for (int t = 0; t < ck.len; ++t) stf(yp + (long)(ck.row + t) * a.ldy + c, 0.0f);
        return;
    }
    float S = 0.0f, keep = 1.0f;
    float* cs = a.cstate + ((long)blockIdx.y * 2) * a.C + c;
    if constexpr (PHASE == 1) {
        if (ck.nch > 1) S = cs[0];
        else if (q.start > 0) S = a.state[(long)q.slot * a.C + c];
    }
#pragma unroll 4
    for (int t = 0; t < ck.len; ++t) {
        const T* r = zp + (long)(ck.row + t) * a.ld + c;
        const float z = sigmoidf_(ldf(r)), cand = gru_candidate(ldf(r + a.C));
        S = fmaf(1.0f - z, S, z * cand);
        if constexpr (PHASE == 0) keep *= 1.0f - z;
        else stf(yp + (long)(ck.row + t) * a.ldy + c, S * siluf_(ldf(r + 2 * a.C)));
    }
    if constexpr (PHASE == 0) {
        cs[0] = S;
        cs[a.C] = keep;
    } else if (last) {
        a.state[(long)q.slot * a.C + c] = S;
    }
}

__global__ void __launch_bounds__(256) k_gru_carry(GruArgs a) {
    const ChunkInfo ck = a.chunks[blockIdx.y];
    if (ck.idx != 0 || ck.nch < 2) return;
    const SeqInfo q = a.seqs[ck.seq];
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= a.C) return;
    float S = q.start > 0 ? a.state[(long)q.slot * a.C + c] : 0.0f;
    for (int k = 0; k < ck.nch; ++k) {
        float* e = a.cstate + ((long)(blockIdx.y + k) * 2) * a.C + c;
        const float end = k + 1 < ck.nch ? e[0] : 0.0f, keep = k + 1 < ck.nch ? e[a.C] : 1.0f;
        e[0] = S;
        S = fmaf(keep, S, end);
    }
}

template <typename T>
void gru_t(hipStream_t s, const GruArgs& a) {
    const dim3 grid((std::max(a.C, a.ldy) + 255) / 256, a.nchunk);
    if (a.multi) {
        hipLaunchKernelGGL((k_gru<T, 0>), grid, dim3(256), 0, s, a);
        hipLaunchKernelGGL(k_gru_carry, grid, dim3(256), 0, s, a);
    }
    hipLaunchKernelGGL((k_gru<T, 1>), grid, dim3(256), 0, s, a);
}

template <typename T>
void conv_t(hipStream_t s, const T* xz, int ldxz, int C, int K, const uint16_t* w, const uint16_t* b,
            const SeqInfo* seqs, int nseq, const ChunkInfo* chunks, int nchunk, float* taps, T* out, int ldo) {
    if (C % 8 == 0 && ldxz % 8 == 0 && ldo % 8 == 0)
        hipLaunchKernelGGL((k_conv_silu<T, 8>), dim3((ldo / 8 + 63) / 64, nchunk), dim3(256), 0, s, xz, ldxz, C, K, w,
                           b, seqs, chunks, taps, out, ldo);
    else
        hipLaunchKernelGGL((k_conv_silu<T, 1>), dim3((ldo + 63) / 64, nchunk), dim3(256), 0, s, xz, ldxz, C, K, w, b,
                           seqs, chunks, taps, out, ldo);
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
