// kernels_matmul.hip -- matrix products of the layered decoders: any M and N, K a multiple of 8.
//
// bf16 activations run on the prefill GEMM kernels (kernels_gemm.hip: LDS-DMA panel, warp-specialised and 8-phase
// forms), a few instantiations chosen by shape; fp32 activations on a plain fp32 tile kernel (no reduced-precision
// matrix mode).  Weights are bf16 [N][ldw] in both.
#define PGMI_GEMM_KERNELS_ONLY
#include "kernels_gemm.hip"

#include <algorithm>

#include "act.h"
#include "decoder.h"

namespace pgmi {

namespace {

// ---------------------------------------------------------------- fp32
constexpr int FT = 64, FK = 16;

__global__ void __launch_bounds__(256) k_matmul_f32(const float* __restrict__ A, int lda, const uint16_t* __restrict__ W,
                                                    int ldw, int M, int N, int K, const uint16_t* __restrict__ bias,
                                                    float* __restrict__ out, int ldo) {
    __shared__ float As[FK][FT + 4], Bs[FK][FT + 4];
    const int tid = threadIdx.x, m0 = blockIdx.y * FT, n0 = blockIdx.x * FT;
    const int tm = (tid >> 4) * 4, tn = (tid & 15) * 4;
    float acc[4][4] = {};
    for (int k0 = 0; k0 < K; k0 += FK) {
#pragma unroll
        for (int i = 0; i < FT * FK / 256; ++i) {
            const int e = tid + 256 * i, r = e / FK, k = e % FK;
            const int m = m0 + r, n = n0 + r, kk = k0 + k;
            As[k][r] = (m < M && kk < K) ? A[(long)m * lda + kk] : 0.0f;
            Bs[k][r] = (n < N && kk < K) ? bf2f(W[(long)n * ldw + kk]) : 0.0f;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < FK; ++k) {
            float a[4], b[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) { a[i] = As[k][tm + i]; b[i] = Bs[k][tn + i]; }
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(a[i], b[j], acc[i][j]);
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int m = m0 + tm + i, n = n0 + tn + j;
            if (m < M && n < ldo) out[(long)m * ldo + n] = n < N ? acc[i][j] + (bias ? bf2f(bias[n]) : 0.0f) : 0.0f;
        }
}

// [M][2N] gate|up -> [M][ldo]
__global__ void k_swiglu_f32(const float* __restrict__ gu, int M, int N, float* __restrict__ out, int ldo) {
    for (long i = blockIdx.x * 256L + threadIdx.x; i < (long)M * ldo; i += gridDim.x * 256L) {
        const long m = i / ldo;
        const int n = (int)(i % ldo);
        out[i] = n < N ? siluf_(gu[m * 2 * N + n]) * gu[m * 2 * N + N + n] : 0.0f;
    }
}

// zeros in columns N .. ldo-1 (the GEMM kernels write columns < N only)
__global__ void k_zero_cols(uint16_t* __restrict__ out, int M, int N, int ldo) {
    const int w = ldo - N;
    for (long i = blockIdx.x * 256L + threadIdx.x; i < (long)M * w; i += gridDim.x * 256L)
        out[i / w * ldo + N + i % w] = 0;
}

// ---------------------------------------------------------------- bf16
template <auto KERN>
void lds_attr(size_t lds) {
    static bool done = false;
    if (!done && lds > 64 * 1024) {
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(KERN), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        done = true;
    }
}

struct Job {
    hipStream_t s;
    const uint16_t* A;
    int lda;
    const uint16_t* W;
    int ldw, M, N, K;
    EpiArgs ea;
    float* ws;
    int split;
    long up;
    int per() const {
        const int nkt = (K + 63) / 64;
        return (nkt + split - 1) / split;
    }
};

// 64 x 64 tiles (dual: 64 x 32 + 32)
template <int EPI, bool SPLIT>
void run_p64(const Job& j) {
    constexpr int NB = epi_dual(EPI) ? 2 : 1, TN = NB == 2 ? 1 : 2, ST = 4;
    constexpr int BM = 64, BN = 2 * TN * 16;
    constexpr size_t lds = (size_t)ST * (BM + NB * BN) * 128;
    const int n_mt = (j.M + BM - 1) / BM, n_nt = (j.N + BN - 1) / BN;
    lds_attr<&k_gemm_p<4, 2, 2, TN, NB, ST, EPI, SPLIT>>(lds);
    hipLaunchKernelGGL((k_gemm_p<4, 2, 2, TN, NB, ST, EPI, SPLIT>), dim3(n_mt * n_nt, j.split), dim3(256), lds, j.s, j.A,
                       j.lda, j.W, j.ldw, j.M, j.N, j.K, j.per(), j.ea, j.ws, j.up, n_mt, 0);
}

// 128 x 128 tiles, loader waves (dual: 128 x 64 + 64)
template <int EPI, bool SPLIT>
void run_w128(const Job& j) {
    constexpr int NB = epi_dual(EPI) ? 2 : 1, TN = NB == 2 ? 1 : 2, ST = 4;
    constexpr int BM = 128, BN = 4 * TN * 16;
    constexpr size_t lds = (size_t)ST * (BM + NB * BN) * 128;
    const int n_mt = (j.M + BM - 1) / BM, n_nt = (j.N + BN - 1) / BN;
    lds_attr<&k_gemm_w<8, 2, 4, TN, NB, ST, 4, EPI, SPLIT>>(lds);
    hipLaunchKernelGGL((k_gemm_w<8, 2, 4, TN, NB, ST, 4, EPI, SPLIT>), dim3(n_mt * n_nt, j.split), dim3(64 * 12), lds, j.s,
                       j.A, j.lda, j.W, j.ldw, j.M, j.N, j.K, j.per(), j.ea, j.ws, j.up, n_mt, n_mt == 1 ? 1 << 30 : 0);
}

// 256 x 256 tiles, 8 phases (dual: 256 x 128 + 128); K % 64 == 0
template <int EPI, bool SPLIT>
void run_e256(const Job& j) {
    constexpr int BM = 256, BN = epi_dual(EPI) ? 128 : 256;
    constexpr size_t lds = (size_t)2 * (2 * 16 * 8 * 128 + 2 * 128 * 128);
    const int n_mt = (j.M + BM - 1) / BM, n_nt = (j.N + BN - 1) / BN;
    lds_attr<&k_gemm_8p<8, EPI, SPLIT>>(lds);
    hipLaunchKernelGGL((k_gemm_8p<8, EPI, SPLIT>), dim3(n_mt * n_nt, j.split), dim3(512), lds, j.s, j.A, j.lda, j.W, j.ldw,
                       j.M, j.N, j.K, j.per(), j.ea, j.ws, j.up, n_mt, 0);
}

long tiles(int M, int N, int bm, int bn) { return (long)((M + bm - 1) / bm) * ((N + bn - 1) / bn); }

template <int EPI, bool SPLIT>
void run_plan(const Job& j) {
    const int bn2 = epi_dual(EPI) ? 2 : 1;
    if (j.K % 64 == 0 && j.K >= 1024 && j.M >= 1024 && tiles(j.M, j.N, 256, 256 / bn2) * j.split >= 160)
        run_e256<EPI, SPLIT>(j);
    else if (j.N > 192 && tiles(j.M, j.N, 128, 128 / bn2) * j.split >= 128)
        run_w128<EPI, SPLIT>(j);
    else
        run_p64<EPI, SPLIT>(j);
}

// K slices for a product whose tiles alone leave CUs idle
int pick_split(int M, int N, int K, size_t out_bytes) {
    const int nkt = (K + 63) / 64;
    const long t = tiles(M, N, 64, 64);
    int split = 1;
    while (t * split < 256 && split < 8 && nkt / (split * 2) >= 4) split *= 2;
    while (split > 1 && (size_t)split * M * N * sizeof(float) > out_bytes) split /= 2;
    if (split > 1) {  // every slice non-empty
        const int per = (nkt + split - 1) / split;
        split = (nkt + per - 1) / per;
    }
    return split;
}

}  // namespace

int matmul_rt(hipStream_t s, Act act, const void* A, int lda, const uint16_t* W, int ldw, int M, int N, int K,
              RtOut mode, const uint16_t* bias, void* out, int ldo, size_t out_bytes, float* scratch) {
    if (M <= 0 || N <= 0) return 1;
    if (act == ACT_F32) {
        const float* a = reinterpret_cast<const float*>(A);
        const bool dual = mode == RT_SWIGLU, plain = mode == RT_F32 || mode == RT_SLABS;
        const int n = dual ? 2 * N : N;
        float* o = dual ? scratch : reinterpret_cast<float*>(out);
        const int ld = dual ? n : plain ? N : ldo;
        hipLaunchKernelGGL(k_matmul_f32, dim3((ld + FT - 1) / FT, (M + FT - 1) / FT), dim3(256), 0, s, a, lda, W, ldw, M,
                           n, K, plain ? nullptr : bias, o, ld);
        if (dual)
            hipLaunchKernelGGL(k_swiglu_f32, dim3(1024), dim3(256), 0, s, scratch, M, N, reinterpret_cast<float*>(out), ldo);
        return 1;
    }
    Job j{s, reinterpret_cast<const uint16_t*>(A), lda, W, ldw, M, N, K, {}, nullptr, 1, 0};
    if (mode == RT_F32 || mode == RT_SLABS) {
        j.ws = reinterpret_cast<float*>(out);
        if (mode == RT_SLABS) j.split = pick_split(M, N, K, out_bytes);
        run_plan<EPI_STORE, true>(j);
        return j.split;
    }
    j.ea.out = reinterpret_cast<uint16_t*>(out);
    j.ea.ldo = ldo;
    j.ea.bias = bias;
    if (mode == RT_SWIGLU) {
        j.up = (long)N * ldw;
        run_plan<EPI_SWIGLU, false>(j);
    } else if (bias) {
        run_plan<EPI_BIAS, false>(j);
    } else {
        run_plan<EPI_STORE, false>(j);
    }
    if (ldo > N && ldo - N < 8)
        hipLaunchKernelGGL(k_zero_cols, dim3(256), dim3(256), 0, s, reinterpret_cast<uint16_t*>(out), M, N, ldo);
    return 1;
}

}  // namespace pgmi
