// kernels_moe.hip -- mixture of experts: the router's choice (group-limited, with a choice correction), and the products
// of the chosen experts over rows gathered by expert.  Router, scores and weights are fp32.
//
//   k_route           a wave per row; entries are counted and listed per expert
//   k_experts         bf16 MFMA, LDS-DMA ring with loader waves: row tiles of one expert's list, gathered by each
//                     loader lane's own source address, results scattered to the entries' rows
//   k_experts_8p      the same rows on the 8-phase 256 x 256 tiles of kernels_gemm.hip, for long lists
//   k_experts_f32     the same product on fp32 FMA tiles
//   k_experts_skinny  few rows: one workgroup per (16 outputs, used expert), MFMA straight from HBM
#define PGMI_GEMM_KERNELS_ONLY
#include "kernels_gemm.hip"

#include <algorithm>

#include "act.h"
#include "decoder.h"
#include "route.h"

namespace pgmi {

namespace {

// ---------------------------------------------------------------- routing
// dynamic LDS: per wave route_words() of its row; then the experts' counters, the places of their local lists, and per
// wave the expert and the place of its row's entries
__global__ void __launch_bounds__(1024) k_route(RouteArgs a) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, NW = blockDim.x / 64, n = a.n, words = route_words(n, a.groups);
    float* sc = sm + (long)wave * words;
    int* lcnt = reinterpret_cast<int*>(sm + (long)NW * words);
    int* base = lcnt + a.experts;
    int* who = base + a.experts + wave * 2 * a.top;
    int* rank = who + a.top;
    for (int e = threadIdx.x; e < a.experts; e += blockDim.x) lcnt[e] = 0;
    __syncthreads();
    const int row = blockIdx.x * NW + wave;
    if (row < a.rows) {
        auto logit = [&](int c) {
            float z = 0.0f;
            for (int q = 0; q < a.split; ++q) z += a.z[(long)q * a.zstride + (long)row * a.ldz + c];
            return z;
        };
        for (int c = lane; c < n; c += 64) sc[c] = logit(c);
        if (a.gate && lane == 0) a.gate[row] = 1.0f / (1.0f + expf(-logit(n)));
        wave_sync();
        route_row(sc, [&](int c) { return bf2f(a.correction[c]); }, n, a.groups, a.keep, a.top, lane, [&](int k, int e, float w) {
            const long at = (long)row * a.top + k;
            a.sel[at] = e;
            a.w[at] = w;
            who[k] = e;
            if (e < a.experts) rank[k] = atomicAdd(&lcnt[e], 1);
        });
    }
    __syncthreads();
    for (int e = threadIdx.x; e < a.experts; e += blockDim.x) base[e] = lcnt[e] > 0 ? atomicAdd(&a.cnt[e], lcnt[e]) : 0;
    __syncthreads();
    if (row < a.rows)
        for (int k = lane; k < a.top; k += 64)
            if (who[k] < a.experts) a.list[(long)who[k] * a.cap + base[who[k]] + rank[k]] = row * a.top + k;
}

// ---------------------------------------------------------------- which expert a tile belongs to
// Tiles of all experts' lists, cut in BM rows, times n_nt column tiles: an expert's tiles are consecutive, the row tiles of
// one column tile adjacent; the list is cut into 8 contiguous runs, one per XCD (workgroup lin -> XCD lin % 8).
struct TileAt {
    int e, m0, nt, cnt;  // e < 0: past the last tile
};
__device__ __forceinline__ TileAt find_tile(const int* cnt, int experts, int BM, int n_nt) {
    const int lane = threadIdx.x & 63;
    int total = 0;
    for (int e0 = 0; e0 < experts; e0 += 64) {
        const int c = e0 + lane < experts ? cnt[e0 + lane] : 0;
        int t = (c + BM - 1) / BM;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) t += __shfl_xor(t, o, 64);
        total += t;
    }
    total *= n_nt;
    const int lin = blockIdx.x, x = lin & 7, j = lin >> 3, q = total >> 3, r = total & 7;
    if (j >= q + (x < r)) return {-1, 0, 0, 0};
    int idx = x * q + min(x, r) + j;
    for (int e0 = 0; e0 < experts; e0 += 64) {
        const int c = e0 + lane < experts ? cnt[e0 + lane] : 0;
        const int t = (c + BM - 1) / BM * n_nt;
        int s = t;  // inclusive sum
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const int u = __shfl_up(s, o, 64);
            if (lane >= o) s += u;
        }
        const unsigned long long in = __ballot(idx < s);
        if (in) {
            const int w = __builtin_amdgcn_readfirstlane(__ffsll((long long)in) - 1);
            const int first = __builtin_amdgcn_readlane(s, w) - __builtin_amdgcn_readlane(t, w);
            const int cw = __builtin_amdgcn_readlane(c, w), mt = (cw + BM - 1) / BM, k = idx - first;
            return {e0 + w, (k % mt) * BM, k / mt, cw};
        }
        idx -= __builtin_amdgcn_readlane(s, 63);
    }
    return {-1, 0, 0, 0};
}

long max_tiles(const ExpertArgs& a, int BM) { return a.entries / BM + std::min(a.experts, a.entries); }

// ---------------------------------------------------------------- bf16
// BM = 32 TM rows x BN = 64 (gate and up: 64 + 64) or 128 columns x 64 deep; 8 compute waves in a 2 x 4 grid, 4 loader
// waves, ST ring slots.  The ring, its LDS image and the fragment schedule are k_gemm_w's.
constexpr int ring_slots(int TM) { return TM <= 2 ? 3 : 4; }  // small tiles: two workgroups per CU

template <int TM, int MODE>
__global__ void __launch_bounds__(64 * 12, 1) k_experts(ExpertArgs a) {
    constexpr int NW = 8, LW = 4, WM = 2, WN = 4, NB = MODE == EX_SWIGLU ? 2 : 1, TN = MODE == EX_SWIGLU ? 1 : 2, ST = ring_slots(TM);
    constexpr int BM = WM * TM * 16, BN = WN * TN * 16;
    constexpr int APC = BM / 8, PCS = APC + NB * BN / 8, GPW = (PCS + LW - 1) / LW;
    constexpr int ABYTES = BM * 128, SBYTES = (BM + NB * BN) * 128;
    extern __shared__ __attribute__((aligned(16))) uint8_t smem_e[];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const TileAt tl = find_tile(a.cnt, a.experts, BM, (a.N + BN - 1) / BN);
    if (tl.e < 0) return;
    const int n0 = tl.nt * BN, K = a.K, nkt = (K + 63) / 64;
    const int* list = a.list + (long)tl.e * a.cap;
    if (wave >= NW) {
        const int lw = wave - NW, prow = lane >> 3, pchunk = lane & 7;
        const uint16_t* src[GPW];
        int loff[GPW];
        const int gk = (pchunk ^ prow) * 8;  // lane (row r, LDS chunk c) fetches global chunk c ^ (r & 7)
        const uint16_t* We = a.W + tl.e * a.wstride;
#pragma unroll
        for (int i = 0; i < GPW; ++i) {
            int p = lw + LW * i;
            if (p >= PCS) p -= PCS;  // padding: repeat a piece (same bytes to the same LDS address)
            loff[i] = p * 1024;
            if (p < APC) {
                const int m = min(tl.m0 + p * 8 + prow, tl.cnt - 1);  // rows past the list: valid memory, never stored
                src[i] = reinterpret_cast<const uint16_t*>(a.A) + (long)(list[m] / a.gather) * a.lda + gk;
            } else {
                const int q = p - APC, bo = q / (BN / 8);
                const int n = min(n0 + (q % (BN / 8)) * 8 + prow, a.N - 1);
                src[i] = We + ((long)bo * a.N + n) * a.ldw + gk;
            }
        }
        const uint16_t* zero = reinterpret_cast<const uint16_t*>(g_zero_chunk);
        auto issue = [&](int kt, int slot) {
            const int kel = kt * 64;
            const bool ok = kel + gk < K;  // K tail: chunks at or past K read zeros (K % 8 == 0)
#pragma unroll
            for (int i = 0; i < GPW; ++i)
                __builtin_amdgcn_global_load_lds(reinterpret_cast<const void*>(ok ? src[i] + kel : zero),
                                                 (__attribute__((address_space(3))) void*)(smem_e + slot * SBYTES + loff[i]),
                                                 16, 0, 0);
        };
#pragma unroll
        for (int sI = 0; sI < ST - 1; ++sI)
            if (sI < nkt) issue(sI, sI);
        int slot_next = ST - 1;
        for (int t = 0; t < nkt; ++t) {
            const int issued = nkt < t + ST - 1 ? nkt : t + ST - 1;
            vm_wait_tiles<GPW, ST - 2>(issued - t - 1);  // tile t landed
            __builtin_amdgcn_s_barrier();
            if (t + ST - 1 < nkt) issue(t + ST - 1, slot_next);
            slot_next = slot_next + 1 == ST ? 0 : slot_next + 1;
        }
        return;
    }
    const int wm = wave / WN, wn = wave % WN;
    int ent[TM][4];  // the entries of this lane's output rows
#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int m = tl.m0 + (wm * TM + i) * 16 + (lane >> 4) * 4 + r;
            const int v = list[min(m, tl.cnt - 1)];
            ent[i][r] = m < tl.cnt ? v : -1;
        }
#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
        for (int r = 0; r < 4; ++r) asm volatile("" : "+v"(ent[i][r]));
    f32x4 acc[NB][TM][TN];
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
        for (int i = 0; i < TM; ++i)
#pragma unroll
            for (int j = 0; j < TN; ++j) acc[b][i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int swz = lane & 7;
    const int arow0 = (wm * TM * 16 + (lane & 15)) * 128, brow0 = ABYTES + (wn * TN * 16 + (lane & 15)) * 128;
    short8 fa0[TM], fb0[NB][TN], fa1[TM], fb1[NB][TN];
    auto read = [&](short8 (&fa)[TM], short8 (&fb)[NB][TN], int slot, int kk) {
        const uint8_t* sb = smem_e + slot * SBYTES;
        const int ch = ((kk * 4 + (lane >> 4)) ^ swz) << 4;
#pragma unroll
        for (int i = 0; i < TM; ++i) fa[i] = *reinterpret_cast<const short8*>(sb + arow0 + i * 16 * 128 + ch);
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
            for (int j = 0; j < TN; ++j)
                fb[b][j] = *reinterpret_cast<const short8*>(sb + brow0 + (b * BN + j * 16) * 128 + ch);
    };
    auto mul = [&](const short8 (&fa)[TM], const short8 (&fb)[NB][TN]) {
#pragma unroll
        for (int b = 0; b < NB; ++b)
#pragma unroll
            for (int i = 0; i < TM; ++i)
#pragma unroll
                for (int j = 0; j < TN; ++j) acc[b][i][j] = mfma16(fa[i], fb[b][j], acc[b][i][j]);
    };
    int slot = 0;
    __builtin_amdgcn_s_barrier();  // tile 0 is in slot 0
    read(fa0, fb0, 0, 0);
    for (int t = 0; t < nkt; ++t) {
        __builtin_amdgcn_s_waitcnt(0xC07F);  // lgkmcnt(0): the kk = 0 fragments
        read(fa1, fb1, slot, 1);
        __builtin_amdgcn_sched_barrier(0);
        mul(fa0, fb0);
        __builtin_amdgcn_sched_barrier(0);
        slot = slot + 1 == ST ? 0 : slot + 1;
        __builtin_amdgcn_s_waitcnt(0xC07F);  // tile t's fragments are in registers
        if (t + 1 < nkt) {
            __builtin_amdgcn_s_barrier();  // tile t + 1 is in slot `slot`
            __builtin_amdgcn_sched_barrier(0);
            read(fa0, fb0, slot, 0);
        }
        __builtin_amdgcn_sched_barrier(0);
        mul(fa1, fb1);
        __builtin_amdgcn_sched_barrier(0);
    }
    uint16_t* out = reinterpret_cast<uint16_t*>(a.out);
#pragma unroll
    for (int i = 0; i < TM; ++i)
#pragma unroll
        for (int j = 0; j < TN; ++j) {
            const int n = n0 + (wn * TN + j) * 16 + (lane & 15);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                float v = acc[0][i][j][r];
                if constexpr (MODE == EX_SWIGLU) v = siluf_(v) * acc[NB - 1][i][j][r];
                if (ent[i][r] >= 0 && n < a.ldo) out[(long)ent[i][r] * a.ldo + n] = n < a.N ? f2bf(v) : 0;
            }
        }
}

template <int TM, int MODE>
void run_experts(hipStream_t s, const ExpertArgs& a) {
    constexpr int BM = 32 * TM, BN = MODE == EX_SWIGLU ? 64 : 128;
    constexpr size_t lds = (size_t)ring_slots(TM) * (BM + 128) * 128;
    static bool done = false;
    if (!done && lds > 64 * 1024) {
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&k_experts<TM, MODE>),
                                  hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        done = true;
    }
    const int n_nt = (a.N + BN - 1) / BN;
    // a run of one XCD is up to one tile longer than total / 8
    hipLaunchKernelGGL((k_experts<TM, MODE>), dim3((unsigned)((max_tiles(a, BM) * n_nt + 7) / 8 * 8)), dim3(64 * 12), lds, s, a);
}

// the row lists of gemm_8p's tiles
struct ExpertRows {
    static constexpr bool kGrouped = true;
    const ExpertArgs& a;
    const int* list = nullptr;
    int e = 0, rows = 0, m0 = 0, nt = 0;
    __device__ __forceinline__ explicit ExpertRows(const ExpertArgs& x) : a(x) {}
    __device__ __forceinline__ bool tile(int BM, int BN) {
        const TileAt t = find_tile(a.cnt, a.experts, BM, (a.N + BN - 1) / BN);
        e = t.e;
        rows = t.cnt;
        m0 = t.m0;
        nt = t.nt;
        list = a.list + (long)e * a.cap;
        return e >= 0;
    }
    __device__ __forceinline__ const uint16_t* weights() const { return a.W + e * a.wstride; }
    __device__ __forceinline__ int source(int m) const { return list[m] / a.gather; }
    __device__ __forceinline__ int target(int m) const { return list[m]; }
};

template <int TM, int MODE>
__global__ void __launch_bounds__(512, 1) k_experts_8p(ExpertArgs a) {
    EpiArgs ea;
    ea.out = reinterpret_cast<uint16_t*>(a.out);
    ea.ldo = a.ldo;
    gemm_8p<TM, MODE == EX_SWIGLU ? EPI_SWIGLU : EPI_STORE, false>(reinterpret_cast<const uint16_t*>(a.A), a.lda, a.W, a.ldw, 0,
                                                                  a.N, a.K, a.K / 64, ea, nullptr, (long)a.N * a.ldw, 0, 0,
                                                                  ExpertRows(a));
}

template <int TM, int MODE>
void run_experts_8p(hipStream_t s, const ExpertArgs& a) {
    constexpr int BM = 32 * TM, BN = MODE == EX_SWIGLU ? 128 : 256;
    constexpr size_t lds = (size_t)2 * (2 * 16 * TM * 128 + 2 * 128 * 128);
    static bool done = false;
    if (!done) {
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&k_experts_8p<TM, MODE>),
                                  hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        done = true;
    }
    const int n_nt = (a.N + BN - 1) / BN;
    hipLaunchKernelGGL((k_experts_8p<TM, MODE>), dim3((unsigned)((max_tiles(a, BM) * n_nt + 7) / 8 * 8)), dim3(512), lds, s, a);
}

// ---------------------------------------------------------------- fp32
constexpr int FT = 64, FK = 16;

template <int MODE>
__global__ void __launch_bounds__(256) k_experts_f32(ExpertArgs a) {
    constexpr int NB = MODE == EX_SWIGLU ? 2 : 1;
    __shared__ float As[FK][FT + 4], Bs[NB][FK][FT + 4];
    __shared__ int ent[FT];
    const TileAt tl = find_tile(a.cnt, a.experts, FT, (a.ldo + FT - 1) / FT);
    if (tl.e < 0) return;
    const int tid = threadIdx.x, n0 = tl.nt * FT, tm = (tid >> 4) * 4, tn = (tid & 15) * 4;
    const uint16_t* We = a.W + tl.e * a.wstride;
    if (tid < FT) ent[tid] = tl.m0 + tid < tl.cnt ? a.list[(long)tl.e * a.cap + tl.m0 + tid] : -1;
    __syncthreads();
    float acc[NB][4][4] = {};
    for (int k0 = 0; k0 < a.K; k0 += FK) {
#pragma unroll
        for (int i = 0; i < FT * FK / 256; ++i) {
            const int x = tid + 256 * i, r = x / FK, k = x % FK, n = n0 + r, kk = k0 + k;
            As[k][r] = ent[r] >= 0 && kk < a.K ? reinterpret_cast<const float*>(a.A)[(long)(ent[r] / a.gather) * a.lda + kk]
                                               : 0.0f;
#pragma unroll
            for (int b = 0; b < NB; ++b)
                Bs[b][k][r] = n < a.N && kk < a.K ? bf2f(We[((long)b * a.N + n) * a.ldw + kk]) : 0.0f;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < FK; ++k)
#pragma unroll
            for (int b = 0; b < NB; ++b)
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int j = 0; j < 4; ++j) acc[b][i][j] = fmaf(As[k][tm + i], Bs[b][k][tn + j], acc[b][i][j]);
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int e = ent[tm + i], n = n0 + tn + j;
            float v = acc[0][i][j];
            if constexpr (MODE == EX_SWIGLU) v = siluf_(v) * acc[NB - 1][i][j];
            if (e >= 0 && n < a.ldo) reinterpret_cast<float*>(a.out)[(long)e * a.ldo + n] = n < a.N ? v : 0.0f;
        }
}

// ---------------------------------------------------------------- few rows
// grid (output tiles of 16, 1 + used experts): y == 0 is the shared expert, y > 0 the (y - 1)-th used one, whose rows are
// its list.  4 waves split K; a lane reads 32 contiguous bytes of its weight row per 64-deep step, as k_skinny.
// U: 64-deep steps a wave has in flight.
template <int MODE, int U>
__global__ void __launch_bounds__(256) k_experts_skinny(ExpertArgs a) {
    constexpr int NM = MODE == EX_SWIGLU ? 2 : 1;
    __shared__ float sums[4][NM][16][17];
    const bool shared = blockIdx.y == 0;
    if (shared ? !a.Wsh : (int)blockIdx.y > a.active[0]) return;
    const int e = shared ? 0 : a.active[blockIdx.y];
    if (e < 0) return;
    const int N = shared ? a.Nsh : a.N, K = shared ? a.Ksh : a.K, ldw = shared ? a.ldwsh : a.ldw, n0 = blockIdx.x * 16;
    const int ldo = shared ? a.ldosh : a.ldo;
    if (n0 >= ldo) return;
    const uint16_t* W = shared ? a.Wsh : a.W + e * a.wstride;
    const int* list = a.list + (long)e * a.cap;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int li = lane & 15, lg = lane >> 4;
    const uint16_t* wp[NM];
#pragma unroll
    for (int q = 0; q < NM; ++q) wp[q] = W + ((long)q * N + min(n0 + li, N - 1)) * ldw;
    f32x4 acc[NM];
#pragma unroll
    for (int q = 0; q < NM; ++q) acc[q] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int nstep = (K + 63) / 64;
    uint4 w[U][NM][2];
    auto wload = [&](int s0) {
#pragma unroll
        for (int i = 0; i < U; ++i) {
            const int k = (s0 + 4 * i) * 64 + lg * 16;
#pragma unroll
            for (int h = 0; h < 2; ++h)
#pragma unroll
                for (int q = 0; q < NM; ++q) w[i][q][h] = ldg16_sel(wp[q] + k + 8 * h, k + 8 * h < K, wp[q]);
        }
    };
    wload(wave);  // in flight while the rows are looked up
    const int cnt = shared ? a.B : a.cnt[e];
    const int m = min(li, cnt - 1), row = shared ? m : list[m] / a.gather;
    const uint16_t* xp = reinterpret_cast<const uint16_t*>(shared ? a.Ash : a.A) + (long)row * (shared ? a.ldash : a.lda);
    for (int s0 = wave; s0 < nstep; s0 += 4 * U) {
        uint4 x[U][2];
#pragma unroll
        for (int i = 0; i < U; ++i) {
            const int k = (s0 + 4 * i) * 64 + lg * 16;
#pragma unroll
            for (int h = 0; h < 2; ++h) x[i][h] = ldg16_sel(xp + k + 8 * h, k + 8 * h < K, xp);
        }
#pragma unroll
        for (int i = 0; i < U; ++i)
#pragma unroll
            for (int h = 0; h < 2; ++h)
#pragma unroll
                for (int q = 0; q < NM; ++q)
                    acc[q] = mfma16(__builtin_bit_cast(short8, w[i][q][h]), __builtin_bit_cast(short8, x[i][h]), acc[q]);
        if (s0 + 4 * U < nstep) wload(s0 + 4 * U);
    }
#pragma unroll
    for (int q = 0; q < NM; ++q)
#pragma unroll
        for (int r = 0; r < 4; ++r) sums[wave][q][4 * lg + r][li] = acc[q][r];
    __syncthreads();
    const int b = tid >> 4, n = n0 + (tid & 15);  // consecutive threads store consecutive outputs
    float v[2] = {0.f, 0.f};
#pragma unroll
    for (int q = 0; q < NM; ++q)
#pragma unroll
        for (int u = 0; u < 4; ++u) v[q] += sums[u][q][tid & 15][b];
    if (b >= cnt || n >= ldo) return;
    if constexpr (MODE == EX_SWIGLU) v[0] = siluf_(v[0]) * v[1];
    if (n >= N) v[0] = 0.0f;
    const long o = (long)(shared ? b : list[b]) * ldo + n;
    if (MODE == EX_STORE && shared) reinterpret_cast<float*>(a.outsh)[o] = v[0];
    else reinterpret_cast<uint16_t*>(shared ? a.outsh : a.out)[o] = f2bf(v[0]);
}

}  // namespace

void route(hipStream_t s, const RouteArgs& a) {
    const int nw = a.rows >= 2048 ? 16 : 4;
    const size_t lds = ((size_t)nw * (route_words(a.n, a.groups) + 2 * a.top) + 2 * a.experts) * sizeof(float);
    if (lds > 60 * 1024)
        (void)hipFuncSetAttribute(reinterpret_cast<const void*>(&k_route), hipFuncAttributeMaxDynamicSharedMemorySize,
                                  (int)lds);
    hipLaunchKernelGGL(k_route, dim3((a.rows + nw - 1) / nw), dim3(64 * nw), lds, s, a);
}

void experts_rt(hipStream_t s, Act act, ExpertMode mode, const ExpertArgs& a) {
    if (act == ACT_F32) {
        const dim3 grid((unsigned)((max_tiles(a, FT) * ((a.ldo + FT - 1) / FT) + 7) / 8 * 8));
        if (mode == EX_SWIGLU) hipLaunchKernelGGL((k_experts_f32<EX_SWIGLU>), grid, dim3(256), 0, s, a);
        else hipLaunchKernelGGL((k_experts_f32<EX_STORE>), grid, dim3(256), 0, s, a);
        return;
    }
    const int per = a.entries / std::max(1, a.experts);  // rows of an average expert
    auto go = [&](auto mode_c) {
        constexpr int MODE = decltype(mode_c)::value;
        const bool p8 = a.K % 64 == 0 && a.K >= 512;
        if (p8 && per > 384) run_experts_8p<8, MODE>(s, a);
        else if (p8 && per > 128) run_experts_8p<6, MODE>(s, a);
        else if (per > 96) run_experts<4, MODE>(s, a);
        else if (per > 32) run_experts<2, MODE>(s, a);
        else run_experts<1, MODE>(s, a);
    };
    if (mode == EX_SWIGLU) go(std::integral_constant<int, EX_SWIGLU>{});
    else go(std::integral_constant<int, EX_STORE>{});
}

void experts_skinny(hipStream_t s, ExpertMode mode, const ExpertArgs& a) {
    const int n = std::max(a.ldo, a.Wsh ? a.ldosh : 0);
    // one row lists its choices by place, identities included
    const dim3 grid((n + 15) / 16, 1 + (a.B == 1 ? a.entries : std::min(a.experts, a.entries)));
    // one row has too few workgroups to cover the memory's latency with four steps: 25.0 -> 20.5 us (width 2048, 6 + 1
    // experts); with more rows, or the shorter rows of the down product, eight are slower
    if (mode == EX_SWIGLU && a.B == 1) hipLaunchKernelGGL((k_experts_skinny<EX_SWIGLU, 8>), grid, dim3(256), 0, s, a);
    else if (mode == EX_SWIGLU) hipLaunchKernelGGL((k_experts_skinny<EX_SWIGLU, 4>), grid, dim3(256), 0, s, a);
    else hipLaunchKernelGGL((k_experts_skinny<EX_STORE, 4>), grid, dim3(256), 0, s, a);
}

}  // namespace pgmi
