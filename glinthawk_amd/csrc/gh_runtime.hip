// Runtime half of libglint_hip.so: device selection, error text, allocation and copies, the
// staging ring for host-side tables, the paged (virtual-memory) KV arena and the event-based
// kernel timer used by the benchmark.
#include "gh_common.h"

#include <algorithm>
#include <atomic>
#include <cstdarg>
#include <mutex>
#include <vector>

namespace gh {

namespace {

thread_local char g_error[512] = "";

std::mutex g_mutex;
bool g_ready = false;
int g_device = -1;
int g_cu_count = 256; // compute units of the initialised device (a full MI355X: 256)
char g_arch[128] = "";

// ---- staging ring ------------------------------------------------------------------------------
constexpr int STAGE_SLOTS = 64;
constexpr int STAGE_LOOKBACK = 8; // how many of the most recently written slots are searched for an identical table
struct StageSlot
{
  char* pinned = nullptr;
  char* device = nullptr;
  hipEvent_t done = nullptr;
  bool in_flight = false;        // `done` has been recorded behind work that reads the slot
  bool staged = false;           // handed out since the last fence on `stream`: must not be rewritten yet
  hipStream_t stream = nullptr;  // stream of the copy that filled the slot
  size_t bytes = 0;              // 0: never written
};
StageSlot g_slots[STAGE_SLOTS];
int g_next_slot = 0;

// ---- grow-only device buffers, one per (stream, purpose) ------------------------------------------
struct ScratchBuffer
{
  hipStream_t stream;
  int which;
  void* ptr;
  uint64_t bytes;
};
std::vector<ScratchBuffer> g_scratch;

// every allocation this library makes (device, page-locked host, physical blocks of the paged arena), for gh_allocation_count()
std::atomic<uint64_t> g_allocations { 0 };

// ---- attention kernel timer ----------------------------------------------------------------
constexpr int TIMER_SLOTS = 8192;
int g_timing = 0; // 0 off; 1 events in front of, between and behind the two kernels; 2 only in front of and behind the pair
std::vector<hipEvent_t> g_events; // 3 per slot
int g_ev_used = 0;

} // namespace

void set_error( const char* fmt, ... )
{
  va_list ap;
  va_start( ap, fmt );
  vsnprintf( g_error, sizeof( g_error ), fmt, ap );
  va_end( ap );
}

int fail( int status, const char* fmt, ... )
{
  va_list ap;
  va_start( ap, fmt );
  vsnprintf( g_error, sizeof( g_error ), fmt, ap );
  va_end( ap );
  return status;
}

// The GEMM kernels bound their buffer loads by the descriptor's size and put row and
// K offsets into the scalar offset operand, including offsets that are meant to fall outside.  That
// is only safe if the scalar offset takes part in the hardware's range check (it does on gfx950;
// the compiler's contract for the intrinsic does not promise it), so initialisation checks it once
// on memory where either answer is harmless.
__global__ void buffer_bounds_probe_kernel( const uint32_t* buf, uint32_t* out, uint32_t scalar_offset )
{
  const __amdgpu_buffer_rsrc_t rsrc = __builtin_amdgcn_make_buffer_rsrc( const_cast<uint32_t*>( buf ), 0, 1024, 0x00020000 );
  const uint32_t so = __builtin_amdgcn_readfirstlane( scalar_offset );
  out[threadIdx.x] = __builtin_amdgcn_raw_buffer_load_b32( rsrc, threadIdx.x * 4, so, 0 );
}

int check_buffer_bounds()
{
  uint32_t* buf = nullptr;
  GH_HIP( hipMalloc( reinterpret_cast<void**>( &buf ), 4096 + 64 * 4 ) );
  g_allocations++;
  uint32_t* out = buf + 1024;
  GH_HIP( hipMemset( buf, 0x5a, 4096 + 64 * 4 ) );
  buffer_bounds_probe_kernel<<<1, 64>>>( buf, out, 2048 ); // descriptor: 1024 bytes; the loads land at 2048.. of a 4096-byte block
  GH_HIP( hipGetLastError() );
  uint32_t host[64];
  GH_HIP( hipMemcpy( host, out, sizeof( host ), hipMemcpyDeviceToHost ) );
  GH_HIP( hipFree( buf ) );
  for ( uint32_t v : host ) {
    if ( v != 0 ) {
      return fail( GH_ERR_DEVICE, "this device does not range-check the scalar offset of buffer loads; the kernels of this library rely on it" );
    }
  }
  return GH_OK;
}

static int init_locked( int device )
{
  int count = 0;
  hipError_t err = hipGetDeviceCount( &count );
  if ( err != hipSuccess || count == 0 ) {
    (void)hipGetLastError();
    return fail( GH_ERR_NO_DEVICE, "no HIP device visible (%s)", err == hipSuccess ? "count is 0" : hipGetErrorString( err ) );
  }
  if ( device < 0 || device >= count ) {
    return fail( GH_ERR_INVALID, "device %d out of range (0..%d)", device, count - 1 );
  }
  GH_HIP( hipSetDevice( device ) );
  hipDeviceProp_t prop;
  GH_HIP( hipGetDeviceProperties( &prop, device ) );
  snprintf( g_arch, sizeof( g_arch ), "%s", prop.gcnArchName );
  if ( strncmp( prop.gcnArchName, "gfx950", 6 ) != 0 ) {
    return fail( GH_ERR_NO_DEVICE, "device %d is %s; this library holds gfx950 code only", device, prop.gcnArchName );
  }
  if ( int rc = check_buffer_bounds() ) {
    return rc;
  }
  if ( attn_static_scratch_init != nullptr ) {
    if ( int rc = attn_static_scratch_init( device ) ) {
      return rc;
    }
  }
  for ( int i = 0; i < STAGE_SLOTS; i++ ) {
    GH_HIP( hipHostMalloc( reinterpret_cast<void**>( &g_slots[i].pinned ), STAGE_SLOT_BYTES, hipHostMallocDefault ) );
    GH_HIP( hipMalloc( reinterpret_cast<void**>( &g_slots[i].device ), STAGE_SLOT_BYTES ) );
    g_allocations += 2;
    GH_HIP( hipEventCreateWithFlags( &g_slots[i].done, hipEventDisableTiming ) );
  }
  g_device = device;
  g_cu_count = prop.multiProcessorCount > 0 ? prop.multiProcessorCount : 256;
  g_ready = true;
  return GH_OK;
}

int cu_count() { return g_cu_count; }

int initialised_device()
{
  std::lock_guard<std::mutex> lock( g_mutex );
  return g_ready ? g_device : -1;
}

int ensure_init()
{
  std::lock_guard<std::mutex> lock( g_mutex );
  if ( g_ready ) {
    return GH_OK;
  }
  return init_locked( 0 );
}

int stage_table( const void* host_src, size_t bytes, hipStream_t stream, void** dev_out )
{
  GH_REQUIRE( bytes > 0 && bytes <= STAGE_SLOT_BYTES, "table of %zu bytes does not fit a staging slot (%zu)", bytes, STAGE_SLOT_BYTES );
  std::lock_guard<std::mutex> lock( g_mutex );
  // The ops of one layer pass the same position and row tables again and again: a table that one of
  // the last few slots already holds, copied on this same stream, is handed out again without a copy.
  for ( int back = 1; back <= STAGE_LOOKBACK; back++ ) {
    StageSlot& old = g_slots[( g_next_slot + STAGE_SLOTS - back ) % STAGE_SLOTS];
    if ( old.bytes == bytes && old.stream == stream && memcmp( old.pinned, host_src, bytes ) == 0 ) {
      old.staged = true;
      *dev_out = old.device;
      return GH_OK;
    }
  }
  int idx = -1;
  for ( int tries = 0; tries < STAGE_SLOTS; tries++ ) {
    const int cand = ( g_next_slot + tries ) % STAGE_SLOTS;
    if ( !g_slots[cand].staged ) {
      idx = cand;
      break;
    }
  }
  if ( idx < 0 ) {
    return fail( GH_ERR_INVALID, "all %d staging slots are handed out and unfenced", STAGE_SLOTS );
  }
  StageSlot& slot = g_slots[idx];
  if ( slot.in_flight ) {
    GH_HIP( hipEventSynchronize( slot.done ) );
    slot.in_flight = false;
  }
  slot.bytes = 0;
  memcpy( slot.pinned, host_src, bytes );
  GH_HIP( hipMemcpyAsync( slot.device, slot.pinned, bytes, hipMemcpyHostToDevice, stream ) );
  slot.bytes = bytes;
  slot.stream = stream;
  slot.staged = true;
  g_next_slot = ( idx + 1 ) % STAGE_SLOTS;
  *dev_out = slot.device;
  return GH_OK;
}

int stage_fence( hipStream_t stream )
{
  std::lock_guard<std::mutex> lock( g_mutex );
  int rc = GH_OK;
  for ( StageSlot& slot : g_slots ) {
    if ( slot.staged && slot.stream == stream ) {
      slot.staged = false;
      const hipError_t err = hipEventRecord( slot.done, stream );
      if ( err != hipSuccess ) {
        slot.bytes = 0; // never hand this content out again; the next writer finds the slot idle
        rc = fail( GH_ERR_DEVICE, "hipEventRecord failed: %s", hipGetErrorString( err ) );
      } else {
        slot.in_flight = true;
      }
    }
  }
  return rc;
}

int stream_scratch( hipStream_t stream, int which, uint64_t bytes, uint64_t min_bytes, void** out )
{
  std::lock_guard<std::mutex> lock( g_mutex );
  ScratchBuffer* buf = nullptr;
  for ( auto& b : g_scratch ) {
    if ( b.stream == stream && b.which == which ) {
      buf = &b;
    }
  }
  if ( buf == nullptr ) {
    g_scratch.push_back( { stream, which, nullptr, 0 } );
    buf = &g_scratch.back();
  }
  if ( bytes > buf->bytes ) {
    if ( buf->ptr ) {
      GH_HIP( hipStreamSynchronize( stream ) ); // only work queued on this stream reads the buffer
      GH_HIP( hipFree( buf->ptr ) );
      buf->ptr = nullptr;
      buf->bytes = 0;
    }
    const uint64_t want = std::max( bytes, min_bytes );
    GH_HIP( hipMalloc( &buf->ptr, want ) );
    g_allocations++;
    buf->bytes = want;
  }
  *out = buf->ptr;
  return GH_OK;
}

// timer hook used by gh_attn_decode: which = 0 claims a slot and records its first event
int timer_mark( hipStream_t stream, int* slot_inout, int which )
{
  if ( which == 0 ) {
    *slot_inout = -1;
    if ( !g_timing ) {
      return GH_OK;
    }
    std::lock_guard<std::mutex> lock( g_mutex );
    if ( g_ev_used >= TIMER_SLOTS ) {
      return GH_OK; // stop sampling; the mean over the recorded calls stays valid
    }
    if ( (int)g_events.size() < 3 * ( g_ev_used + 1 ) ) {
      for ( int k = 0; k < 3; k++ ) {
        hipEvent_t e;
        GH_HIP( hipEventCreate( &e ) );
        g_events.push_back( e );
      }
    }
    *slot_inout = g_ev_used++;
  }
  if ( *slot_inout < 0 ) {
    return GH_OK;
  }
  if ( which == 1 && g_timing == 2 ) {
    return GH_OK; // the pair as it runs in production: nothing between the two kernels
  }
  GH_HIP( hipEventRecord( g_events[3 * ( *slot_inout ) + which], stream ) );
  return GH_OK;
}

namespace {
bool copy_kind( gh_copy_kind kind, hipMemcpyKind* out )
{
  switch ( kind ) {
    case GH_HOST_TO_DEVICE: *out = hipMemcpyHostToDevice; return true;
    case GH_DEVICE_TO_HOST: *out = hipMemcpyDeviceToHost; return true;
    case GH_DEVICE_TO_DEVICE: *out = hipMemcpyDeviceToDevice; return true;
    case GH_HOST_TO_HOST: *out = hipMemcpyHostToHost; return true;
    default: return false;
  }
}
} // namespace
} // namespace gh

using namespace gh;

extern "C" {

int gh_init( int device )
{
  std::lock_guard<std::mutex> lock( g_mutex );
  if ( g_ready ) {
    if ( device != g_device ) {
      return fail( GH_ERR_INVALID, "already initialised on device %d", g_device );
    }
    return GH_OK;
  }
  return init_locked( device );
}

const char* gh_last_error( void ) { return g_error; }

int gh_device_name( char* out, size_t len )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  snprintf( out, len, "%s", g_arch );
  return GH_OK;
}

int gh_stream_create( gh_stream* out )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  GH_REQUIRE( out != nullptr, "gh_stream_create: NULL output" );
  hipStream_t s = nullptr;
  GH_HIP( hipStreamCreateWithFlags( &s, hipStreamNonBlocking ) ); // default priority
  *out = s;
  return GH_OK;
}

int gh_stream_destroy( gh_stream stream )
{
  GH_REQUIRE( stream != nullptr, "gh_stream_destroy: the default stream is not the caller's" );
  hipStream_t st = as_stream( stream );
  GH_HIP( hipStreamSynchronize( st ) );
  {
    // What the library keeps for this stream goes with it: the grow-only scratch buffers (nothing queued reads them after the
    // synchronise above) and the staging slots' memory of having been filled on it -- a later stream may get the same handle
    // value and must neither inherit the buffers' contents nor be handed a table that was copied on the old stream.
    std::lock_guard<std::mutex> lock( g_mutex );
    for ( size_t i = 0; i < g_scratch.size(); ) {
      if ( g_scratch[i].stream == st ) {
        if ( g_scratch[i].ptr != nullptr ) {
          GH_HIP( hipFree( g_scratch[i].ptr ) );
        }
        g_scratch.erase( g_scratch.begin() + (long)i );
      } else {
        i++;
      }
    }
    for ( StageSlot& slot : g_slots ) {
      if ( slot.stream == st ) {
        slot.stream = nullptr;
        slot.bytes = 0;
        slot.staged = false;
        slot.in_flight = false; // its event, if recorded, lies behind the synchronise above
      }
    }
  }
  GH_HIP( hipStreamDestroy( st ) );
  return GH_OK;
}

int gh_event_create( gh_event* out )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  GH_REQUIRE( out != nullptr, "gh_event_create: NULL output" );
  hipEvent_t e = nullptr;
  GH_HIP( hipEventCreateWithFlags( &e, hipEventDisableTiming ) );
  *out = e;
  return GH_OK;
}

int gh_event_create_timed( gh_event* out )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  GH_REQUIRE( out != nullptr, "gh_event_create_timed: NULL output" );
  hipEvent_t e = nullptr;
  GH_HIP( hipEventCreate( &e ) );
  *out = e;
  return GH_OK;
}

int gh_event_elapsed_ms( gh_event begin, gh_event end, float* ms )
{
  GH_REQUIRE( begin != nullptr && end != nullptr && ms != nullptr, "gh_event_elapsed_ms: NULL argument" );
  GH_HIP( hipEventSynchronize( static_cast<hipEvent_t>( end ) ) );
  GH_HIP( hipEventElapsedTime( ms, static_cast<hipEvent_t>( begin ), static_cast<hipEvent_t>( end ) ) );
  return GH_OK;
}

int gh_event_destroy( gh_event event )
{
  GH_REQUIRE( event != nullptr, "gh_event_destroy: NULL event" );
  GH_HIP( hipEventDestroy( static_cast<hipEvent_t>( event ) ) );
  return GH_OK;
}

int gh_event_record( gh_event event, gh_stream stream )
{
  GH_REQUIRE( event != nullptr, "gh_event_record: NULL event" );
  GH_HIP( hipEventRecord( static_cast<hipEvent_t>( event ), as_stream( stream ) ) );
  return GH_OK;
}

int gh_stream_wait_event( gh_stream stream, gh_event event )
{
  GH_REQUIRE( event != nullptr, "gh_stream_wait_event: NULL event" );
  GH_HIP( hipStreamWaitEvent( as_stream( stream ), static_cast<hipEvent_t>( event ), 0 ) );
  return GH_OK;
}

int gh_sync( gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  if ( stream == nullptr ) {
    GH_HIP( hipDeviceSynchronize() );
  } else {
    GH_HIP( hipStreamSynchronize( as_stream( stream ) ) );
  }
  return GH_OK;
}

int gh_malloc( void** out, uint64_t bytes )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  GH_REQUIRE( out != nullptr, "gh_malloc: out is NULL" );
  *out = nullptr;
  if ( bytes == 0 ) {
    return GH_OK;
  }
  GH_HIP( hipMalloc( out, bytes ) );
  g_allocations++;
  return GH_OK;
}

uint64_t gh_allocation_count( void ) { return g_allocations.load(); }

int gh_free( void* ptr )
{
  if ( ptr != nullptr ) {
    GH_HIP( hipFree( ptr ) );
  }
  return GH_OK;
}

int gh_host_malloc( void** out, uint64_t bytes )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  GH_REQUIRE( out != nullptr, "gh_host_malloc: out is NULL" );
  *out = nullptr;
  if ( bytes == 0 ) {
    return GH_OK;
  }
  GH_HIP( hipHostMalloc( out, bytes, hipHostMallocDefault ) );
  g_allocations++;
  return GH_OK;
}

int gh_host_free( void* ptr )
{
  if ( ptr != nullptr ) {
    GH_HIP( hipHostFree( ptr ) );
  }
  return GH_OK;
}

int gh_memcpy( void* dst, const void* src, uint64_t bytes, gh_copy_kind kind, int async, gh_stream stream )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  if ( bytes == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( dst != nullptr && src != nullptr, "gh_memcpy: NULL pointer" );
  hipMemcpyKind k;
  GH_REQUIRE( copy_kind( kind, &k ), "gh_memcpy: bad copy kind %d", (int)kind );
  GH_HIP( hipMemcpyAsync( dst, src, bytes, k, as_stream( stream ) ) );
  if ( !async ) {
    GH_HIP( hipStreamSynchronize( as_stream( stream ) ) );
  }
  return GH_OK;
}

int gh_memcpy_rows( void* dst, uint64_t dst_stride, const void* src, uint64_t src_stride, uint64_t bytes, uint64_t rows, gh_copy_kind kind, gh_stream stream )
{
  if ( dst_stride == bytes && src_stride == bytes ) {
    return gh_memcpy( dst, src, bytes * rows, kind, 0, stream );
  }
  if ( int rc = ensure_init() ) {
    return rc;
  }
  if ( bytes == 0 || rows == 0 ) {
    return GH_OK;
  }
  GH_REQUIRE( dst != nullptr && src != nullptr && dst_stride >= bytes && src_stride >= bytes, "gh_memcpy_rows: bad argument" );
  hipMemcpyKind k;
  GH_REQUIRE( copy_kind( kind, &k ), "gh_memcpy_rows: bad copy kind %d", (int)kind );
  GH_HIP( hipMemcpy2DAsync( dst, dst_stride, src, src_stride, bytes, rows, k, as_stream( stream ) ) );
  GH_HIP( hipStreamSynchronize( as_stream( stream ) ) );
  return GH_OK;
}

// ---- paged arena ------------------------------------------------------------------------------
struct gh_vmm
{
  void* base = nullptr;
  uint64_t len = 0;
  uint64_t granularity = 0;
  struct Span
  {
    uint64_t offset;
    uint64_t len;
    hipMemGenericAllocationHandle_t handle;
  };
  std::vector<Span> spans;
  uint64_t committed = 0;
};

static int vmm_props( hipMemAllocationProp* prop )
{
  memset( prop, 0, sizeof( *prop ) );
  prop->type = hipMemAllocationTypePinned;
  prop->location.type = hipMemLocationTypeDevice;
  int dev = 0;
  GH_HIP( hipGetDevice( &dev ) );
  prop->location.id = dev;
  return GH_OK;
}

int gh_vmm_granularity( uint64_t* out )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  hipMemAllocationProp prop;
  if ( int rc = vmm_props( &prop ) ) {
    return rc;
  }
  size_t g = 0;
  GH_HIP( hipMemGetAllocationGranularity( &g, &prop, hipMemAllocationGranularityMinimum ) );
  *out = g;
  return GH_OK;
}

int gh_vmm_reserve( gh_vmm** out, uint64_t bytes )
{
  if ( int rc = ensure_init() ) {
    return rc;
  }
  GH_REQUIRE( out != nullptr && bytes > 0, "gh_vmm_reserve: bad arguments" );
  uint64_t gran = 0;
  if ( int rc = gh_vmm_granularity( &gran ) ) {
    return rc;
  }
  const uint64_t rounded = ( bytes + gran - 1 ) / gran * gran;
  void* base = nullptr;
  GH_HIP( hipMemAddressReserve( &base, rounded, 0, nullptr, 0 ) );
  gh_vmm* r = new gh_vmm;
  r->base = base;
  r->len = rounded;
  r->granularity = gran;
  *out = r;
  return GH_OK;
}

void* gh_vmm_ptr( const gh_vmm* r ) { return r ? r->base : nullptr; }
uint64_t gh_vmm_max_len( const gh_vmm* r ) { return r ? r->len : 0; }
uint64_t gh_vmm_committed_bytes( const gh_vmm* r ) { return r ? r->committed : 0; }

int gh_vmm_commit( gh_vmm* r, uint64_t offset, uint64_t len )
{
  GH_REQUIRE( r != nullptr, "gh_vmm_commit: NULL region" );
  GH_REQUIRE( len > 0 && offset + len <= r->len, "gh_vmm_commit: span [%llu, +%llu) outside the %llu-byte region",
              (unsigned long long)offset, (unsigned long long)len, (unsigned long long)r->len );
  GH_REQUIRE( offset % r->granularity == 0 && len % r->granularity == 0,
              "gh_vmm_commit: span must be a multiple of the %llu-byte granularity", (unsigned long long)r->granularity );
  hipMemAllocationProp prop;
  if ( int rc = vmm_props( &prop ) ) {
    return rc;
  }
  hipMemGenericAllocationHandle_t handle;
  GH_HIP( hipMemCreate( &handle, len, &prop, 0 ) );
  g_allocations++;
  void* at = static_cast<char*>( r->base ) + offset;
  hipError_t err = hipMemMap( at, len, 0, handle, 0 );
  if ( err != hipSuccess ) {
    (void)hipMemRelease( handle );
    return fail( GH_ERR_DEVICE, "hipMemMap failed: %s", hipGetErrorString( err ) );
  }
  hipMemAccessDesc access;
  memset( &access, 0, sizeof( access ) );
  access.location = prop.location;
  access.flags = hipMemAccessFlagsProtReadWrite;
  err = hipMemSetAccess( at, len, &access, 1 );
  if ( err != hipSuccess ) {
    (void)hipMemUnmap( at, len );
    (void)hipMemRelease( handle );
    return fail( GH_ERR_DEVICE, "hipMemSetAccess failed: %s", hipGetErrorString( err ) );
  }
  r->spans.push_back( { offset, len, handle } );
  r->committed += len;
  return GH_OK;
}

int gh_vmm_clear( gh_vmm* r )
{
  GH_REQUIRE( r != nullptr, "gh_vmm_clear: NULL region" );
  for ( auto& s : r->spans ) {
    GH_HIP( hipMemUnmap( static_cast<char*>( r->base ) + s.offset, s.len ) );
    GH_HIP( hipMemRelease( s.handle ) );
  }
  r->spans.clear();
  r->committed = 0;
  return GH_OK;
}

int gh_vmm_free( gh_vmm* r )
{
  if ( r == nullptr ) {
    return GH_OK;
  }
  if ( int rc = gh_vmm_clear( r ) ) {
    return rc;
  }
  GH_HIP( hipMemAddressFree( r->base, r->len ) );
  delete r;
  return GH_OK;
}

// ---- kernel timer ------------------------------------------------------------------------------
int gh_attn_timing_enable( int on )
{
  std::lock_guard<std::mutex> lock( g_mutex );
  g_timing = on == 2 ? 2 : ( on != 0 ? 1 : 0 );
  return GH_OK;
}

int gh_attn_timing_reset( void )
{
  std::lock_guard<std::mutex> lock( g_mutex );
  g_ev_used = 0;
  return GH_OK;
}

int gh_attn_timing_read( double* kernel_ms, double* merge_ms, uint64_t* launches )
{
  std::lock_guard<std::mutex> lock( g_mutex );
  double k_total = 0.0, m_total = 0.0;
  for ( int i = 0; i < g_ev_used; i++ ) {
    GH_HIP( hipEventSynchronize( g_events[3 * i + 2] ) );
    float ms = 0.0f;
    if ( g_timing == 2 ) { // one span per call
      GH_HIP( hipEventElapsedTime( &ms, g_events[3 * i], g_events[3 * i + 2] ) );
      k_total += ms;
      continue;
    }
    GH_HIP( hipEventElapsedTime( &ms, g_events[3 * i], g_events[3 * i + 1] ) );
    k_total += ms;
    GH_HIP( hipEventElapsedTime( &ms, g_events[3 * i + 1], g_events[3 * i + 2] ) );
    m_total += ms;
  }
  if ( kernel_ms ) {
    *kernel_ms = k_total;
  }
  if ( merge_ms ) {
    *merge_ms = m_total;
  }
  if ( launches ) {
    *launches = (uint64_t)g_ev_used;
  }
  return GH_OK;
}

} // extern "C"
