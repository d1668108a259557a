// Device time of a model driver's forward(): the span on the stream from the first kernel of a step to its last, without the copies of
// the state over the host boundary on either side.  Off by default; two event records per step when on.
#pragma once

#include <cstdint>
#include <memory>
#include <utility>

#include "glint/hip/ops.hh"

namespace glint {

class DeviceSpans
{
  struct Timer
  {
    gh_event mark[2] {};
    double total_ms { 0 };
    uint64_t spans { 0 };
    bool open { false };
    Timer()
    {
      GLINT_GH( gh_event_create_timed( &mark[0] ) );
      GLINT_GH( gh_event_create_timed( &mark[1] ) );
    }
    ~Timer()
    {
      (void)gh_event_destroy( mark[0] );
      (void)gh_event_destroy( mark[1] );
    }
    Timer( const Timer& ) = delete;
    Timer& operator=( const Timer& ) = delete;
  };
  std::unique_ptr<Timer> timer_ {};

public:
  void enable( const bool on )
  {
    if ( on && !timer_ ) {
      timer_ = std::make_unique<Timer>();
    } else if ( !on ) {
      timer_.reset();
    }
  }
  // the accumulated milliseconds and steps, which a read resets
  std::pair<double, uint64_t> take()
  {
    std::pair<double, uint64_t> out { 0.0, 0 };
    if ( timer_ ) {
      out = { timer_->total_ms, timer_->spans };
      timer_->total_ms = 0;
      timer_->spans = 0;
    }
    return out;
  }
  // 0 in front of the first kernel, 1 behind the last
  void mark( const int which, const gh_stream stream )
  {
    if ( timer_ ) {
      GLINT_GH( gh_event_record( timer_->mark[which], stream ) );
      timer_->open = which == 1;
    }
  }
  // once the step is over
  void close()
  {
    if ( timer_ && timer_->open ) {
      float ms = 0;
      GLINT_GH( gh_event_elapsed_ms( timer_->mark[0], timer_->mark[1], &ms ) );
      timer_->total_ms += ms;
      timer_->spans++;
      timer_->open = false;
    }
  }
};

} // namespace glint
